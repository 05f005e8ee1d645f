"""Models by name: config.json -> the class that builds a decoder over a paged pool.

A model folder holds config.json and *.safetensors.  `architecture` (or the first of `architectures`, or `model_type`) names the
model; load_decoder() returns an object with the interface BatchScheduler drives (prefill, prefill_batch, decode, greedy, .pool).
Register another design with @register("Name").
"""
from __future__ import annotations

import json
import os
from typing import Callable, Dict, Optional

import torch

from .weights import load_checkpoint

DTYPES = {"bfloat16": torch.bfloat16, "float16": torch.float16, "float32": torch.float32}


class UnsupportedDtype(ValueError):
    """The model is not served in the element type asked for."""


_BUILDERS: Dict[str, Callable] = {}


def register(*names: str):
    def wrap(fn):
        for n in names:
            _BUILDERS[n] = fn
        return fn
    return wrap


def architectures():
    return sorted(_BUILDERS)


def read_config(model_dir: str) -> dict:
    with open(os.path.join(model_dir, "config.json")) as f:
        return json.load(f)


def architecture_of(config: dict) -> str:
    for name in (config.get("architecture"), *(config.get("architectures") or ()), config.get("model_type")):
        if name in _BUILDERS:
            return name
    raise ValueError(f"config.json names no known architecture (known: {', '.join(architectures())})")


def load_decoder(model_dir: str, *, dtype: Optional[str] = None, max_tokens: int, max_seqs: int, max_length: Optional[int] = None,
                 device="cuda:0", **decoder_kw):
    """The decoder of a model folder over a pool of max_tokens tokens and max_seqs live sequences.  dtype: None = what the model
    is served in."""
    config = read_config(model_dir)
    name = architecture_of(config)
    if dtype is not None and dtype not in DTYPES:
        raise UnsupportedDtype(f"unknown element type {dtype}")
    dev = torch.device(device)
    return _BUILDERS[name](config, lambda: load_checkpoint(model_dir), None if dtype is None else DTYPES[dtype], dev,
                           max_tokens=max_tokens, max_seqs=max_seqs, max_length=max_length, **decoder_kw)


def _hybrid(name, config_class, build_model, config, tensors, dtype, device, *, max_tokens, max_seqs, max_length=None, page_size=64, **kw):
    from .hybrid_decoder import HybridDecoder

    dtype = dtype or torch.bfloat16
    if dtype not in (torch.bfloat16, torch.float32):
        raise UnsupportedDtype(f"{name} is built for bfloat16 and float32, not {dtype}")
    model = build_model(config_class.from_json(config), tensors(), dtype, device)
    return HybridDecoder(model, model.make_pool(max_tokens, max_seqs, page_size, max_length), **kw)


@register("Voduvik")
def _voduvik(config, *args, **kw):
    from .voduvik import VoduvikConfig, build_model

    return _hybrid("Voduvik", VoduvikConfig, build_model, config, *args, **kw)


@register("Fetelorn")
def _fetelorn(config, *args, **kw):
    from .fetelorn import FetelornConfig, build_model

    return _hybrid("Fetelorn", FetelornConfig, build_model, config, *args, **kw)


@register("GPT2LMHeadModel", "gpt2")
def _gpt2(config, tensors, dtype, device, *, max_tokens, max_seqs, max_length=None, page_size=16, **kw):
    from .gpt2_decode import GPT2Dims, GPT2PagedDecoder
    from .kv_pool import PagedKVPool

    dtype = dtype or torch.float16
    if dtype != torch.float16:
        raise UnsupportedDtype(f"GPT-2 is served in float16, not {dtype}")
    d = GPT2Dims(**{k: config[k] for k in ("vocab_size", "n_positions", "n_embd", "n_layer", "n_head", "layer_norm_epsilon",
                                           "eos_token_id") if k in config})
    per_seq = -(-min(max_length or d.n_positions, d.n_positions) // page_size)
    pool = PagedKVPool(max(1, max_tokens // page_size) * d.n_layer, d.n_head, d.head_size, page_size, per_seq + 1, d.n_layer,
                       device=device, max_seqs=max_seqs)
    sd = {k: t.to(device, dtype) for k, t in tensors().items()}
    if "lm_head.weight" not in sd:
        sd["lm_head.weight"] = sd["transformer.wte.weight"]         # tied
    return GPT2PagedDecoder(d, sd, pool, **kw)
