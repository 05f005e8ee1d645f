"""The Voduvik decoder: its configuration and the construction of its layers (hybrid_layers) from a checkpoint's tensors.

A list of layers, each a recurrent block ("rglru") or latent attention ("latent_attention") with an optional clamped gated
feed-forward; a stretch of the layers may run several times, with W_in [x ; embedding] in front of every pass.  All sizes come
from config.json; every layer may have its own.
"""
from __future__ import annotations

import dataclasses
from typing import Dict, List, Optional, Tuple

import torch

from .hybrid_decoder import HybridModel, LayerRun
from .hybrid_layers import ClampedGLU, ConcatProjection, Head, LatentAttention, Norm, RGLRU, spread
from .hybrid_ops import pad32


@dataclasses.dataclass(frozen=True)
class VoduvikConfig:
    vocab: int
    width: int
    layers: Tuple[dict, ...]
    norm_eps: float
    embedding_scale: float
    logit_scale: float
    loop: Optional[Tuple[int, int, int]] = None     # start, stop, times

    @classmethod
    def from_json(cls, c: dict) -> "VoduvikConfig":
        loop = c.get("loop")
        cfg = cls(vocab=int(c["vocab"]), width=int(c["width"]), layers=tuple(c["layers"]), norm_eps=float(c["norm"]["eps"]),
                  embedding_scale=float(c["embedding"]["scale"]), logit_scale=float(c["logit_scale"]),
                  loop=(int(loop["start"]), int(loop["stop"]), int(loop["times"])) if loop else None)
        for i, layer in enumerate(cfg.layers):
            if layer["type"] not in ("rglru", "latent_attention"):
                raise ValueError(f"layer {i}: unknown mixer {layer['type']!r}")
            if layer.get("mlp") is not None and layer["mlp"].get("kind") != "dense":
                raise ValueError(f"layer {i}: unknown feed-forward {layer['mlp'].get('kind')!r}")
        if cfg.loop is not None and not (0 <= cfg.loop[0] < cfg.loop[1] <= len(cfg.layers) and cfg.loop[2] >= 1):
            raise ValueError(f"loop {cfg.loop} does not lie inside {len(cfg.layers)} layers")
        return cfg

    def order(self) -> List[Tuple[int, bool]]:
        """(layer, does a pass of the loop begin here) in running order."""
        n = len(self.layers)
        if self.loop is None:
            return [(i, False) for i in range(n)]
        start, stop, times = self.loop
        once = [(i, i == start) for i in range(start, stop)]
        return [(i, False) for i in range(start)] + times * once + [(i, False) for i in range(stop, n)]

    def tensor_shapes(self) -> Dict[str, Tuple[int, ...]]:
        E = self.width
        out: Dict[str, Tuple[int, ...]] = {"embed": (self.vocab, E), "head": (self.vocab, E), "final.norm": (E,)}
        if self.loop is not None:
            out["loop.in"] = (E, 2 * E)
        for i, layer in enumerate(self.layers):
            p, m = f"l{i}.mix.", layer["mixer"]
            out[f"l{i}.norm1"] = (E,)
            if layer["type"] == "rglru":
                W, b = m["width"], m["blocks"]
                out.update({p + "y": (W, E), p + "y.b": (W,), p + "x": (W, E), p + "x.b": (W,), p + "conv": (W, m["conv"]),
                            p + "conv.b": (W,), p + "ra": (b, W // b, W // b), p + "ra.b": (b, W // b), p + "ri": (b, W // b, W // b),
                            p + "ri.b": (b, W // b), p + "lam": (W,), p + "o": (E, W)})
            else:
                H = m["heads"]
                out.update({p + "q": (H * (m["dim"] + m["rot_dim"]), E), p + "dkv": (m["kv_rank"] + m["rot_dim"], E),
                            p + "dkv.norm": (m["kv_rank"],), p + "uk": (H * m["dim"], m["kv_rank"]), p + "uv": (H * m["vdim"], m["kv_rank"]),
                            p + "g": (H, E), p + "o": (E, H * m["vdim"])})
            if layer.get("mlp") is not None:
                ff = layer["mlp"]["ff"]
                out.update({f"l{i}.norm2": (E,), f"l{i}.mlp.gate": (ff, E), f"l{i}.mlp.up": (ff, E), f"l{i}.mlp.down": (E, ff)})
        return out


def random_tensors(cfg: VoduvikConfig, device, seed: int = 0) -> Dict[str, torch.Tensor]:
    """Random bfloat16 weights of a configuration, scaled so that activations keep their size (no checkpoint exists)."""
    g = torch.Generator(device=device).manual_seed(seed)
    out = {}
    for name, shape in cfg.tensor_shapes().items():
        t = torch.randn(shape, generator=g, device=device)
        if name.endswith("norm") or name.endswith("norm1") or name.endswith("norm2"):
            t = 1 + 0.1 * t
        elif name.endswith(".lam"):
            t = t - 3.0              # decays of a few to a few hundred tokens
        elif name == "embed":
            t = t / cfg.embedding_scale
        elif len(shape) >= 2:
            t = t * shape[-1] ** -0.5
        else:
            t = 0.1 * t
        out[name] = t.to(torch.bfloat16)
    return out


def build_model(cfg: VoduvikConfig, tensors: Dict[str, torch.Tensor], dtype: torch.dtype, device) -> HybridModel:
    device = torch.device(device)
    for name, shape in cfg.tensor_shapes().items():
        if name not in tensors:
            raise KeyError(f"the checkpoint lacks {name}")
        if tuple(tensors[name].shape) != tuple(shape):
            raise ValueError(f"{name} has shape {tuple(tensors[name].shape)}, the configuration says {tuple(shape)}")
    w = {k: t.to(device) for k, t in tensors.items()}
    E, ld, eps = cfg.width, pad32(cfg.width), cfg.norm_eps

    def norm(name):
        return Norm(w[name], ld, eps)

    mixers, mlps = [], []
    for i, layer in enumerate(cfg.layers):
        p, m = f"l{i}.mix.", layer["mixer"]
        if layer["type"] == "rglru":
            mixers.append(RGLRU(width=E, size=m["width"], blocks=m["blocks"], taps=m["conv"], norm=norm(f"l{i}.norm1"), y=w[p + "y"],
                                y_b=w[p + "y.b"], x=w[p + "x"], x_b=w[p + "x.b"], conv=w[p + "conv"], conv_b=w[p + "conv.b"],
                                ra=w[p + "ra"], ra_b=w[p + "ra.b"], ri=w[p + "ri"], ri_b=w[p + "ri.b"], lam=w[p + "lam"], o=w[p + "o"],
                                dtype=dtype))
        else:
            mixers.append(LatentAttention(width=E, heads=m["heads"], dim=m["dim"], rot=m["rot_dim"], vdim=m["vdim"], rank=m["kv_rank"],
                                          scale=m["scale"], rot_base=m["rot"]["base"], rot_dims=m["rot"].get("dims", m["rot_dim"]),
                                          norm=norm(f"l{i}.norm1"), q=w[p + "q"], dkv=w[p + "dkv"], dkv_norm=w[p + "dkv.norm"],
                                          uk=w[p + "uk"], uv=w[p + "uv"], g=w[p + "g"], o=w[p + "o"], dtype=dtype))
        mlps.append(None if layer.get("mlp") is None else
                    ClampedGLU(width=E, limit=layer["mlp"]["limit"], norm=norm(f"l{i}.norm2"), gate=w[f"l{i}.mlp.gate"],
                               up=w[f"l{i}.mlp.up"], down=w[f"l{i}.mlp.down"], dtype=dtype))
    enter = ConcatProjection(width=E, weight=w["loop.in"], dtype=dtype) if cfg.loop is not None else None
    return HybridModel(vocab_size=cfg.vocab, width=E, dtype=dtype, device=device,
                       embed=spread(w["embed"].to(torch.bfloat16), 1, torch.arange(E), ld).contiguous(), embed_scale=cfg.embedding_scale,
                       runs=[LayerRun(mixers[i], mlps[i], enter if first else None) for i, first in cfg.order()],
                       head=Head(norm("final.norm"), w["head"], ld, cfg.logit_scale, dtype))
