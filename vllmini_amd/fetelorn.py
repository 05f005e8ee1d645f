"""The Fetelorn decoder: its configuration and the construction of its layers (hybrid_layers) from a checkpoint's tensors.

A list of layers, each x <- x + (mixer(h) + ff(h)) with h = RMS norm of x and a gated feed-forward or none.  The mixer is retention
("retention") or two mixers side by side ("parallel"): softmax attention inside chunks, and the gated delta rule.  The vocabulary
projection is the embedding.  Sizes come from config.json, or from a tensor's shape where it does not name them (the ranks of the
low-rank gates, the rows of the distance bias); every layer may have its own.
"""
from __future__ import annotations

import dataclasses
from typing import Dict, Optional, Tuple

import torch

from .hybrid_decoder import HybridModel, LayerRun
from .hybrid_layers import GatedDelta, GroupedAttention, Head, Norm, ParallelBlock, Retention, TwoArms, spread
from .hybrid_ops import SILU_UNIT, pad32

Shape = Tuple[Optional[int], ...]      # None: the tensor decides


@dataclasses.dataclass(frozen=True)
class FetelornConfig:
    vocab: int
    width: int
    layers: Tuple[dict, ...]
    norm_eps: float

    @classmethod
    def from_json(cls, c: dict) -> "FetelornConfig":
        cfg = cls(vocab=int(c["vocab"]), width=int(c["width"]), layers=tuple(c["layers"]), norm_eps=float(c["norm"]["eps"]))
        for i, layer in enumerate(cfg.layers):
            if layer["type"] not in ("retention", "parallel"):
                raise ValueError(f"layer {i}: unknown mixer {layer['type']!r}")
            if layer.get("mlp") is not None and layer["mlp"].get("kind") != "dense":
                raise ValueError(f"layer {i}: unknown feed-forward {layer['mlp'].get('kind')!r}")
            for arm in ("left", "right") if layer["type"] == "parallel" else ():
                m = layer["mixer"][arm]
                if m["heads"] % m["kv_heads"]:
                    raise ValueError(f"layer {i}: {m['heads']} heads over {m['kv_heads']} key heads")
        return cfg

    def tensor_shapes(self) -> Dict[str, Shape]:
        E = self.width
        out: Dict[str, Shape] = {"embed": (self.vocab, E), "final.norm": (E,)}
        for i, layer in enumerate(self.layers):
            p, m = f"l{i}.mix.", layer["mixer"]
            out[f"l{i}.norm1"] = (E,)
            if layer["type"] == "retention":
                qk, v = m["heads"] * m["dim"], m["heads"] * m["vdim"]
                out.update({p + "q": (qk, E), p + "k": (qk, E), p + "v": (v, E), p + "g": (v, E), p + "o": (E, v)})
            else:
                a, b = m["left"], m["right"]
                H, G = a["heads"], a["kv_heads"]
                out.update({p + "left." + n: s for n, s in {
                    "q": (H * a["dim"], E), "k": (G * a["dim"], E), "v": (G * a["vdim"], E), "rel": (None, H), "sink": (H,), "g": (H, E),
                    "o": (E, H * a["vdim"]), "out": (E,)}.items()})
                H, G, taps = b["heads"], b["kv_heads"], b["conv"]
                qk, d, v = G * b["dim"], H * b["dim"], H * b["vdim"]
                out.update({p + "right." + n: s for n, s in {
                    "q": (qk, E), "k": (qk, E), "v": (v, E), "q.conv": (qk, taps), "k.conv": (qk, taps), "v.conv": (v, taps), "b": (H, E),
                    "A_log": (H,), "norm": (b["vdim"],), "a1": (None, E), "a2": (d, None), "dt_bias": (d,), "g1": (None, E),
                    "g2": (v, None), "o": (E, v), "out": (E,)}.items()})
            if layer.get("mlp") is not None:
                ff = layer["mlp"]["ff"]
                out.update({f"l{i}.mlp.gate": (ff, E), f"l{i}.mlp.up": (ff, E), f"l{i}.mlp.down": (E, ff)})
        return out


def random_tensors(cfg: FetelornConfig, device, seed: int = 0, rank: int = 128, buckets: int = 32) -> Dict[str, torch.Tensor]:
    """Random bfloat16 weights of a configuration, scaled so that activations keep their size (no checkpoint exists)."""
    g = torch.Generator(device=device).manual_seed(seed)
    out = {}
    for name, shape in cfg.tensor_shapes().items():
        free = buckets if name.endswith(".rel") else rank
        t = torch.randn([free if n is None else n for n in shape], generator=g, device=device)
        if name.endswith(("norm", "norm1", ".out")):
            t = 1 + 0.1 * t
        elif name.endswith(".dt_bias"):
            t = t - 4.0              # decays of a few to a few hundred tokens
        elif name.endswith((".A_log", ".sink", ".rel")):
            t = 0.5 * t
        elif name != "embed":
            t = t * t.shape[-1] ** -0.5
        out[name] = t.to(torch.bfloat16)
    return out


def _check(cfg: FetelornConfig, tensors: Dict[str, torch.Tensor]) -> None:
    for name, shape in cfg.tensor_shapes().items():
        if name not in tensors:
            raise KeyError(f"the checkpoint lacks {name}")
        have = tuple(tensors[name].shape)
        if len(have) != len(shape) or any(want is not None and n != want for n, want in zip(have, shape)):
            raise ValueError(f"{name} has shape {have}, the configuration says {tuple(shape)}")
    for name in tensors:
        if name.endswith((".right.a1", ".right.g1")) and tensors[name].shape[0] != tensors[name[:-1] + "2"].shape[1]:
            raise ValueError(f"{name} and {name[:-1]}2 have different ranks")


def build_model(cfg: FetelornConfig, tensors: Dict[str, torch.Tensor], dtype: torch.dtype, device) -> HybridModel:
    device = torch.device(device)
    _check(cfg, tensors)
    w = {k: t.to(device) for k, t in tensors.items()}
    E, ld, eps = cfg.width, pad32(cfg.width), cfg.norm_eps
    runs = []
    for i, layer in enumerate(cfg.layers):
        p, m = f"l{i}.mix.", layer["mixer"]
        if layer["type"] == "retention":
            mixer = Retention(width=E, heads=m["heads"], dim=m["dim"], vdim=m["vdim"], decay=m["decay"], rot_base=m["rot"]["base"],
                              rot_dims=m["rot"]["dims"], eps=eps, q=w[p + "q"], k=w[p + "k"], v=w[p + "v"], g=w[p + "g"], o=w[p + "o"],
                              dtype=dtype)
        else:
            a, b = m["left"], m["right"]
            left = GroupedAttention(width=E, heads=a["heads"], kv_heads=a["kv_heads"], dim=a["dim"], vdim=a["vdim"], scale=a["scale"],
                                    chunk=a["mask"]["size"], bias_max=a["bias_max"], eps=eps, dtype=dtype,
                                    **{n: w[p + "left." + n] for n in ("q", "k", "v", "rel", "sink", "g", "o")})
            r = p + "right."
            right = GatedDelta(width=E, heads=b["heads"], kv_heads=b["kv_heads"], dim=b["dim"], vdim=b["vdim"], taps=b["conv"], eps=eps,
                               q_conv=w[r + "q.conv"], k_conv=w[r + "k.conv"], v_conv=w[r + "v.conv"], a_log=w[r + "A_log"], dtype=dtype,
                               **{n: w[r + n] for n in ("q", "k", "v", "b", "a1", "a2", "dt_bias", "norm", "g1", "g2", "o")})
            mixer = TwoArms(width=E, left=left, right=right, left_out=w[p + "left.out"], right_out=w[p + "right.out"], eps=eps)
        ff = {n: w.get(f"l{i}.mlp.{n}") if layer.get("mlp") is not None else None for n in ("gate", "up", "down")}
        runs.append(LayerRun(ParallelBlock(width=E, norm=Norm(w[f"l{i}.norm1"], ld, eps, rms=True), mixer=mixer, unit=SILU_UNIT,
                                           dtype=dtype, **ff)))
    embed = spread(w["embed"].to(torch.bfloat16), 1, torch.arange(E), ld).contiguous()
    return HybridModel(vocab_size=cfg.vocab, width=E, dtype=dtype, device=device, embed=embed, embed_scale=1.0, runs=runs,
                       head=Head(Norm(w["final.norm"], ld, eps, rms=True), w["embed"], ld, 1.0, dtype))
