"""Small Voduvik configurations, random weights and model folders for the tests (nothing of the product is used here)."""
from __future__ import annotations

import json
import os
import struct

import numpy as np
import torch


def rglru(width, blocks, conv=4, mlp=None):
    return {"type": "rglru", "mixer": {"width": width, "blocks": blocks, "conv": conv}, "mlp": mlp}


def attention(heads, dim, rot_dim, vdim, kv_rank, scale, base=10000.0, mlp=None):
    return {"type": "latent_attention", "mlp": mlp,
            "mixer": {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "kv_rank": kv_rank, "scale": scale,
                      "rot": {"base": base, "dims": rot_dim}}}


def dense(ff, limit):
    return {"kind": "dense", "ff": ff, "limit": limit}


def config(layers, *, vocab=211, width=96, loop=None, eps=1e-5, embedding_scale=3.0, logit_scale=0.75):
    c = {"architecture": "Voduvik", "vocab": vocab, "width": width, "layers": layers, "norm": {"eps": eps},
         "embedding": {"scale": embedding_scale}, "logit_scale": logit_scale}
    if loop is not None:
        c["loop"] = {"start": loop[0], "stop": loop[1], "times": loop[2]}
    return c


# name -> configuration: sizes that are no multiples of 32 or 16, layers of one kind with different sizes, loops of every extent
CONFIGS = {
    "mixed": config([rglru(120, 3, 3), attention(3, 20, 12, 24, 40, 0.31, 500.0, dense(72, 0.9)), rglru(64, 2, 5, dense(40, 2.0)),
                     attention(5, 16, 8, 40, 72, 0.17)], loop=(1, 3, 2), width=88, vocab=203),
    "loop_all": config([attention(2, 40, 32, 16, 48, 0.2, mlp=dense(50, 1.1)), rglru(100, 1, 2)], loop=(0, 2, 3), width=64, vocab=97),
    "no_loop": config([rglru(56, 7, 4, dense(33, 0.7)), rglru(192, 1, 1), attention(17, 8, 6, 10, 20, 0.4)], width=50, vocab=130),
    "only_recurrent": config([rglru(70, 2, 4), rglru(90, 9, 6)], width=72, vocab=64, loop=(1, 2, 4)),
    "only_attention": config([attention(4, 33, 10, 17, 100, 0.15, mlp=dense(64, 1.0)), attention(1, 48, 16, 48, 32, 0.3)], width=40,
                             vocab=77, loop=(0, 1, 1)),
}


def shapes(c):
    E = c["width"]
    out = {"embed": (c["vocab"], E)}
    if "loop" in c:
        out["loop.in"] = (E, 2 * E)
    for i, L in enumerate(c["layers"]):
        p, m = f"l{i}.mix.", L["mixer"]
        out[f"l{i}.norm1"] = (E,)
        if L["type"] == "rglru":
            W, b = m["width"], m["blocks"]
            n = W // b
            out.update({p + "y": (W, E), p + "y.b": (W,), p + "x": (W, E), p + "x.b": (W,), p + "conv": (W, m["conv"]), p + "conv.b": (W,),
                        p + "ra": (b, n, n), p + "ra.b": (b, n), p + "ri": (b, n, n), p + "ri.b": (b, n), p + "lam": (W,), p + "o": (E, W)})
        else:
            H, r = m["heads"], m["kv_rank"]
            out.update({p + "q": (H * (m["dim"] + m["rot_dim"]), E), p + "dkv": (r + m["rot_dim"], E), p + "dkv.norm": (r,),
                        p + "uk": (H * m["dim"], r), p + "uv": (H * m["vdim"], r), p + "g": (H, E), p + "o": (E, H * m["vdim"])})
        if L["mlp"] is not None:
            ff = L["mlp"]["ff"]
            out.update({f"l{i}.norm2": (E,), f"l{i}.mlp.gate": (ff, E), f"l{i}.mlp.up": (ff, E), f"l{i}.mlp.down": (E, ff)})
    out["final.norm"] = (E,)
    out["head"] = (c["vocab"], E)
    return out


def tensors(c, seed=0):
    """bfloat16 weights, lively enough that a wrong key, a lost state or a missing bias moves the logits: products keep the size of
    their inputs, biases and norms vary, decays reach from a token to hundreds."""
    g = torch.Generator().manual_seed(seed)
    out = {}
    for name, shape in shapes(c).items():
        t = torch.randn(shape, generator=g)
        if "norm" in name:
            t = 1 + 0.3 * t
        elif name.endswith(".lam"):
            t = 2 * t - 3
        elif name == "embed":
            t = t / c["embedding"]["scale"]
        elif name.endswith(".q"):
            t = t * 2 / shape[-1] ** 0.5
        elif len(shape) >= 2:
            t = t / shape[-1] ** 0.5
        else:
            t = 0.5 * t
        out[name] = t.to(torch.bfloat16)
    return out


def tokens(c, n, seed=0):
    return np.random.default_rng(seed).integers(0, c["vocab"], n).tolist()


def write_safetensors(path, named):
    """The format by hand: an independent writer for the product's reader."""
    kinds = {torch.bfloat16: "BF16", torch.float32: "F32", torch.int32: "I32"}
    header, data, at = {"__metadata__": {"format": "pt"}}, [], 0
    for name, t in named.items():
        raw = t.contiguous().view(torch.uint8 if t.dtype != torch.bfloat16 else torch.int16).numpy().tobytes()
        header[name] = {"dtype": kinds[t.dtype], "shape": list(t.shape), "data_offsets": [at, at + len(raw)]}
        data.append(raw)
        at += len(raw)
    h = json.dumps(header).encode()
    h += b" " * (-len(h) % 8)
    with open(path, "wb") as f:
        f.write(struct.pack("<Q", len(h)) + h + b"".join(data))


def write_model(folder, c, w):
    os.makedirs(folder, exist_ok=True)
    with open(os.path.join(folder, "config.json"), "w") as f:
        json.dump(c, f)
    write_safetensors(os.path.join(folder, "model.safetensors"), w)
    return str(folder)
