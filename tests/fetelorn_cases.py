"""Small Fetelorn configurations and random weights for the tests (nothing of the product is used here)."""
from __future__ import annotations

import torch

from tests.voduvik_cases import tokens, write_model  # noqa: F401  (they only need a configuration's vocabulary)


def retention(heads, dim, vdim, rot, decay, base=10000.0, mlp=None):
    return {"type": "retention", "mlp": mlp,
            "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "decay": list(decay), "rot": {"base": base, "dims": rot}}}


def parallel(left, right, mlp=None):
    return {"type": "parallel", "mlp": mlp, "mixer": {"left": left, "right": right}}


def attention(heads, kv_heads, dim, vdim, scale, chunk, bias_max):
    return {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale, "bias_max": bias_max, "mask": {"size": chunk}}


def delta(heads, kv_heads, dim, vdim, conv):
    return {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": conv}


def dense(ff):
    return {"kind": "dense", "ff": ff}


def config(layers, *, vocab=211, width=96, eps=1e-5):
    return {"architecture": "Fetelorn", "vocab": vocab, "width": width, "layers": layers, "norm": {"eps": eps}}


# name -> configuration: sizes that are no multiples of 32 or 16, layers of one kind with different sizes, heads that share keys and heads
# that do not, convolutions of one tap, chunks of a few tokens, of a page and of several, layers without a feed-forward
CONFIGS = {
    "mixed": config([retention(3, 20, 24, 12, (0.5, 0.9, 0.999), 500.0, dense(72)),
                     parallel(attention(6, 2, 20, 12, 0.4, 13, 9), delta(4, 2, 24, 40, 3), dense(33)),
                     retention(2, 40, 72, 40, (0.97, 0.8)),
                     parallel(attention(5, 5, 24, 20, 0.3, 37, 100), delta(3, 1, 16, 8, 4))], width=88, vocab=203),
    "chunks": config([parallel(attention(4, 1, 40, 56, 0.25, 32, 30), delta(2, 2, 40, 20, 1)),
                      parallel(attention(3, 3, 9, 70, 0.6, 16, 64), delta(6, 3, 8, 33, 7), dense(50))], width=64, vocab=97),
    "only_retention": config([retention(1, 10, 33, 10, (1.0,), 50.0), retention(4, 36, 17, 6, (0.1, 0.7, 0.99, 0.9999), mlp=dense(90))],
                             width=50, vocab=64),
    "large_heads": config([parallel(attention(8, 1, 130, 150, 0.12, 50, 49), delta(2, 1, 140, 150, 5), dense(40)),
                           retention(2, 150, 160, 100, (0.9, 0.98))], width=72, vocab=77),
}
RANKS, BUCKETS = (5, 40), {13: 6, 37: 12, 32: 16, 16: 9, 50: 20}      # of the low-rank gates; of the bias by chunk


def shapes(c):
    E = c["width"]
    out = {"embed": (c["vocab"], E)}
    for i, L in enumerate(c["layers"]):
        p, m = f"l{i}.mix.", L["mixer"]
        out[f"l{i}.norm1"] = (E,)
        if L["type"] == "retention":
            a, b = m["heads"] * m["dim"], m["heads"] * m["vdim"]
            out.update({p + "q": (a, E), p + "k": (a, E), p + "v": (b, E), p + "g": (b, E), p + "o": (E, b)})
        else:
            a, b = m["left"], m["right"]
            H, G = a["heads"], a["kv_heads"]
            out.update({p + "left.q": (H * a["dim"], E), p + "left.k": (G * a["dim"], E), p + "left.v": (G * a["vdim"], E),
                        p + "left.rel": (BUCKETS.get(a["mask"]["size"], 8), H), p + "left.sink": (H,), p + "left.g": (H, E),
                        p + "left.o": (E, H * a["vdim"]), p + "left.out": (E,)})
            H, G, r = b["heads"], b["kv_heads"], RANKS
            qk, v, t = G * b["dim"], H * b["vdim"], b["conv"]
            out.update({p + "right.q": (qk, E), p + "right.k": (qk, E), p + "right.v": (v, E), p + "right.q.conv": (qk, t),
                        p + "right.k.conv": (qk, t), p + "right.v.conv": (v, t), p + "right.b": (H, E), p + "right.A_log": (H,),
                        p + "right.norm": (b["vdim"],), p + "right.a1": (r[0], E), p + "right.a2": (H * b["dim"], r[0]),
                        p + "right.dt_bias": (H * b["dim"],), p + "right.g1": (r[1], E), p + "right.g2": (v, r[1]), p + "right.o": (E, v),
                        p + "right.out": (E,)})
        if L["mlp"] is not None:
            ff = L["mlp"]["ff"]
            out.update({f"l{i}.mlp.gate": (ff, E), f"l{i}.mlp.up": (ff, E), f"l{i}.mlp.down": (E, ff)})
    out["final.norm"] = (E,)
    return out


def tensors(c, seed=0):
    """bfloat16 weights, lively enough that a wrong key, a lost state or a sink left out moves the logits: products keep the size of their
    inputs, norms, biases and sinks vary, decays reach from a token to hundreds."""
    g = torch.Generator().manual_seed(seed)
    out = {}
    for name, shape in shapes(c).items():
        t = torch.randn(shape, generator=g)
        if name.endswith(("norm", "norm1", ".out")):
            t = 1 + 0.3 * t
        elif name.endswith(".dt_bias"):
            t = 2 * t - 3
        elif name.endswith((".rel", ".sink")):
            t = 1.5 * t
        elif name.endswith(".A_log"):
            t = 0.7 * t
        elif name != "embed":
            t = t / shape[-1] ** 0.5
        out[name] = t.to(torch.bfloat16)
    return out
