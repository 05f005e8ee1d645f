"""Plain restatement of the Fetelorn decoder, one function per mechanism — TEST INFRASTRUCTURE ONLY.

Written from the design's equations for whole sequences: recurrences walk token by token, attention looks at one query at a time;
no cache, no batching, no chunked form of a recurrence and no weight layout of the product's; shares no code with vllmini_amd.
`dtype` is the arithmetic (float64 by default: a yardstick).

    tensors   dict name -> torch tensor (any float type), the names of a checkpoint of the design
    config    the parsed config.json (a dict)
"""
from __future__ import annotations

import math
from typing import Dict, Optional

import torch

Tensors = Dict[str, torch.Tensor]


def silu(z: torch.Tensor) -> torch.Tensor:
    return z * torch.sigmoid(z)


def softplus(z: torch.Tensor) -> torch.Tensor:
    return torch.log1p(torch.exp(-z.abs())) + torch.clamp(z, min=0)


def unit_rms(x: torch.Tensor, eps: float) -> torch.Tensor:
    """x over its root mean square along the last axis."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def unit_length(x: torch.Tensor, eps: float = 1e-6) -> torch.Tensor:
    return x / torch.sqrt((x * x).sum(-1, keepdim=True) + eps)


def rotate(v: torch.Tensor, position: int, base: float, dims: int) -> torch.Tensor:
    """Rotary embedding of the first `dims` components of v (last axis), component i paired with i + dims / 2."""
    half = dims // 2
    out = v.clone()
    for i in range(half):
        a = position * base ** (-2.0 * i / dims)
        c, s = math.cos(a), math.sin(a)
        out[..., i] = v[..., i] * c - v[..., i + half] * s
        out[..., i + half] = v[..., i + half] * c + v[..., i] * s
    return out


def causal_conv(x: torch.Tensor, weight: torch.Tensor) -> torch.Tensor:
    """x [T, C], weight [C, taps]: the last tap multiplies the current token, what lies before the sequence is zero."""
    T, taps = x.shape[0], weight.shape[1]
    out = torch.zeros_like(x)
    for t in range(T):
        for j in range(taps):
            src = t - (taps - 1) + j
            if src >= 0:
                out[t] += weight[:, j] * x[src]
    return out


def distance_bucket(n: int, buckets: int, far: float) -> int:
    """Which row of the bias table a distance of n tokens reads: one row each below half the rows, logarithmic above."""
    half = buckets // 2
    if n < half:
        return n
    return min(buckets - 1, half + math.floor(math.log(n / half) / math.log(far / half) * (buckets - half)))


def chunk_attend(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, i: int, size: int, scale: float, rel: torch.Tensor, far: float,
                 sink: torch.Tensor) -> torch.Tensor:
    """Token i over the keys of its own chunk: q [H, dim], k [T, G, dim], v [T, G, vdim], rel [buckets, H], sink [H] -> [H, vdim]."""
    H, G = q.shape[0], k.shape[1]
    js = [j for j in range(i + 1) if j // size == i // size]
    out = []
    for h in range(H):
        g = h // (H // G)
        s = torch.stack([k[j, g] @ q[h] * scale + rel[distance_bucket(i - j, rel.shape[0], far), h] for j in js])
        m = torch.maximum(s.max(), sink[h])
        e = torch.exp(s - m)
        out.append((e / (e.sum() + torch.exp(sink[h] - m))) @ v[js, g])
    return torch.stack(out)


def chunked_attention(h: torch.Tensor, w: Tensors, p: str, m: dict, eps: float) -> torch.Tensor:
    H, G, dim, vd, T = m["heads"], m["kv_heads"], m["dim"], m["vdim"], h.shape[0]
    q = unit_rms((h @ w[p + "q"].T).view(T, H, dim), eps)
    k = unit_rms((h @ w[p + "k"].T).view(T, G, dim), eps)
    v = (h @ w[p + "v"].T).view(T, G, vd)
    gate = torch.sigmoid(h @ w[p + "g"].T)
    rows = [(chunk_attend(q[t], k, v, t, m["mask"]["size"], m["scale"], w[p + "rel"], m["bias_max"], w[p + "sink"])
             * gate[t][:, None]).reshape(-1) for t in range(T)]
    return torch.stack(rows) @ w[p + "o"].T


def delta_rule(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, g: torch.Tensor, beta: torch.Tensor,
               state: Optional[torch.Tensor] = None):
    """Per head: decay the rows of S, correct what it holds under k towards v, read with q.  q, k, g [T, H, dim], v [T, H, vdim],
    beta [T, H] -> (o [T, H, vdim], S [H, dim, vdim])."""
    T, H, dim = q.shape
    S = torch.zeros(H, dim, v.shape[2], dtype=q.dtype) if state is None else state.clone()
    out = []
    for t in range(T):
        S = g[t][:, :, None] * S
        held = (S * k[t][:, :, None]).sum(1)
        u = beta[t][:, None] * (v[t] - held)
        S = S + k[t][:, :, None] * u[:, None, :]
        out.append((S * q[t][:, :, None]).sum(1))
    return torch.stack(out), S


def gated_delta(h: torch.Tensor, w: Tensors, p: str, m: dict, eps: float) -> torch.Tensor:
    H, G, dim, vd, T = m["heads"], m["kv_heads"], m["dim"], m["vdim"], h.shape[0]
    q, k, v = (silu(causal_conv(h @ w[p + n].T, w[p + n + ".conv"])) for n in "qkv")
    rep = H // G
    q = (unit_length(q.view(T, G, dim)) * dim ** -0.5).repeat_interleave(rep, dim=1)
    k = unit_length(k.view(T, G, dim)).repeat_interleave(rep, dim=1)
    beta = torch.sigmoid(h @ w[p + "b"].T)
    z = (h @ w[p + "a1"].T) @ w[p + "a2"].T + w[p + "dt_bias"]
    g = torch.exp(-torch.exp(w[p + "A_log"])[None, :, None] * softplus(z).view(T, H, dim))
    o, _ = delta_rule(q, k, v.view(T, H, vd), g, beta)
    o = unit_rms(o, eps) * w[p + "norm"] * torch.sigmoid((h @ w[p + "g1"].T) @ w[p + "g2"].T).view(T, H, vd)
    return o.reshape(T, H * vd) @ w[p + "o"].T


def mixer_parallel(h: torch.Tensor, w: Tensors, p: str, m: dict, eps: float) -> torch.Tensor:
    left = chunked_attention(h, w, p + "left.", m["left"], eps)
    right = gated_delta(h, w, p + "right.", m["right"], eps)
    return 0.5 * (unit_rms(left, eps) * w[p + "left.out"] + unit_rms(right, eps) * w[p + "right.out"])


def retain(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, decay: torch.Tensor, state: Optional[torch.Tensor] = None):
    """Linear attention that forgets at a fixed rate per head: q, k [T, H, dim], v [T, H, vdim], decay [H]."""
    T, H, dim = q.shape
    S = torch.zeros(H, dim, v.shape[2], dtype=q.dtype) if state is None else state.clone()
    out = []
    for t in range(T):
        S = decay[:, None, None] * S + k[t][:, :, None] * v[t][:, None, :]
        out.append((S * q[t][:, :, None]).sum(1))
    return torch.stack(out), S


def mixer_retention(h: torch.Tensor, w: Tensors, p: str, m: dict, eps: float) -> torch.Tensor:
    H, dim, vd, T = m["heads"], m["dim"], m["vdim"], h.shape[0]
    q, k = ((h @ w[p + n].T).view(T, H, dim) for n in "qk")
    base, dims = m["rot"]["base"], m["rot"]["dims"]
    q = torch.stack([rotate(q[t], t, base, dims) for t in range(T)])
    k = torch.stack([rotate(k[t], t, base, dims) for t in range(T)]) * dim ** -0.5
    o, _ = retain(q, k, (h @ w[p + "v"].T).view(T, H, vd), torch.tensor(m["decay"], dtype=h.dtype))
    return (unit_rms(o, eps).reshape(T, H * vd) * silu(h @ w[p + "g"].T)) @ w[p + "o"].T


def feed_forward(h: torch.Tensor, w: Tensors, p: str) -> torch.Tensor:
    return (silu(h @ w[p + "gate"].T) * (h @ w[p + "up"].T)) @ w[p + "down"].T


MIXERS = {"parallel": mixer_parallel, "retention": mixer_retention}


@torch.no_grad()
def forward(config: dict, tensors: Tensors, tokens, dtype=torch.float64):
    """(logits [T, vocab], residual stream after every layer [layers, T, width]) of one sequence."""
    w = {k: v.to(dtype) for k, v in tensors.items()}
    eps = config["norm"]["eps"]
    x = w["embed"][torch.as_tensor(list(tokens), dtype=torch.long)]
    streams = []
    for i, L in enumerate(config["layers"]):
        h = unit_rms(x, eps) * w[f"l{i}.norm1"]
        branch = MIXERS[L["type"]](h, w, f"l{i}.mix.", L["mixer"], eps)
        if L["mlp"] is not None:
            branch = branch + feed_forward(h, w, f"l{i}.mlp.")
        x = x + branch
        streams.append(x)
    return unit_rms(x, eps) * w["final.norm"] @ w["embed"].T, torch.stack(streams)
