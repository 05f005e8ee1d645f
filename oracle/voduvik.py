"""Plain restatement of the Voduvik decoder, one function per mechanism — TEST INFRASTRUCTURE ONLY.

Written from the design's equations for whole sequences, one token at a time where the design is sequential, with no cache,
no batching, no fusing and no weight layout of the product's; shares no code with vllmini_amd.  `dtype` is the arithmetic
(float64 by default: a yardstick; float32 to see what rounding alone does).

    tensors   dict name -> torch tensor (any float type), the names of a checkpoint of the design
    config    the parsed config.json (a dict)
"""
from __future__ import annotations

import math
from typing import Dict, List, Optional, Tuple

import torch

Tensors = Dict[str, torch.Tensor]


def gelu_tanh(z: torch.Tensor) -> torch.Tensor:
    return 0.5 * z * (1 + torch.tanh(math.sqrt(2 / math.pi) * (z + 0.044715 * z ** 3)))


def layer_norm(x: torch.Tensor, weight: torch.Tensor, eps: float) -> torch.Tensor:
    d = x - x.mean(-1, keepdim=True)
    return d / torch.sqrt((d * d).mean(-1, keepdim=True) + eps) * weight


def rms_norm(x: torch.Tensor, weight: torch.Tensor, eps: float) -> torch.Tensor:
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps) * weight


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


def causal_conv(x: torch.Tensor, weight: torch.Tensor, bias: torch.Tensor) -> torch.Tensor:
    """x [T, C], weight [C, taps]: the last tap multiplies the current token, what lies before the sequence is zero."""
    T, taps = x.shape[0], weight.shape[1]
    out = torch.zeros_like(x)
    for t in range(T):
        acc = bias.clone()
        for j in range(taps):
            src = t - (taps - 1) + j
            if src >= 0:
                acc = acc + weight[:, j] * x[src]
        out[t] = acc
    return out


def rglru_gate(u: torch.Tensor, mats: torch.Tensor, bias: torch.Tensor) -> torch.Tensor:
    """sigmoid of the block-diagonal product: block b of u through mats[b] ([out, in])."""
    nb, n = mats.shape[0], mats.shape[1]
    parts = [torch.sigmoid(u[..., b * n:(b + 1) * n] @ mats[b].T + bias[b]) for b in range(nb)]
    return torch.cat(parts, dim=-1)


def rglru_scan(u: torch.Tensor, r: torch.Tensor, i: torch.Tensor, lam: torch.Tensor, state: Optional[torch.Tensor] = None):
    """The linear recurrence over [T, C]; returns (S of every token, the last one)."""
    softplus = torch.log1p(torch.exp(-lam.abs())) + torch.clamp(lam, min=0)
    S = torch.zeros_like(u[0]) if state is None else state
    out = []
    for t in range(u.shape[0]):
        log_a = -8 * r[t] * softplus
        a = torch.exp(log_a)
        S = a * S + torch.sqrt(-torch.expm1(2 * log_a)) * i[t] * u[t]
        out.append(S)
    return torch.stack(out), S


def mixer_rglru(h: torch.Tensor, w: Tensors, p: str) -> torch.Tensor:
    y = gelu_tanh(h @ w[p + "y"].T + w[p + "y.b"])
    u = causal_conv(h @ w[p + "x"].T + w[p + "x.b"], w[p + "conv"], w[p + "conv.b"])
    r = rglru_gate(u, w[p + "ra"], w[p + "ra.b"])
    i = rglru_gate(u, w[p + "ri"], w[p + "ri.b"])
    S, _ = rglru_scan(u, r, i, w[p + "lam"])
    return (S * y) @ w[p + "o"].T


def latent_attend(qn: torch.Tensor, qr: torch.Tensor, c: torch.Tensor, kr: torch.Tensor, uk: torch.Tensor, uv: torch.Tensor,
                  scale: float) -> torch.Tensor:
    """One query token over the latents it sees: qn [H, dim], qr [H, rot], c [n, rank], kr [n, rot], uk [H, dim, rank],
    uv [H, vdim, rank] -> [H, vdim]."""
    H = qn.shape[0]
    out = []
    for h in range(H):
        k, v = c @ uk[h].T, c @ uv[h].T
        s = (k @ qn[h] + kr @ qr[h]) * scale
        w = torch.exp(s - s.max())
        out.append((w / w.sum()) @ v)
    return torch.stack(out)


def mixer_latent_attention(h: torch.Tensor, w: Tensors, p: str, m: dict, eps: float) -> torch.Tensor:
    H, dim, rot, vd, rank = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    T = h.shape[0]
    q = (h @ w[p + "q"].T).view(T, H, dim + rot)
    d = h @ w[p + "dkv"].T
    c = rms_norm(d[:, :rank], w[p + "dkv.norm"], eps)
    base = m["rot"]["base"]
    kr = torch.stack([rotate(d[t, rank:], t, base, rot) for t in range(T)])
    uk, uv = w[p + "uk"].view(H, dim, rank), w[p + "uv"].view(H, vd, rank)
    gate = torch.sigmoid(h @ w[p + "g"].T)
    rows = []
    for t in range(T):
        o = latent_attend(q[t, :, :dim], rotate(q[t, :, dim:], t, base, rot), c[:t + 1], kr[:t + 1], uk, uv, m["scale"])
        rows.append((o * gate[t][:, None]).reshape(-1))
    return torch.stack(rows) @ w[p + "o"].T


def feed_forward(h: torch.Tensor, w: Tensors, p: str, limit: float) -> torch.Tensor:
    g = torch.clamp(h @ w[p + "gate"].T, max=limit)
    u = torch.clamp(h @ w[p + "up"].T, min=-limit, max=limit)
    return (g * torch.sigmoid(1.702 * g) * (u + 1)) @ w[p + "down"].T


def layer_runs(config: dict) -> List[Tuple[int, bool]]:
    """(layer, whether the loop's input projection comes right before it) in the order they run."""
    n, loop = len(config["layers"]), config.get("loop")
    if not loop:
        return [(i, False) for i in range(n)]
    a, b = loop["start"], loop["stop"]
    body = [(i, i == a) for i in range(a, b)]
    return [(i, False) for i in range(a)] + body * loop["times"] + [(i, False) for i in range(b, n)]


@torch.no_grad()
def forward(config: dict, tensors: Tensors, tokens, dtype=torch.float64):
    """(logits [T, vocab], residual stream after every layer run [runs, T, width]) of one sequence."""
    w = {k: v.to(dtype) for k, v in tensors.items()}
    eps = config["norm"]["eps"]
    x = w["embed"][torch.as_tensor(list(tokens), dtype=torch.long)] * config["embedding"]["scale"]
    x0, streams = x, []
    for i, enter in layer_runs(config):
        if enter:
            x = torch.cat([x, x0], dim=-1) @ w["loop.in"].T
        L = config["layers"][i]
        h = layer_norm(x, w[f"l{i}.norm1"], eps)
        if L["type"] == "rglru":
            x = x + mixer_rglru(h, w, f"l{i}.mix.")
        else:
            x = x + mixer_latent_attention(h, w, f"l{i}.mix.", L["mixer"], eps)
        if L["mlp"] is not None:
            x = x + feed_forward(layer_norm(x, w[f"l{i}.norm2"], eps), w, f"l{i}.mlp.", L["mlp"]["limit"])
        streams.append(x)
    return layer_norm(x, w["final.norm"], eps) @ w["head"].T * config["logit_scale"], torch.stack(streams)
