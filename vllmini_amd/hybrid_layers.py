"""Layers of decoders that mix recurrences, linear and softmax attention, over hybrid_ops: each class lays its weights out for the
kernels once (heads, blocks and ranks zero-padded to multiples of 32, so no kernel has a ragged edge) and runs one step.

Layers with a residual add behind each branch:
    LatentAttention   softmax attention whose cache holds one latent row per token, query side folded into the latent space
    RGLRU             the recurrent block: convolution, block-diagonal gates, gated linear recurrence
    ClampedGLU        the feed-forward with a clamped gated unit
    ConcatProjection  x <- W [x ; x0]

One norm in front of mixer and feed-forward, one residual add behind both:
    ParallelBlock     x <- x + (mixer(h) + ff(h)), h = norm(x): ONE product in front of a mixer's core and the gated unit, and behind
                      them one (the concatenated rows times [W_o | W_down]) or, for a mixer of two arms, one per arm
    its mixers        Retention, GroupedAttention, GatedDelta, TwoArms (two mixers side by side, their normed outputs averaged)

What a decoder asks of a mixer: page_rows() and state_shapes(), the cache tensors and states it keeps, tiling() if it is an attention
(how its query rows are cut), and run() with the step's plans and what it holds: its page tensors first, then its states.

The residual stream is float32 (`Residual`).  Steps of few tokens run on the streaming kernels with everything fused around the
products (norm in front, gated unit / head gate / residual add behind); from DENSE_MIN_TOKENS tokens on (from DENSE_MIN_TOKENS_LARGE
for matrices of DENSE_LARGE elements) the products go to the vendor library (F.linear, as the prefill of the GPT-2 decoder does)
with one elementwise kernel between two of them.
"""
from __future__ import annotations

import math
from typing import Dict, List, NamedTuple, Optional, Sequence, Tuple

import torch
import torch.nn.functional as F

from . import hybrid_ops as ops
from .hybrid_ops import SILU_UNIT, GatedUnit, MatrixTiles, StepLayout, pad32, state_dim

DENSE_MIN_TOKENS = 48
DENSE_MIN_TOKENS_LARGE, DENSE_LARGE = 17, 32 << 20


def dense(tokens: int, w: MatrixTiles) -> bool:
    return tokens >= DENSE_MIN_TOKENS or (tokens >= DENSE_MIN_TOKENS_LARGE and w.N * w.K >= DENSE_LARGE)


def float_product(x: torch.Tensor, w: torch.Tensor) -> torch.Tensor:
    """x W^T as float32, whatever the operands' type."""
    return torch.mm(x, w.t()) if x.dtype == torch.float32 else torch.mm(x, w.t(), out_dtype=torch.float32)


class Norm:
    """A layer norm's (rms: an RMS norm's) weight, zero-padded (padding columns of the stream stay zero)."""

    def __init__(self, weight: torch.Tensor, ld: int, eps: float, rms: bool = False):
        self.n, self.eps, self.rms = weight.numel(), float(eps), rms
        self.weight = torch.zeros(ld, dtype=torch.float32, device=weight.device)
        self.weight[: self.n] = weight.float()

    @property
    def args(self) -> ops.NormArgs:
        return self.weight, self.n, self.eps, self.rms


class QueryTiling(NamedTuple):
    """How an attention's query rows are cut into tiles: `rep` rows per token and set of rows, `sets` of them (a launch dimension),
    partial results of `width` columns when keys are split, at most `chunk` keys (0: all) per row.  `kernel` names whose row tiles
    they are."""
    kernel: str
    rep: int
    sets: int
    width: int
    chunk: int = 0
    sizes: Tuple[int, ...] = ()

    def row_tiles(self, want: int, dtype: torch.dtype) -> int:
        return (ops.latent_row_tiles if self.kernel == "latent" else ops.attention_row_tiles)(*self.sizes, want, dtype)


class AttentionPlan(NamedTuple):
    """How the query rows of a step are dealt to workgroups, for layers of one QueryTiling."""
    tiles: torch.Tensor
    row_tiles: int
    splits: int


Plans = Dict[QueryTiling, AttentionPlan]


class Head:
    """Final norm and vocabulary projection, logits float32 times a scale (folded into the norm's weight on the dense path)."""

    def __init__(self, norm: Norm, weight: torch.Tensor, ld: int, scale: float, dtype: torch.dtype):
        self.norm, self.vocab, self.scale, self.dtype = norm, weight.shape[0], float(scale), dtype
        self.w = MatrixTiles(spread(weight, 1, torch.arange(weight.shape[1]), ld), dtype, dense=True)
        self.scaled = (norm.weight * self.scale, *norm.args[1:])

    def run(self, x: torch.Tensor, rows: torch.Tensor) -> torch.Tensor:
        if dense(rows.numel(), self.w):
            h = ops.add_norm(x.index_select(0, rows), None, self.scaled, self.dtype)
            return float_product(h, self.w.dense)[:, : self.vocab]
        return ops.linear(x, self.w, norm=self.norm.args, rows=rows, float_out=(self.vocab, self.scale))


class Residual:
    """The residual stream [T, ld] float32, and a branch output that still has to be added to it (dense path: the add rides in the
    kernel that normalises the stream for the next branch)."""

    def __init__(self, x: torch.Tensor, dtype: torch.dtype):
        self.x, self.dtype = x, dtype
        self.pending: Optional[torch.Tensor] = None

    def settle(self) -> torch.Tensor:
        if self.pending is not None:
            ops.add_norm(self.x, self.pending, None, self.dtype)
            self.pending = None
        return self.x

    def normed(self, norm: Norm) -> torch.Tensor:
        h = ops.add_norm(self.x, self.pending, norm.args, self.dtype)
        self.pending = None
        return h

    def branch_in(self, norm: Norm, w: MatrixTiles, step: StepLayout, bias: Optional[torch.Tensor] = None,
                  dense_bias: Optional[torch.Tensor] = None) -> torch.Tensor:
        """norm(x) W^T (+ bias) in the element type."""
        if dense(step.T, w):
            return F.linear(self.normed(norm), w.dense, dense_bias)
        return ops.linear(self.settle(), w, norm=norm.args, bias=bias)

    def branch_out(self, o: torch.Tensor, w: MatrixTiles, step: StepLayout) -> None:
        """x += o W^T."""
        if dense(step.T, w):
            self.pending = F.linear(o, w.dense)
        else:
            ops.linear(o, w, residual=True, out=self.settle())


def spread(t: torch.Tensor, dim: int, index: torch.Tensor, size: int) -> torch.Tensor:
    """`t` with its `dim` stretched to `size` zeros-padded entries, entry i going to index[i]."""
    shape = list(t.shape)
    shape[dim] = size
    out = torch.zeros(shape, dtype=t.dtype, device=t.device)
    return out.index_copy_(dim, index.to(t.device), t)


def strided_index(parts: int, n: int, stride: int, offset: int = 0) -> torch.Tensor:
    """Where `parts` runs of n entries go when each run gets `stride` places."""
    return (torch.arange(parts)[:, None] * stride + torch.arange(n)[None, :] + offset).reshape(-1)


def interleaved(gate: torch.Tensor, up: torch.Tensor, ld: int) -> torch.Tensor:
    """The rows (gate 0, up 0, gate 1, up 1, ...) of a gated feed-forward, padded to a multiple of 32 of either and `ld` columns."""
    ff, width = gate.shape
    both = torch.zeros((2 * pad32(ff), ld), dtype=gate.dtype, device=gate.device)
    both[0:2 * ff:2, :width], both[1:2 * ff:2, :width] = gate, up
    return both


def padded_heads(w: torch.Tensor, heads: int, n: int, dim: int = 0) -> torch.Tensor:
    """`dim` of w, heads runs of equal length, with every run padded to n."""
    return spread(w, dim, strided_index(heads, w.shape[dim] // heads, n), heads * n)


def padded_rows(w: torch.Tensor, n: int, dim: int = 0) -> torch.Tensor:
    return spread(w, dim, torch.arange(w.shape[dim]), n)


class LatentAttention:
    """q [heads (dim + rot), E], dkv [rank + rot, E], uk [heads dim, rank], uv [heads vdim, rank], g [heads, E], o [E, heads vdim]."""

    def __init__(self, *, width: int, heads: int, dim: int, rot: int, vdim: int, rank: int, scale: float, rot_base: float, rot_dims: int,
                 norm: Norm, q: torch.Tensor, dkv: torch.Tensor, dkv_norm: torch.Tensor, uk: torch.Tensor, uv: torch.Tensor,
                 g: torch.Tensor, o: torch.Tensor, dtype: torch.dtype):
        if rot_dims % 2 or rot_dims > rot:
            raise ValueError(f"rotated dimensions {rot_dims} must be even and at most rot_dim {rot}")
        dev, E = q.device, pad32(width)
        self.heads, self.scale, self.rot_n, self.rank_n, self.norm = heads, float(scale), rot_dims, rank, norm
        self.dim, self.rot, self.vdim, self.rank = pad32(dim), pad32(rot), pad32(vdim), pad32(rank)
        self.row = self.rank + self.rot                    # a cache row: [latent | rotated shared key]
        hd = self.dim + self.rot
        self.gate_at = heads * hd + self.row
        rows = torch.cat([
            spread(spread(q.view(heads, dim + rot, width), 1,
                          torch.cat([torch.arange(dim), self.dim + torch.arange(rot)]), hd).reshape(heads * hd, width),
                   1, torch.arange(width), E),
            spread(spread(dkv, 0, torch.cat([torch.arange(rank), self.rank + torch.arange(rot)]), self.row), 1, torch.arange(width), E),
            spread(spread(g, 0, torch.arange(heads), pad32(heads)), 1, torch.arange(width), E)])
        self.w_in = MatrixTiles(rows, dtype, dense=True)
        self.w_uk = MatrixTiles(uk.view(heads, dim, rank).transpose(1, 2).contiguous(), dtype)     # [rank, dim]: q into the latent space
        self.w_uv = MatrixTiles(uv.view(heads, vdim, rank), dtype)
        self.w_o = MatrixTiles(spread(spread(o, 1, strided_index(heads, vdim, self.vdim), heads * self.vdim), 0, torch.arange(width), E),
                               dtype, dense=True)
        self.norm_w = torch.zeros(self.rank, dtype=torch.float32, device=dev)
        self.norm_w[:rank] = dkv_norm.float()
        i = torch.arange(rot_dims // 2, dtype=torch.float64)
        self.freq = (float(rot_base) ** (-2.0 * i / rot_dims)).to(dev)
        self.eps = norm.eps

    def page_rows(self) -> List[int]:
        return [self.row]

    def state_shapes(self) -> List[Tuple[Sequence[int], torch.dtype]]:
        return []

    def tiling(self) -> Optional[QueryTiling]:
        return QueryTiling("latent", self.heads, 1, self.row, sizes=(self.row,))

    def run(self, res: Residual, step: StepLayout, plans: Plans, held: Sequence[torch.Tensor]) -> None:
        H, D, plan, (cache,) = self.heads, self.row, plans[self.tiling()], held
        proj = res.branch_in(self.norm, self.w_in, step)
        q = torch.empty((step.T, H * D), dtype=proj.dtype, device=proj.device)
        ops.linear(proj, self.w_uk, x_gstride=self.dim + self.rot, y_gstride=D, out=q)
        ops.latent_prep(proj, q, cache, step, norm_w=self.norm_w, freq=self.freq, heads=H, dim=self.dim, rot=self.rot, rank=self.rank,
                        rot_n=self.rot_n, rank_n=self.rank_n, eps=self.eps)
        lat = ops.latent_attention(q, cache, step, plan.tiles, heads=H, rank=self.rank, rot=self.rot, scale=self.scale,
                                   row_tiles=plan.row_tiles, splits=plan.splits)
        o = ops.linear(lat, self.w_uv, x_gstride=self.rank, y_gstride=self.vdim, gate=proj[:, self.gate_at:])
        res.branch_out(o, self.w_o, step)


class RGLRU:
    """y, x [W, E] with biases, conv [W, taps] with bias, ra / ri [blocks, W / blocks, W / blocks] with biases, lam [W], o [E, W]."""

    def __init__(self, *, width: int, size: int, blocks: int, taps: int, norm: Norm, y: torch.Tensor, y_b: torch.Tensor, x: torch.Tensor,
                 x_b: torch.Tensor, conv: torch.Tensor, conv_b: torch.Tensor, ra: torch.Tensor, ra_b: torch.Tensor, ri: torch.Tensor,
                 ri_b: torch.Tensor, lam: torch.Tensor, o: torch.Tensor, dtype: torch.dtype):
        if size % blocks:
            raise ValueError(f"{size} channels do not divide into {blocks} blocks")
        dev, E, bw = y.device, pad32(width), size // blocks
        bp = pad32(bw)
        self.norm, self.blocks, self.taps, self.width = norm, blocks, taps, blocks * bp
        idx = strided_index(blocks, bw, bp)
        W = self.width

        def ch(t, dim=0):          # a tensor over channels, each block padded
            return spread(t, dim, idx, W)

        cols = torch.arange(width)
        self.w_in = MatrixTiles(torch.cat([spread(ch(y), 1, cols, E), spread(ch(x), 1, cols, E)]), dtype, dense=True)
        self.bias = torch.cat([ch(y_b), ch(x_b)]).float().contiguous()
        self.dense_bias = self.bias.to(dtype)
        self.conv_w = ch(conv).float().t().contiguous()
        self.conv_b = ch(conv_b).float().contiguous()
        both = torch.zeros((2, blocks, bp, bp), dtype=torch.float32, device=dev)
        both[0, :, :bw, :bw], both[1, :, :bw, :bw] = ra.float(), ri.float()
        self.gates = MatrixTiles(both.view(2 * blocks, bp, bp), dtype).tiles
        self.gate_b = torch.stack([ch(ra_b.reshape(-1)), ch(ri_b.reshape(-1))]).float().contiguous()
        self.decay = (-8.0 * F.softplus(ch(lam).double(), threshold=1e9)).float().contiguous()
        self.w_o = MatrixTiles(spread(spread(o, 1, idx, W), 0, cols, E), dtype, dense=True)
        self.dtype = dtype

    def page_rows(self) -> List[int]:
        return []

    def tiling(self) -> Optional[QueryTiling]:
        return None

    def state_shapes(self) -> List[Tuple[Sequence[int], torch.dtype]]:
        """The recurrence's state and the two halves of the convolution's tail (at least one row, so that a tensor exists)."""
        return [((self.width,), torch.float32), ((2, self.taps - 1, self.width), self.dtype)]

    def run(self, res: Residual, step: StepLayout, plans: Plans, held: Sequence[torch.Tensor]) -> None:
        state, tail = held
        yx = res.branch_in(self.norm, self.w_in, step, self.bias, self.dense_bias)
        o = ops.rglru(yx, step, conv_w=self.conv_w, conv_b=self.conv_b, gates=self.gates, gate_b=self.gate_b, decay=self.decay,
                      blocks=self.blocks, state=state, tail=tail)
        res.branch_out(o, self.w_o, step)


class ClampedGLU:
    """gate, up [ff, E], down [E, ff]."""

    def __init__(self, *, width: int, limit: float, norm: Norm, gate: torch.Tensor, up: torch.Tensor, down: torch.Tensor,
                 dtype: torch.dtype):
        E, ff = pad32(width), gate.shape[0]
        self.unit, self.norm = GatedUnit.clamped(limit), norm
        fp = pad32(ff)
        self.w_in = MatrixTiles(interleaved(gate, up, E), dtype, dense=True)
        self.w_out = MatrixTiles(spread(spread(down, 1, torch.arange(ff), fp), 0, torch.arange(width), E), dtype, dense=True)

    def run(self, res: Residual, step: StepLayout) -> None:
        if dense(step.T, self.w_in):
            h = ops.glu(F.linear(res.normed(self.norm), self.w_in.dense), self.unit)
        else:
            h = ops.linear(res.settle(), self.w_in, norm=self.norm.args, glu=self.unit)
        res.branch_out(h, self.w_out, step)


class ConcatProjection:
    """x <- W [x ; x0], W [E, 2 E]."""

    def __init__(self, *, width: int, weight: torch.Tensor, dtype: torch.dtype):
        E = pad32(width)
        cols = torch.cat([torch.arange(width), E + torch.arange(width)])
        self.w = MatrixTiles(spread(spread(weight, 1, cols, 2 * E), 0, torch.arange(width), E), dtype, dense=True)

    def run(self, res: Residual, x0: torch.Tensor) -> None:
        x = res.settle()
        if dense(x.shape[0], self.w):
            res.x = float_product(ops.concat(x, x0, res.dtype), self.w.dense)      # (the stream stays float32)
        else:
            res.x = ops.linear(x, self.w, x2=x0, float_out=(x.shape[1], 1.0))


class Retention:
    """q, k [heads dim, E], v, g [heads vdim, E], o [E, heads vdim]; decay: one per head."""

    def __init__(self, *, width: int, heads: int, dim: int, vdim: int, decay: Sequence[float], rot_base: float, rot_dims: int, eps: float,
                 q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, g: torch.Tensor, o: torch.Tensor, dtype: torch.dtype):
        if rot_dims % 2 or rot_dims > dim:
            raise ValueError(f"rotated dimensions {rot_dims} must be even and at most {dim}")
        if len(decay) != heads or not all(0.0 <= float(d) <= 1.0 for d in decay):
            raise ValueError(f"a decay between 0 and 1 for each of {heads} heads")
        dp, vp, dev = state_dim(dim), pad32(vdim), q.device
        self.sizes = dict(heads=heads, kv_heads=heads, dim=dp, vdim=vp, dim_n=dim, vdim_n=vdim, eps=float(eps))
        self.in_weight = torch.cat([padded_heads(q, heads, dp), padded_heads(k, heads, dp), padded_heads(v, heads, vp),
                                    padded_heads(g, heads, vp)])
        self.outs = [padded_heads(o, heads, vp, 1)]
        self.gate_at = 2 * heads * dp + heads * vp
        self.decay = torch.tensor([float(d) for d in decay], dtype=torch.float32, device=dev)
        self.log2_decay = torch.tensor([max(math.log2(d), -1e30) if d > 0 else -1e30 for d in map(float, decay)], dtype=torch.float32,
                                       device=dev)
        i = torch.arange(rot_dims // 2, dtype=torch.float64)
        self.freq, self.turn_key = (float(rot_base) ** (-2.0 * i / max(rot_dims, 1))).to(dev), (float(rot_base), rot_dims)

    def page_rows(self) -> List[int]:
        return []

    def tiling(self) -> Optional[QueryTiling]:
        return None

    def state_shapes(self) -> List[Tuple[Sequence[int], torch.dtype]]:
        z = self.sizes
        return [((z["heads"], z["dim"], z["vdim"]), torch.float32)]

    def run(self, proj: torch.Tensor, out: torch.Tensor, step: StepLayout, plans: Plans, held: Sequence[torch.Tensor]) -> None:
        ops.linear_state(proj, step, kind=ops.RETENTION, state=held[0], gate=proj[:, self.gate_at:self.gate_at + out.shape[1]], act="silu",
                         out=out, turns=step.rotations(self.freq, self.turn_key), decay=self.decay, log2_decay=self.log2_decay, **self.sizes)


class GatedDelta:
    """The gated delta rule with a decay per head and key channel.  q, k [kv_heads dim, E], v [heads vdim, E], their convolutions
    [channels, taps], b [heads, E], a1 [rank, E], a2 [heads dim, rank], dt_bias [heads dim], a_log [heads], norm [vdim],
    g1 [rank, E], g2 [heads vdim, rank], o [E, heads vdim]."""

    def __init__(self, *, width: int, heads: int, kv_heads: int, dim: int, vdim: int, taps: int, eps: float, q: torch.Tensor,
                 k: torch.Tensor, v: torch.Tensor, q_conv: torch.Tensor, k_conv: torch.Tensor, v_conv: torch.Tensor, b: torch.Tensor,
                 a1: torch.Tensor, a2: torch.Tensor, dt_bias: torch.Tensor, a_log: torch.Tensor, norm: torch.Tensor, g1: torch.Tensor,
                 g2: torch.Tensor, o: torch.Tensor, dtype: torch.dtype):
        if heads % kv_heads:
            raise ValueError(f"{heads} heads do not divide into {kv_heads} groups")
        dp, vp, rp, dev = state_dim(dim), pad32(vdim), max(pad32(a1.shape[0]), pad32(g1.shape[0])), q.device
        self.sizes = dict(heads=heads, kv_heads=kv_heads, dim=dp, vdim=vp, dim_n=dim, vdim_n=vdim, eps=float(eps))
        self.taps, self.dtype, self.rank = taps, dtype, rp
        self.channels = 2 * kv_heads * dp + heads * vp
        self.low_at = self.channels + pad32(heads)
        self.in_weight = torch.cat([padded_heads(q, kv_heads, dp), padded_heads(k, kv_heads, dp), padded_heads(v, heads, vp),
                                    padded_rows(b, pad32(heads)), padded_rows(a1, rp), padded_rows(g1, rp)])
        self.conv_w = torch.cat([padded_heads(q_conv, kv_heads, dp), padded_heads(k_conv, kv_heads, dp),
                                 padded_heads(v_conv, heads, vp)]).float().t().contiguous()
        n = heads * max(dp, vp)
        self.low_n = n
        self.w_low = MatrixTiles(torch.stack([padded_rows(padded_rows(padded_heads(a2, heads, dp), n), rp, 1),
                                              padded_rows(padded_rows(padded_heads(g2, heads, vp), n), rp, 1)]), dtype)
        self.dt_bias = padded_heads(dt_bias, heads, dp).float().contiguous()
        self.rate = torch.exp(a_log.double()).float().contiguous()
        self.norm_w = padded_rows(norm, vp).float().contiguous()
        self.outs = [padded_heads(o, heads, vp, 1)]

    def page_rows(self) -> List[int]:
        return []

    def tiling(self) -> Optional[QueryTiling]:
        return None

    def state_shapes(self) -> List[Tuple[Sequence[int], torch.dtype]]:
        """The state and the two halves of the convolution's tail."""
        z = self.sizes
        return [((z["heads"], z["dim"], z["vdim"]), torch.float32), ((2, self.taps - 1, self.channels), self.dtype)]

    def run(self, proj: torch.Tensor, out: torch.Tensor, step: StepLayout, plans: Plans, held: Sequence[torch.Tensor]) -> None:
        z, n = self.sizes, self.low_n
        low = ops.linear(proj[:, self.low_at:], self.w_low, x_gstride=self.rank, y_gstride=n)
        ops.linear_state(proj, step, kind=ops.DELTA, state=held[0], tail=held[1], beta=proj[:, self.channels:self.channels + z["heads"]],
                         z=low[:, :z["heads"] * z["dim"]], gate=low[:, n:n + z["heads"] * z["vdim"]], act="sigmoid", norm_w=self.norm_w,
                         conv_w=self.conv_w, rate=self.rate, dt_bias=self.dt_bias, out=out, **z)


def distance_buckets(n: int, buckets: int, far: float) -> torch.Tensor:
    """The row of a learned distance bias for distances 0 .. n - 1: one row each below half the rows, logarithmically wider ones up to
    `far` above, the last one beyond."""
    half = buckets // 2
    d = torch.arange(n, dtype=torch.float64)
    if buckets == 1 or n <= half:
        return torch.clamp(d, max=buckets - 1).long()
    if not float(far) > half:
        raise ValueError(f"a distance bias of {buckets} rows needs a largest distance beyond {half}")
    # (a distance that lies on an edge belongs above it, whatever the logarithms round to)
    up = torch.floor(torch.log(torch.clamp(d, min=1) / half) / math.log(float(far) / half) * (buckets - half) + 1e-9)
    return torch.where(d < half, d, torch.clamp(half + up, max=buckets - 1)).long()


class GroupedAttention:
    """Grouped-query softmax attention inside chunks of the sequence, with a learned bias by distance, a sink and an output gate per
    head.  q [heads dim, E], k [kv_heads dim, E], v [kv_heads vdim, E], rel [buckets, heads], sink [heads], g [heads, E],
    o [E, heads vdim]; q and k are divided by their root mean square per head."""

    def __init__(self, *, width: int, heads: int, kv_heads: int, dim: int, vdim: int, scale: float, chunk: int, bias_max: float, eps: float,
                 q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, rel: torch.Tensor, sink: torch.Tensor, g: torch.Tensor,
                 o: torch.Tensor, dtype: torch.dtype):
        if heads % kv_heads or chunk < 1:
            raise ValueError(f"{heads} heads over {kv_heads} key heads, chunks of {chunk}")
        log2e = math.log2(math.e)
        dp, vp = pad32(dim), pad32(vdim)
        self.sizes = dict(heads=heads, kv_heads=kv_heads, dim=dp, vdim=vp)
        self.scale, self.chunk, self.dim_n, self.eps = float(scale), int(chunk), dim, float(eps)
        self.in_weight = torch.cat([padded_heads(q, heads, dp), padded_heads(k, kv_heads, dp), padded_heads(v, kv_heads, vp),
                                    padded_rows(g, pad32(heads))])
        self.gate_at = (heads + kv_heads) * dp + kv_heads * vp
        rows = distance_buckets(chunk, rel.shape[0], bias_max).to(rel.device)
        self.bias = (rel.double()[rows] * log2e).t().float().contiguous()      # [heads, distances that occur]
        self.sink = (sink.double() * log2e).float().contiguous()
        self.outs = [padded_heads(o, heads, vp, 1)]

    def page_rows(self) -> List[int]:
        z = self.sizes
        return [z["kv_heads"] * (z["dim"] + z["vdim"])]

    def state_shapes(self) -> List[Tuple[Sequence[int], torch.dtype]]:
        return []

    def tiling(self) -> Optional[QueryTiling]:
        z = self.sizes
        return QueryTiling("grouped", z["heads"] // z["kv_heads"], z["kv_heads"], z["vdim"], self.chunk, (z["dim"], z["vdim"]))

    def run(self, proj: torch.Tensor, out: torch.Tensor, step: StepLayout, plans: Plans, held: Sequence[torch.Tensor]) -> None:
        z, plan = self.sizes, plans[self.tiling()]
        q = torch.empty((step.T, z["heads"] * z["dim"]), dtype=proj.dtype, device=proj.device)
        ops.kv_prep(proj, q, held[0], step, dim_n=self.dim_n, eps=self.eps, **z)
        ops.attention(q, held[0], step, plan.tiles, scale=self.scale, row_tiles=plan.row_tiles, splits=plan.splits, out=out,
                      chunk=self.chunk, bias=self.bias, sink=self.sink, gate=proj[:, self.gate_at:self.gate_at + z["heads"]], **z)


class TwoArms:
    """Two mixers over one input; half the sum of their outputs, each RMS-normed over the model width with its own weight."""

    def __init__(self, *, width: int, left, right, left_out: torch.Tensor, right_out: torch.Tensor, eps: float):
        E = pad32(width)
        self.arms, self.eps, self.width = (left, right), float(eps), width
        self.in_weight = torch.cat([left.in_weight, right.in_weight])
        self.outs = [left.outs[0], right.outs[0]]
        self.spans = [(a.in_weight.shape[0], a.outs[0].shape[1]) for a in self.arms]      # rows of proj, columns of the result
        for a in self.arms:
            del a.in_weight, a.outs                               # (they live on in the joined ones)
        self.out_norms = [padded_rows(w, E).float().contiguous() for w in (left_out, right_out)]

    def page_rows(self) -> List[int]:
        return [n for a in self.arms for n in a.page_rows()]

    def state_shapes(self) -> List[Tuple[Sequence[int], torch.dtype]]:
        return [s for a in self.arms for s in a.state_shapes()]

    def tiling(self) -> Optional[QueryTiling]:
        kinds = [a.tiling() for a in self.arms if a.tiling() is not None]
        if len(kinds) > 1:
            raise ValueError("at most one arm is an attention")
        return kinds[0] if kinds else None

    def run(self, proj: torch.Tensor, out: torch.Tensor, step: StepLayout, plans: Plans, held: Sequence[torch.Tensor]) -> None:
        pages = len(self.page_rows())
        pg, st, at, col = list(held[:pages]), list(held[pages:]), 0, 0
        for a, (rows, cols) in zip(self.arms, self.spans):
            n, m = len(a.page_rows()), len(a.state_shapes())
            a.run(proj[:, at:], out[:, col:col + cols], step, plans, pg[:n] + st[:m])
            pg, st, at, col = pg[n:], st[m:], at + rows, col + cols

    def merge(self, res: Residual, branches: Sequence[torch.Tensor], add: Optional[torch.Tensor]) -> None:
        ops.merge(res.settle(), branches[0], self.out_norms[0], branches[1], self.out_norms[1], add, n=self.width, eps=self.eps, scale=0.5)


class ParallelBlock:
    """x <- x + (mixer(h) + ff(h)), h = norm(x); gate, up [ff, E], down [E, ff] or None: no feed-forward."""

    def __init__(self, *, width: int, norm: Norm, mixer, gate: Optional[torch.Tensor], up: Optional[torch.Tensor],
                 down: Optional[torch.Tensor], unit: GatedUnit, dtype: torch.dtype):
        E = pad32(width)
        self.norm, self.mixer, self.unit, self.dtype = norm, mixer, unit, dtype
        self.n_in, self.n_mix = mixer.in_weight.shape[0], sum(w.shape[1] for w in mixer.outs)
        rows = padded_rows(mixer.in_weight, E, 1)
        self.ff = 0 if gate is None else pad32(gate.shape[0])
        tail = [] if gate is None else [padded_rows(padded_rows(down, self.ff, 1), E)]
        outs = [padded_rows(w, E) for w in mixer.outs]
        self.w_in = MatrixTiles(rows if gate is None else torch.cat([rows, interleaved(gate, up, E)]), dtype, dense=True)
        groups = [[*outs, *tail]] if len(outs) == 1 else [[w] for w in (*outs, *tail)]
        self.w_out = [MatrixTiles(torch.cat(g, dim=1), dtype, dense=True) for g in groups]
        del mixer.in_weight, mixer.outs      # (they live on in the tiles)

    def page_rows(self) -> List[int]:
        return self.mixer.page_rows()

    def state_shapes(self) -> List[Tuple[Sequence[int], torch.dtype]]:
        return self.mixer.state_shapes()

    def tiling(self) -> Optional[QueryTiling]:
        return self.mixer.tiling()

    def run(self, res: Residual, step: StepLayout, plans: Plans, held: Sequence[torch.Tensor]) -> None:
        T, m = step.T, self.n_mix
        rows = torch.empty((T, m + self.ff), dtype=self.dtype, device=res.x.device)      # [mixer cores | gated unit]
        if dense(T, self.w_in):
            proj = F.linear(res.normed(self.norm), self.w_in.dense)
            if self.ff:
                ops.glu(proj[:, self.n_in:], self.unit, out=rows[:, m:])
        else:
            proj = ops.linear(res.settle(), self.w_in, norm=self.norm.args, **(
                {"glu": self.unit, "glu_from": self.n_in, "glu_out": rows[:, m:]} if self.ff else {}))
        self.mixer.run(proj, rows[:, :m], step, plans, held)
        if len(self.w_out) == 1:
            res.branch_out(rows, self.w_out[0], step)
            return
        at, branches = 0, []
        for w in self.w_out[:2]:
            o = rows[:, at:at + w.K]
            branches.append(F.linear(o, w.dense) if dense(T, w) else ops.linear(o, w))
            at += w.K
        add = None
        if self.ff:
            if dense(T, self.w_out[2]):
                add = F.linear(rows[:, m:], self.w_out[2].dense)
            else:
                ops.linear(rows[:, m:], self.w_out[2], residual=True, out=res.settle())
        self.mixer.merge(res, branches, add)
