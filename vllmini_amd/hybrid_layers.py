"""Layers of decoders with recurrent blocks and latent attention, over hybrid_ops: each class lays its weights out for the kernels
once (heads, blocks and ranks zero-padded to multiples of 32, so no kernel has a ragged edge) and runs one step.

    LatentAttention   softmax attention whose cache holds one latent row per token, query side folded into the latent space
    RGLRU             the recurrent block: convolution, block-diagonal gates, gated linear recurrence
    ClampedGLU        the feed-forward with a clamped gated unit
    ConcatProjection  x <- W [x ; x0]

The residual stream is float32 (`Residual`).  Steps of few tokens run on the streaming kernels with everything fused around the
products (norm in front, gated unit / head gate / residual add behind); from DENSE_MIN_TOKENS tokens on (from DENSE_MIN_TOKENS_LARGE
for matrices of DENSE_LARGE elements) the products go to the vendor library (F.linear, as the prefill of the GPT-2 decoder does)
with one elementwise kernel between two of them.
"""
from __future__ import annotations

from typing import List, Optional, Sequence, Tuple

import torch
import torch.nn.functional as F

from . import hybrid_ops as ops
from .hybrid_ops import MatrixTiles, StepLayout, pad32

DENSE_MIN_TOKENS = 48
DENSE_MIN_TOKENS_LARGE, DENSE_LARGE = 17, 32 << 20


def dense(tokens: int, w: MatrixTiles) -> bool:
    return tokens >= DENSE_MIN_TOKENS or (tokens >= DENSE_MIN_TOKENS_LARGE and w.N * w.K >= DENSE_LARGE)


def float_product(x: torch.Tensor, w: torch.Tensor) -> torch.Tensor:
    """x W^T as float32, whatever the operands' type."""
    return torch.mm(x, w.t()) if x.dtype == torch.float32 else torch.mm(x, w.t(), out_dtype=torch.float32)


class Norm:
    """A layer norm's weight, zero-padded (padding columns of the stream stay zero)."""

    def __init__(self, weight: torch.Tensor, ld: int, eps: float):
        self.n, self.eps = weight.numel(), float(eps)
        self.weight = torch.zeros(ld, dtype=torch.float32, device=weight.device)
        self.weight[: self.n] = weight.float()

    @property
    def args(self) -> Tuple[torch.Tensor, int, float]:
        return self.weight, self.n, self.eps


class Head:
    """Final norm and vocabulary projection, logits float32 times a scale (folded into the norm's weight on the dense path)."""

    def __init__(self, norm: Norm, weight: torch.Tensor, ld: int, scale: float, dtype: torch.dtype):
        self.norm, self.vocab, self.scale, self.dtype = norm, weight.shape[0], float(scale), dtype
        self.w = MatrixTiles(spread(weight, 1, torch.arange(weight.shape[1]), ld), dtype, dense=True)
        self.scaled = (norm.weight * self.scale, norm.n, norm.eps)

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

    def page_row(self) -> int:
        return self.row

    def run(self, res: Residual, step: StepLayout, plan, cache: torch.Tensor) -> None:
        H, D = self.heads, self.row
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

    def state_shapes(self) -> List[Tuple[Sequence[int], torch.dtype]]:
        """The recurrence's state and the two halves of the convolution's tail (at least one row, so that a tensor exists)."""
        return [((self.width,), torch.float32), ((2, self.taps - 1, self.width), self.dtype)]

    def run(self, res: Residual, step: StepLayout, state: torch.Tensor, tail: torch.Tensor) -> None:
        yx = res.branch_in(self.norm, self.w_in, step, self.bias, self.dense_bias)
        o = ops.rglru(yx, step, conv_w=self.conv_w, conv_b=self.conv_b, gates=self.gates, gate_b=self.gate_b, decay=self.decay,
                      blocks=self.blocks, state=state, tail=tail)
        res.branch_out(o, self.w_o, step)


class ClampedGLU:
    """gate, up [ff, E], down [E, ff]."""

    def __init__(self, *, width: int, limit: float, norm: Norm, gate: torch.Tensor, up: torch.Tensor, down: torch.Tensor,
                 dtype: torch.dtype):
        E, ff = pad32(width), gate.shape[0]
        self.limit, self.norm = float(limit), norm
        fp = pad32(ff)
        both = torch.zeros((2 * fp, E), dtype=gate.dtype, device=gate.device)      # rows (gate 0, up 0, gate 1, up 1, ...)
        both[0:2 * ff:2, :width], both[1:2 * ff:2, :width] = gate, up
        self.w_in = MatrixTiles(both, dtype, dense=True)
        self.w_out = MatrixTiles(spread(spread(down, 1, torch.arange(ff), fp), 0, torch.arange(width), E), dtype, dense=True)

    def run(self, res: Residual, step: StepLayout) -> None:
        if dense(step.T, self.w_in):
            h = ops.glu(F.linear(res.normed(self.norm), self.w_in.dense), self.limit)
        else:
            h = ops.linear(res.settle(), self.w_in, norm=self.norm.args, glu_limit=self.limit)
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
