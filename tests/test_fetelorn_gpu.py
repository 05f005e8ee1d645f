"""The Fetelorn design on the GPU, mechanism by mechanism and end to end, against the plain restatement (oracle/fetelorn.py, float64).

float32 runs are compared tightly: there a wrong key, position, page or state shows at once.  bfloat16 runs are compared within what
rounding explains, and with inputs that make one key stand out where an average would hide it."""
from __future__ import annotations

import json
import os
import subprocess
import sys

import numpy as np
import pytest
import torch

from oracle import fetelorn as plain
from tests import fetelorn_cases as cases
from tests.test_voduvik_gpu import BOTH, close, dev, i32, layout, logits_close

pytestmark = pytest.mark.gpu
REPO = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
LOG2E = 1.4426950408889634


# ---- norms, gated unit, merge ----------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("dtype", BOTH)
@pytest.mark.parametrize("M", [1, 7, 40, 130])
@pytest.mark.parametrize("split,ff,K", [(32, 40, 64), (96, 96, 288), (64, 33, 800)])
def test_one_product_stores_columns_and_gates_the_others(dtype, M, split, ff, K):
    from vllmini_amd import hybrid_ops as ops
    from vllmini_amd.hybrid_layers import interleaved

    g = torch.Generator().manual_seed(M + K)
    rnd = lambda *s: torch.randn(*s, generator=g)      # noqa: E731
    n = K - 5
    x, nw = (rnd(M, K) * 2 + 3).to(dev()), torch.zeros(K, device=dev())
    x[:, n:] = 0
    nw[:n] = 1 + 0.5 * rnd(n).to(dev())
    w, gate, up = (torch.cat([rnd(m, n), torch.zeros(m, K - n)], 1).div(K ** 0.5).to(torch.bfloat16).to(dev()) for m in (split, ff, ff))
    h = torch.zeros(M, K, dtype=torch.float64, device=dev())
    h[:, :n] = plain.unit_rms(x[:, :n].double(), 1e-3) * nw[:n].double()
    t = ops.MatrixTiles(torch.cat([w, interleaved(gate, up, K)]), dtype)
    rest = torch.full((M, 64 + ops.pad32(ff)), 7.0, dtype=dtype, device=dev())
    got = ops.linear(x, t, norm=(nw, n, 1e-3, True), glu=ops.SILU_UNIT, glu_from=split, glu_out=rest[:, 64:])
    assert got.shape == (M, split)
    close(got, h @ w.double().T, dtype, tol32=1e-4)
    close(rest[:, 64:64 + ff], plain.silu(h @ gate.double().T) * (h @ up.double().T), dtype, tol32=1e-4, tol16=3e-2)
    assert (rest[:, :64] == 7).all() and not rest[:, 64 + ff:].any()
    close(ops.add_norm(x, None, (nw, n, 1e-3, True), dtype), h, dtype, tol32=1e-5)
    close(ops.linear(x, t, norm=(nw, n, 1e-3, True)), h @ torch.cat([w, interleaved(gate, up, K)]).double().T, dtype, tol32=1e-4)


@pytest.mark.parametrize("dtype", BOTH)
@pytest.mark.parametrize("n", [50, 96, 1500, 9001])
def test_merge_of_two_normed_branches(dtype, n):
    from vllmini_amd import hybrid_ops as ops

    g = torch.Generator().manual_seed(n)
    ld = ops.pad32(n)

    def padded(dt, scale=1.0):
        t = torch.zeros(5, ld, dtype=dt, device=dev())
        t[:, :n] = (torch.randn(5, n, generator=g) * scale).to(dt).to(dev())
        return t

    x, a, b, add, wa, wb = padded(torch.float32, 3), padded(dtype, 20), padded(dtype, 0.01), padded(dtype), padded(torch.float32)[0], padded(torch.float32)[0]
    for extra in (None, add):
        y = x.clone()
        ops.merge(y, a, wa, b, wb, extra, n=n, eps=1e-5, scale=0.5)
        want = x.double() + 0.5 * torch.cat([plain.unit_rms(a[:, :n].double(), 1e-5) * wa[:n].double() + plain.unit_rms(b[:, :n].double(), 1e-5) *
                                             wb[:n].double(), torch.zeros(5, ld - n, device=dev())], 1) + (0 if extra is None else add.double())
        close(y, want, torch.float32)


# ---- linear attention with a matrix state ------------------------------------------------------------------------------------------
def heads_at(n, per, ld):
    """Where n heads of `per` entries lie when each gets ld places."""
    return (torch.arange(n)[:, None] * ld + torch.arange(per)[None]).reshape(-1).to(dev())


class _State:
    """Operands of the linear-attention kernels for a layer, the plain result for a whole sequence, and the run of a step."""

    def __init__(self, layer, slots, dtype):
        self.layer, self.dtype, self.z = layer, dtype, layer.sizes
        self.held = [torch.full((slots, *s), 3.0, device=dev()).to(dt) for s, dt in layer.state_shapes()]      # former owners' leavings
        z = self.z
        self.cols = [heads_at(z["kv_heads"], z["dim_n"], z["dim"]), heads_at(z["kv_heads"], z["dim_n"], z["dim"]),
                     heads_at(z["heads"], z["vdim_n"], z["vdim"])]
        self.cols[1] = self.cols[1] + z["kv_heads"] * z["dim"]
        self.cols[2] = self.cols[2] + 2 * z["kv_heads"] * z["dim"]

    def inputs(self, T, seed):
        """(what the plain form takes, proj, the other operands of the kernel)"""
        g, z = torch.Generator().manual_seed(seed), self.z
        rnd = lambda *s: torch.randn(*s, generator=g).to(self.dtype).to(dev())      # noqa: E731
        H, C = z["heads"], 2 * z["kv_heads"] * z["dim"] + z["heads"] * z["vdim"]
        qkv = [rnd(T, len(c)) for c in self.cols]
        proj = torch.zeros(T, C + 64, dtype=self.dtype, device=dev())
        for t, c in zip(qkv, self.cols):
            proj[:, c] = t
        beta, zed, gate = 2 * rnd(T, H), 2 * rnd(T, H * z["dim_n"]), rnd(T, H * z["vdim_n"])
        proj[:, C:C + H] = beta
        zp = torch.zeros(T, H * z["dim"], dtype=self.dtype, device=dev())
        zp[:, heads_at(H, z["dim_n"], z["dim"])] = zed
        gp = torch.zeros(T, H * z["vdim"], dtype=self.dtype, device=dev())
        gp[:, heads_at(H, z["vdim_n"], z["vdim"])] = gate
        return [t.double().cpu() for t in (*qkv, beta, zed, gate)], (proj, zp, gp)

    def run(self, ops_in, step):
        from vllmini_amd import hybrid_ops as ops

        proj, zp, gp = ops_in
        z, L = self.z, self.layer
        out = torch.full((step.T, z["heads"] * z["vdim"]), float("nan"), dtype=self.dtype, device=dev())
        C = 2 * z["kv_heads"] * z["dim"] + z["heads"] * z["vdim"]
        if hasattr(L, "decay"):
            ops.linear_state(proj, step, kind=ops.RETENTION, state=self.held[0], gate=gp, act="silu", out=out, decay=L.decay,
                             turns=step.rotations(L.freq, L.turn_key), log2_decay=L.log2_decay, **z)
        else:
            ops.linear_state(proj, step, kind=ops.DELTA, state=self.held[0], tail=self.held[1], beta=proj[:, C:C + z["heads"]], z=zp, gate=gp,
                             act="sigmoid", out=out, norm_w=L.norm_w, conv_w=L.conv_w, rate=L.rate, dt_bias=L.dt_bias, **z)
        return out[:, heads_at(z["heads"], z["vdim_n"], z["vdim"])]


def retention_case(heads, dim, vdim, rot, decay, dtype, slots=5, base=300.0):
    from vllmini_amd.hybrid_layers import Retention

    E = 32
    zero = lambda n: torch.zeros(n, E, device=dev())      # noqa: E731
    k = _State(Retention(width=E, heads=heads, dim=dim, vdim=vdim, decay=decay, rot_base=base, rot_dims=rot, eps=1e-4, q=zero(heads * dim),
                         k=zero(heads * dim), v=zero(heads * vdim), g=zero(heads * vdim), o=zero(heads * vdim).t(), dtype=dtype), slots, dtype)

    def want(x, first=0):
        q, kk, v, _, _, gate = x
        T = len(q)
        q, kk = (torch.stack([plain.rotate(t.view(T, heads, dim)[i], first + i, base, rot) for i in range(T)]) for t in (q, kk))
        o, _ = plain.retain(q, kk * dim ** -0.5, v.view(T, heads, vdim), torch.tensor(decay, dtype=torch.float64))
        return plain.unit_rms(o, 1e-4).reshape(T, -1) * plain.silu(gate)

    return k, want


def delta_case(heads, kv_heads, dim, vdim, taps, dtype, slots=5, rate=0.0, bias=-3.0):
    from vllmini_amd.hybrid_layers import GatedDelta

    E, g = 32, torch.Generator().manual_seed(heads * dim + taps)
    zero = lambda n: torch.zeros(n, E, device=dev())      # noqa: E731
    rnd = lambda *s: torch.randn(*s, generator=g)         # noqa: E731
    w = {"q_conv": rnd(kv_heads * dim, taps), "k_conv": rnd(kv_heads * dim, taps), "v_conv": rnd(heads * vdim, taps),
         "dt_bias": rnd(heads * dim) + bias, "a_log": 0.5 * rnd(heads) + rate, "norm": 1 + 0.3 * rnd(vdim)}
    w = {n: t.to(torch.bfloat16).to(dev()) for n, t in w.items()}
    k = _State(GatedDelta(width=E, heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, taps=taps, eps=1e-4, q=zero(kv_heads * dim),
                          k=zero(kv_heads * dim), v=zero(heads * vdim), b=zero(heads), a1=zero(4), a2=torch.zeros(heads * dim, 4, device=dev()),
                          g1=zero(4), g2=torch.zeros(heads * vdim, 4, device=dev()), o=zero(heads * vdim).t(), dtype=dtype, **w), slots, dtype)
    p = {n: t.double().cpu() for n, t in w.items()}

    def want(x):
        q, kk, v, beta, z, gate = x
        T, rep = len(q), heads // kv_heads
        q, kk, v = (plain.silu(plain.causal_conv(t, p[n + "_conv"])) for t, n in ((q, "q"), (kk, "k"), (v, "v")))
        q = (plain.unit_length(q.view(T, kv_heads, dim)) * dim ** -0.5).repeat_interleave(rep, 1)
        kk = plain.unit_length(kk.view(T, kv_heads, dim)).repeat_interleave(rep, 1)
        g_ = torch.exp(-torch.exp(p["a_log"])[None, :, None] * plain.softplus(z + p["dt_bias"]).view(T, heads, dim))
        o, _ = plain.delta_rule(q, kk, v.view(T, heads, vdim), g_, torch.sigmoid(beta))
        return (plain.unit_rms(o, 1e-4) * p["norm"] * torch.sigmoid(gate).view(T, heads, vdim)).reshape(T, -1)

    return k, want


def _portions(k, want, T, cuts, slots):
    """Sequences cut differently in shared steps, states in slots whose former contents are garbage; against whole plain sequences."""
    n_seq = len(cuts)
    seqs = [k.inputs(T, 10 + i) for i in range(n_seq)]
    cuts, at, flips, out = [list(c) for c in cuts], [0] * n_seq, [0] * n_seq, [[] for _ in range(n_seq)]
    while any(a < T for a in at):
        live = [i for i in range(n_seq) if at[i] < T]
        n = [cuts[i].pop(0) if cuts[i] else T - at[i] for i in live]
        step = layout(n, [at[i] for i in live], [[0]] * len(live), 64, [slots[i] for i in live], [flips[i] for i in live], pos_slots=False)
        got = k.run([torch.cat([seqs[i][1][j][at[i]:at[i] + c] for i, c in zip(live, n)]) for j in range(3)], step)
        for i, c, g in zip(live, n, got.split(n)):
            out[i].append(g)
            at[i] += c
            flips[i] ^= 1
    for i in range(n_seq):
        close(torch.cat(out[i]), want(seqs[i][0]), k.dtype, tol32=5e-5, tol16=1.5e-2)


CUTS = [[70], [15, 2, 16, 3, 1, 1, 17, 2, 9], [1] * 5 + [2, 31, 1, 2]]


@pytest.mark.parametrize("dtype", BOTH)
@pytest.mark.parametrize("heads,dim,vdim,rot,decay", [(1, 10, 33, 10, (1.0,)), (3, 20, 24, 12, (0.5, 0.01, 0.999)), (2, 64, 160, 36, (0.9, 0.99)),
                                                      (2, 150, 40, 2, (0.7, 0.95)), (1, 300, 96, 300, (0.98,)), (4, 96, 16, 0, (0.0, 0.3, 0.6, 0.9))])
def test_retention_over_portions_of_every_size(dtype, heads, dim, vdim, rot, decay):
    k, want = retention_case(heads, dim, vdim, rot, decay, dtype)
    _portions(k, want, 70, CUTS, [4, 0, 2])


@pytest.mark.parametrize("dtype", BOTH)
@pytest.mark.parametrize("heads,kv_heads,dim,vdim,taps,rate", [(1, 1, 16, 8, 4, 0.0), (4, 2, 24, 40, 3, 0.0), (6, 1, 40, 20, 1, 1.0),
                                                               (2, 2, 100, 33, 7, 3.0), (3, 3, 64, 150, 2, -1.0), (2, 1, 140, 70, 4, 4.0),
                                                               (1, 1, 260, 48, 4, 0.5)])
def test_delta_rule_over_portions_of_every_size(dtype, heads, kv_heads, dim, vdim, taps, rate):
    """Decays from a fraction of a token to hundreds of tokens: chunks of both kinds, the deep ones and the shallow ones."""
    k, want = delta_case(heads, kv_heads, dim, vdim, taps, dtype, rate=rate)
    _portions(k, want, 70, CUTS, [4, 0, 2])


@pytest.mark.parametrize("kind", ["retention", "delta"])
def test_many_states_take_two_column_tiles_a_workgroup(kind):
    """Enough (sequence, head, columns) for the chip: the walk's wider form, against the same sequences alone."""
    B, T = 66, 35
    k, want = (retention_case(4, 24, 64, 24, (0.9, 0.5, 0.99, 1.0), torch.float32, B) if kind == "retention" else
               delta_case(4, 2, 40, 64, 4, torch.float32, B))
    seqs = [k.inputs(T, 100 + i) for i in range(B)]
    out = []
    for first, n in ((0, 18), (18, 17)):
        step = layout([n] * B, [first] * B, [[0]] * B, 64, flips=[int(first > 0)] * B, pos_slots=False)
        out.append(k.run([torch.cat([s[1][j][first:first + n] for s in seqs]) for j in range(3)], step).view(B, n, -1))
    got = torch.cat(out, 1)
    for i in (0, 31, 65):
        close(got[i], want(seqs[i][0]), torch.float32, tol32=5e-5)
    alone = k.run(seqs[7][1], layout([T], [0], [[0]], 64, pos_slots=False))
    close(got[7], alone, torch.float32, tol32=1e-5)


def test_delta_rule_survives_decays_that_leave_nothing():
    k, want = delta_case(2, 1, 32, 32, 4, torch.float32, rate=6.0, bias=8.0)
    _portions(k, want, 40, [[40], [17, 2, 21], [1] * 40], [1, 0, 3])


@pytest.mark.parametrize("dtype", BOTH)
@pytest.mark.parametrize("kind", ["retention", "delta", "delta_sliced"])
def test_states_decode_alone_as_in_a_padded_batch(dtype, kind):
    """Single tokens of many sequences, padding entries behind them as in a captured batch; untouched slots stay as they are."""
    from vllmini_amd import hybrid_ops as ops

    T, B = 12, 9
    k, want = (retention_case(2, 20, 24, 20, (0.9, 0.5), dtype, 12) if kind == "retention" else
               delta_case(2, 1, 24, 40, 4, dtype, 12) if kind == "delta" else delta_case(2, 1, 24, 150, 3, dtype, 12))
    seqs = [k.inputs(T, 50 + i) for i in range(B)]
    ref = [want(s[0]) for s in seqs]
    before = [t[B:].clone() for t in k.held]
    for t in range(T):
        step = layout([1] * B, [t] * B, [[0]] * B, 64, flips=[t & 1] * B, pos_slots=False)
        f = dict(step.fields)
        for n, fill in (("tok_seq", -1), ("tok_pos", 0), ("tok_slot", -1), ("q_start", B), ("q_len", 0), ("ctx", 0), ("state_slot", B), ("flip", 0)):
            f[n] = torch.cat([f[n], i32([fill, fill])])
        f["table"] = i32([[0]] * (B + 2))
        pad = ops.StepLayout(f, B + 2, B + 2, 64, True, False, 1, t + 1)
        got = k.run([torch.cat([s[1][j][t:t + 1] for s in seqs] + [torch.full_like(seqs[0][1][j][:1], float("nan"))] * 2) for j in range(3)], pad)
        for i in range(B):
            close(got[i], ref[i][t], dtype, tol32=1e-4, tol16=3e-2)
    assert all(torch.equal(a, t[B:]) for a, t in zip(before, k.held))


def test_retention_keeps_a_long_memory_and_far_angles():
    """Decay one: a thousand tokens later the first key still answers alone, at the angle of its distance."""
    k, _ = retention_case(1, 32, 32, 32, (1.0,), torch.float32, base=10000.0)
    T = 1500
    x, (proj, zp, gp) = k.inputs(T, 3)
    proj[1:, 32:64] = 0                                   # one key only
    gp.fill_(1.0)
    got = k.run((proj, zp, gp), layout([T], [0], [[0]], 64, pos_slots=False)).double().cpu()
    q, v = proj[:, :32].double().cpu(), proj[0, 64:96].double().cpu()
    key = proj[0, 32:64].double().cpu()
    for t in (0, 1, 15, 16, 17, 700, 1023, 1499):
        s = float(plain.rotate(q[t], t, 10000.0, 32) @ key) * 32 ** -0.5
        close(got[t], plain.unit_rms(s * v, 1e-4) * float(plain.silu(torch.tensor(1.0, dtype=torch.float64))), torch.float32, tol32=2e-3 if abs(s) < 0.05 else 2e-4)


# ---- attention -----------------------------------------------------------------------------------------------------------------------
def _attend(dtype, H, G, dim, vdim, chunk, counts, ctx, page, row_tiles=4, splits=1, spike=(), seed=0, parts=("bias", "sink", "gate")):
    from vllmini_amd import hybrid_ops as ops

    D, B, rep = dim + vdim, len(counts), H // G
    g = torch.Generator().manual_seed(seed)
    total = [c + n for c, n in zip(ctx, counts)]
    per = [-(-t // page) for t in total]
    pages = torch.randperm(sum(per) + 3, generator=g).numpy()
    cache = torch.randn(len(pages), page, G * D, generator=g).to(dtype).to(dev())
    tables = np.zeros((B, max(per)), dtype=np.int64)
    at = 0
    for b in range(B):
        tables[b, :per[b]] = pages[at:at + per[b]]
        at += per[b]
    q = torch.randn(sum(counts), H, dim, generator=g).to(dtype).to(dev())
    scale, buckets, far = 1.7 * dim ** -0.5, 8, max(chunk, 5) * 0.8
    rel, sink = 2 * torch.randn(buckets, H, generator=g, dtype=torch.float64), torch.randn(H, generator=g, dtype=torch.float64)
    if "bias" not in parts:
        rel.zero_()
    if "sink" not in parts:
        sink.fill_(-1e4)
    flat = cache.view(-1, G, D)
    row = lambda b, p: int(tables[b, p // page]) * page + p % page      # noqa: E731
    for b, t, p in spike:      # query `t` of entry b meets a key of its own direction at position p: that score stands far out
        u = torch.randn(dim, generator=g)
        u = (u / u.norm() * (25 / scale) ** 0.5).to(dtype).to(dev())
        q[sum(counts[:b]) + t] = u
        flat[row(b, p), :, :dim] = u
    gate = torch.randn(sum(counts), 32, generator=g).to(dtype).to(dev()) if "gate" in parts else None
    step = layout(counts, ctx, tables, page)
    rt = ops.attention_row_tiles(dim, vdim, row_tiles, dtype)
    tiles = [(b, r) for b in range(B) for r in range(0, counts[b] * rep, 16 * rt)]
    tiles.insert(1, (-1, -1))
    dist = torch.tensor([plain.distance_bucket(d, buckets, far) for d in range(chunk)])
    out = torch.zeros(sum(counts), H * vdim + 32, dtype=dtype, device=dev())
    ops.attention(q.view(-1, H * dim), cache, step, i32(tiles), heads=H, kv_heads=G, dim=dim, vdim=vdim, scale=scale, row_tiles=rt, splits=splits,
                  out=out[:, 32:], chunk=chunk, bias=(rel[dist] * LOG2E).t().float().contiguous().to(dev()) if "bias" in parts else None,
                  sink=(sink * LOG2E).float().to(dev()) if "sink" in parts else None, gate=None if gate is None else gate[:, 5:5 + H])
    want, at = [], 0
    keys = flat.double().cpu()
    for b in range(B):
        seq = keys[[row(b, p) for p in range(total[b])]]
        for t in range(counts[b]):
            i = ctx[b] + t
            lo = i // chunk * chunk
            K, V = (seq[lo:i + 1, :, :dim].repeat_interleave(rep, 1), seq[lo:i + 1, :, dim:].repeat_interleave(rep, 1))
            s = (K * q[at].double().cpu()[None]).sum(-1) * scale + rel[[plain.distance_bucket(i - j, buckets, far) for j in range(lo, i + 1)]]
            m = torch.maximum(s.max(0).values, sink)
            e = torch.exp(s - m)
            o = (e[..., None] * V).sum(0) / (e.sum(0) + torch.exp(sink - m))[:, None]
            want.append((o * (1 if gate is None else torch.sigmoid(gate[at, 5:5 + H].double().cpu())[:, None])).reshape(-1))
            at += 1
    assert not out[:, :32].any()
    return out[:, 32:], torch.stack(want)


@pytest.mark.parametrize("dtype", BOTH)
@pytest.mark.parametrize("H,G,dim,vdim,chunk,page", [(1, 1, 32, 32, 7, 16), (6, 2, 64, 32, 100, 64), (5, 5, 32, 96, 64, 32), (20, 1, 128, 128, 48, 16),
                                                     (8, 4, 160, 64, 300, 64), (3, 3, 96, 288, 33, 8), (4, 2, 256, 320, 40, 64)])
def test_attention_over_pages_and_chunks(dtype, H, G, dim, vdim, chunk, page):
    for counts, ctx in (([1], [0]), ([1, 1, 1], [63, 64, 130]), ([70, 1, 2], [0, 99, 62]), ([33], [95])):
        for rt in (1, 4) if dtype == torch.bfloat16 else (1,):
            for sp in (1, 3):
                got, want = _attend(dtype, H, G, dim, vdim, chunk, counts, ctx, page, rt, sp)
                close(got, want, dtype, tol32=3e-5, tol16=1.5e-2)


@pytest.mark.parametrize("parts", [(), ("bias",), ("sink",), ("gate",)])
def test_attention_without_some_of_its_parts(parts):
    for rt, dtype in ((1, torch.float32), (4, torch.bfloat16)):
        got, want = _attend(dtype, 4, 2, 32, 64, 50, [40, 1], [30, 77], 16, rt, 2, parts=parts)
        close(got, want, dtype, tol32=3e-5, tol16=1.5e-2)


@pytest.mark.parametrize("dtype", BOTH)
@pytest.mark.parametrize("decoded", [False, True])
def test_attention_sees_just_inside_its_chunk_and_not_just_outside(dtype, decoded):
    """One score stands out: at the chunk's first and last key, at page borders inside it, at the query's own position — and one token
    outside either end, where it must not be seen."""
    c = chunk = 136
    page = 16
    for i, p in ((2 * c - 1, c), (2 * c - 1, c - 1), (2 * c, 2 * c - 1), (2 * c, 2 * c), (2 * c + 10, 2 * c), (2 * c + 10, 2 * c - 1),
                 (3 * c - 1, 399), (3 * c - 1, 400), (3 * c - 1, 2 * c), (2 * c + 60, 2 * c + 60), (2 * c + 60, 2 * c + 61)):
        n = 1 if decoded else 40
        if decoded and p > i:
            continue
        ctx = i if decoded else i - 20
        seen = p // chunk == i // chunk and p <= i
        got, want = _attend(dtype, 4, 2, 32, 32, chunk, [n], [ctx], page, splits=2, spike=[(0, i - ctx, p)], seed=p, parts=("sink",))
        close(got, want, dtype)
        other, w2 = _attend(dtype, 4, 2, 32, 32, chunk, [n], [ctx], page, splits=2, seed=p, parts=("sink",))
        assert seen or not torch.equal(got, other)        # (the query itself was changed too)


@pytest.mark.parametrize("dtype", BOTH)
def test_kv_prep_normalises_and_writes_the_cache(dtype):
    from vllmini_amd import hybrid_ops as ops

    H, G, dim, dim_n, vdim, page = 6, 2, 160, 150, 64, 16
    g = torch.Generator().manual_seed(4)
    counts, ctx = [3, 1], [30, 77]
    tables = np.arange(12).reshape(2, 6)[:, ::-1].copy()
    step = layout(counts, ctx, tables, page)
    proj = torch.zeros(4, (H + G) * dim + G * vdim + 32)
    proj[:, :(H + G) * dim].view(4, H + G, dim)[:, :, :dim_n] = 4 * torch.randn(4, H + G, dim_n, generator=g)
    proj[:, (H + G) * dim:] = torch.randn(4, G * vdim + 32, generator=g)
    proj = proj.to(dtype).to(dev())
    q = torch.full((4, H * dim), 3.0, dtype=dtype, device=dev())
    cache = torch.full((13, page, G * (dim + vdim)), 9.0, dtype=dtype, device=dev())
    ops.kv_prep(proj, q, cache, step, heads=H, kv_heads=G, dim=dim, vdim=vdim, dim_n=dim_n, eps=1e-5)
    P, flat, used = proj.double().cpu(), cache.view(-1, G, dim + vdim), []
    for t in range(4):
        b, pos = (0, 30 + t) if t < 3 else (1, 77)
        r = int(tables[b, pos // page]) * page + pos % page
        used.append(r)
        x = P[t, :(H + G) * dim].view(H + G, dim)
        unit = torch.cat([plain.unit_rms(x[:, :dim_n], 1e-5), torch.zeros(H + G, dim - dim_n)], 1)
        close(q[t].view(H, dim), unit[:H], dtype, tol16=6e-3)
        close(flat[r, :, :dim], unit[H:], dtype, tol16=6e-3)
        assert torch.equal(flat[r, :, dim:], proj[t, (H + G) * dim:(H + G) * dim + G * vdim].view(G, vdim))
    rest = torch.ones(flat.shape[0], dtype=torch.bool, device=dev())
    rest[used] = False
    assert (flat[rest] == 9).all()


# ---- the whole decoder -------------------------------------------------------------------------------------------------------------
_PLAIN = {}
N = 90


def expected(name, toks):
    key = (name, tuple(toks))
    if key not in _PLAIN:
        c = cases.CONFIGS[name]
        _PLAIN[key] = plain.forward(c, cases.tensors(c), toks)
    return _PLAIN[key]


def decoder(name, dtype, max_tokens=640, max_seqs=4, page=16, **kw):
    from vllmini_amd.fetelorn import FetelornConfig, build_model
    from vllmini_amd.hybrid_decoder import HybridDecoder

    c = cases.CONFIGS[name]
    m = build_model(FetelornConfig.from_json(c), cases.tensors(c), dtype, dev())
    d = HybridDecoder(m, m.make_pool(max_tokens, max_seqs, page), **kw)
    g = torch.Generator(device=dev()).manual_seed(3)
    for t in d.pool.row_pages + d.pool.state:          # stale contents must never matter
        t.copy_(torch.empty(t.shape, device=dev()).uniform_(-4, 4, generator=g))
    return d


@pytest.mark.parametrize("dtype", BOTH)
@pytest.mark.parametrize("name", sorted(cases.CONFIGS))
def test_whole_prompt_and_the_stream_after_every_layer(name, dtype):
    toks = cases.tokens(cases.CONFIGS[name], N, 1)
    want, streams = expected(name, toks)
    d = decoder(name, dtype)
    d.pool.open(0)
    d.tap = []
    got = d.step([0], [toks], [list(range(N))])
    logits_close(got, want, dtype)
    assert len(d.tap) == len(streams)
    for a, b in zip(d.tap, streams):
        close(a, b, dtype, tol32=1e-4, tol16=8e-2)


@pytest.mark.parametrize("tokens", [1, 10 ** 9], ids=["vendor", "streaming"])
@pytest.mark.parametrize("name", sorted(cases.CONFIGS))
def test_both_kinds_of_products_give_the_same_logits(name, tokens, monkeypatch):
    from vllmini_amd import hybrid_layers

    monkeypatch.setattr(hybrid_layers, "DENSE_MIN_TOKENS", tokens)
    toks = cases.tokens(cases.CONFIGS[name], N, 1)
    for dtype in BOTH:
        d = decoder(name, dtype)
        d.pool.open(0)
        first = d.step([0], [toks[:60]], [list(range(60))])
        rest = torch.cat([d.decode([0], [t]) for t in toks[60:70]])
        logits_close(torch.cat([first, rest]), expected(name, toks)[0][:70], dtype)


@pytest.mark.parametrize("dtype", BOTH)
@pytest.mark.parametrize("name", sorted(cases.CONFIGS))
def test_portions_single_tokens_and_neighbours_do_not_change_the_logits(name, dtype):
    """Unequal requests cut in every way, pages and slots given back and used again, requests left out of steps."""
    c = cases.CONFIGS[name]
    lens = [90, 40, 3, 1, 66, 90]
    toks = [cases.tokens(c, N, 1)[:n] for n in lens]       # prefixes of one sequence: one plain run checks all of them
    want = expected(name, cases.tokens(c, N, 1))[0]
    d = decoder(name, dtype, max_tokens=16 * 14, max_seqs=3)
    rng = np.random.default_rng(5)
    sizes = [[90], [2, 3, 2, 31, 2], [1, 2], [1], [64, 2], [17] + [2] * 20 + [1] * 33]
    waiting, live, at, rows = list(range(6)), [], {}, {i: [] for i in range(6)}
    while waiting or live:
        while waiting and len(live) < 3 and len(d.pool.free_blocks) >= sum(-(-lens[i] // 16) for i in live) + -(-lens[waiting[0]] // 16) - \
                sum(len(d.pool.allocated_blocks[i]) for i in live):
            i = waiting.pop(0)
            d.pool.open(i)
            live.append(i)
            at[i] = 0
        now = [i for i in live if len(live) == 1 or rng.random() < 0.8] or live[:1]
        n = [sizes[i].pop(0) if sizes[i] else lens[i] - at[i] for i in now]
        got = d.step(now, [toks[i][at[i]:at[i] + k] for i, k in zip(now, n)], [list(range(k)) for k in n])
        for i, k, g in zip(now, n, got.split(n)):
            rows[i].append(g.cpu())
            at[i] += k
            if at[i] == lens[i]:
                d.pool.free(i)
                live.remove(i)
    for i in range(6):
        logits_close(torch.cat(rows[i]), want[: lens[i]], dtype)
    assert len(d.pool.free_blocks) == 14 and d.pool.free_state_slots == 3


@pytest.mark.parametrize("dtype", BOTH)
def test_long_decoding_from_one_token(dtype):
    name, n = "mixed", 200
    toks = cases.tokens(cases.CONFIGS[name], n, 9)
    want = expected(name, toks)[0]
    d = decoder(name, dtype, page=32)
    first = d.prefill(0, toks[:1])
    got = torch.cat([first[None]] + [d.decode([0], torch.tensor([t], device=dev())).clone() for t in toks[1:]])
    logits_close(got, want, dtype, tol32=5e-4)


@pytest.mark.parametrize("vendor", [False, True], ids=["streaming", "vendor"])
@pytest.mark.parametrize("name", ["mixed", "large_heads"])
def test_graph_replay_equals_eager_steps(name, vendor, monkeypatch):
    """Both ways a layer's products may run, captured; eager steps run between the replays, and positions move on in both."""
    from vllmini_amd import hybrid_layers

    if vendor:
        monkeypatch.setattr(hybrid_layers, "DENSE_MIN_TOKENS", 1)
    c = cases.CONFIGS[name]
    a, b = decoder(name, torch.bfloat16, pad_batch_to=4), decoder(name, torch.bfloat16)
    prompts = [cases.tokens(c, n, n) for n in (5, 30, 100)]
    la, lb = a.prefill_batch([0, 1, 2], prompts), b.prefill_batch([0, 1, 2], prompts)
    for i in range(40):      # every replay against the eager step; the batch shrinks once, contexts cross a split bucket
        ids = [0, 1, 2] if i < 25 else [0, 2]
        tok = b.greedy(lb[: len(ids)] if i != 25 else lb[[0, 2]])
        la, lb = a.decode(ids, tok, use_graph=True).clone(), b.decode(ids, tok).clone()
        logits_close(la, lb, torch.bfloat16, tol16=2e-2)
    assert len(a._sets) >= 1 and all(s["graph"] is not None for s in a._sets.values())
    assert torch.isfinite(la).all()


# ---- generation through the framework's entry points ----------------------------------------------------------------------------------
def _plain_greedy(name, prompt, n):
    c = cases.CONFIGS[name]
    w, seq = cases.tensors(c), list(prompt)
    for _ in range(n):
        seq.append(int(plain.forward(c, w, seq)[0][-1].argmax()))
    return seq


@pytest.fixture(scope="module")
def greedy_case():
    name = "mixed"
    prompts = [cases.tokens(cases.CONFIGS[name], n, 40 + n) for n in (1, 19, 34)]
    return name, prompts, [_plain_greedy(name, p, 10) for p in prompts]


@pytest.mark.parametrize("kw", [{}, {"use_graph": True}, {"prefill_chunk": 7}, {"prefill_chunk": 16, "use_graph": True}, {"preempt_after": 4}],
                         ids=["plain", "graph", "chunks", "chunks+graph", "preempted"])
def test_greedy_generation_through_the_scheduler(kw, greedy_case):
    from vllmini_amd.scheduler import BatchScheduler

    name, prompts, want = greedy_case
    kw, blocks = dict(kw), 12
    after = kw.pop("preempt_after", 0)
    d = decoder(name, torch.float32, max_tokens=16 * blocks, max_seqs=3)
    sch = BatchScheduler(d, max_length=46, eos_token_id=-1, max_batch=3, sampler=lambda lg, generator=None: d.greedy(lg), **kw)
    ids = [sch.submit(p, max_new_tokens=10) for p in prompts]
    if after:                                          # a victim leaves for the host in mid-run and comes back by itself
        sch.run(max_steps=after)
        assert sch._make_room(exclude=()) and len(sch.swapped) == 1
    sch.run(max_steps=500)
    assert [sch.sequences[i] for i in ids] == want and not sch.pending() and not sch.rejected
    assert len(d.pool.free_blocks) == blocks and d.pool.free_state_slots == 3


def test_swapped_out_sequences_continue_where_they_were():
    name = "mixed"
    c = cases.CONFIGS[name]
    d = decoder(name, torch.float32)
    toks = cases.tokens(c, N, 1)
    want = expected(name, toks)[0]
    d.prefill(0, toks[:50])
    d.prefill(1, toks[:33])
    d.pool.swap_out(0)
    d.prefill(2, cases.tokens(c, 60, 8))               # takes the blocks and the slot that came free
    d.pool.free(1)
    assert d.pool.swap_in(0)
    got = torch.cat([d.step([0], [toks[50:70]], [list(range(20))])] + [d.decode([0], [t]) for t in toks[70:80]])
    logits_close(got, want[50:80], torch.float32)


def test_command_line_generation_and_trace_replay(tmp_path, greedy_case):
    name, prompts, want = greedy_case
    c = cases.CONFIGS[name]
    folder = cases.write_model(tmp_path / "model", c, cases.tensors(c))
    args = [a for p in prompts for a in ("--prompt-ids", ",".join(map(str, p)))]
    r = subprocess.run([sys.executable, "-m", "vllmini_amd", "generate", "--model", folder, "--dtype", "float32", "--max-new-tokens", "10",
                        "--prefill-chunk", "9", *args], capture_output=True, text=True, cwd=REPO, timeout=100)
    assert r.returncode == 0, r.stderr[-2000:]
    assert [g["prompt"] + g["generated"] for g in map(json.loads, r.stdout.splitlines())] == want
    out = tmp_path / "out"
    out.mkdir()
    toks = cases.tokens(c, N, 1)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": toks[:40], "want": [0, 39]}, {"id": "b", "tokens": toks[:2], "want": []}], "end": []},
             {"step": 1, "entries": [{"id": "b", "tokens": toks[2:3], "want": []}], "end": ["a"]},
             {"step": 2, "entries": [{"id": "b", "tokens": toks[3:70], "want": [66]}, {"id": "c", "tokens": toks[:1], "want": [0]}], "end": ["b", "c"]}]
    r = subprocess.run([os.path.join(REPO, "bin", "trace_run"), "--model", folder, "--dtype", "float32", "--out", str(out), "--max-tokens", "256"],
                       input="\n".join(json.dumps(s) for s in steps) + "\n", capture_output=True, text=True, timeout=100)
    assert r.returncode == 0 and r.stdout.split("\n")[:3] == ["done 0", "done 1", "done 2"], r.stderr[-2000:]
    ref = expected(name, toks)[0]
    read = lambda n: torch.from_numpy(np.fromfile(out / n, "<f4").reshape(-1, c["vocab"]))      # noqa: E731
    logits_close(read("0.f32"), ref[[0, 39]], torch.float32)
    logits_close(read("2.f32"), ref[[69, 0]], torch.float32)
