"""The Voduvik design on the GPU, mechanism by mechanism and end to end, against the plain restatement (oracle/voduvik.py, float64).

float32 runs of the kernels are compared tightly: there a wrong key, position, page or state shows at once.  bfloat16 runs are
compared within what rounding explains, and with inputs that make one key stand out where an average would hide it."""
from __future__ import annotations

import json
import os
import subprocess
import sys

import numpy as np
import pytest
import torch

from oracle import voduvik as plain
from tests import voduvik_cases as cases

pytestmark = pytest.mark.gpu
REPO = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
BOTH = [torch.float32, torch.bfloat16]


def dev():
    return torch.device("cuda:0")


def i32(v):
    return torch.as_tensor(np.asarray(v), dtype=torch.int32).to(dev())


def close(got, want, dtype, tol32=2e-5, tol16=2e-2):
    got, want = got.double().cpu(), want.double().cpu()
    scale = float(want.abs().max()) + 1e-6
    err = float((got - want).abs().max()) / scale
    assert err <= (tol32 if dtype == torch.float32 else tol16), f"max|d| / max = {err:.3e}"


def layout(counts, ctx, tables, page, slots=None, flips=None, pos_slots=True):
    """A StepLayout for portions of `counts` tokens behind `ctx` ones."""
    from vllmini_amd import hybrid_ops as ops

    counts, ctx = np.asarray(counts), np.asarray(ctx)
    starts = np.cumsum(counts) - counts
    seq = np.repeat(np.arange(len(counts)), counts)
    pos = np.arange(counts.sum()) - np.repeat(starts, counts) + np.repeat(ctx, counts)
    tables = np.asarray(tables)
    slot = tables[seq, pos // page] * page + pos % page if pos_slots else np.full(len(seq), -1)
    f = dict(tok_seq=i32(seq), tok_pos=i32(pos), tok_slot=i32(slot), q_start=i32(starts), q_len=i32(counts), ctx=i32(ctx),
             state_slot=i32(range(len(counts)) if slots is None else slots), flip=i32([0] * len(counts) if flips is None else flips),
             table=i32(tables))
    if (counts > 1).any():
        per = -(-counts // ops.CHUNK_ROWS)
        f["chunk_start"] = i32(np.cumsum(per) - per)
        f["chunks"] = i32([(b, 16 * c) for b in range(len(counts)) for c in range(per[b])])
    spans = bool((starts // ops.ROW_TILE != (starts + counts - 1) // ops.ROW_TILE).any())
    return ops.StepLayout(f, int(counts.sum()), len(counts), page, bool((counts == 1).all()), spans, int(counts.max()),
                          int((ctx + counts).max()))


# ---- linear layers ---------------------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("dtype", BOTH)
@pytest.mark.parametrize("M", [1, 5, 17, 40, 130])
@pytest.mark.parametrize("N,K", [(32, 32), (96, 288), (352, 800), (1056, 1312)])
def test_linear_kinds(dtype, M, N, K):
    from vllmini_amd import hybrid_ops as ops

    g = torch.Generator().manual_seed(M * N + K)
    rnd = lambda *s: torch.randn(*s, generator=g)      # noqa: E731
    x, w = rnd(M, K).to(dtype).to(dev()), (rnd(N, K) / K ** 0.5).to(torch.bfloat16).to(dev())
    t = ops.MatrixTiles(w, dtype)
    W = w.double()
    bias = rnd(N).to(dev())
    close(ops.linear(x, t, bias=bias), x.double() @ W.T + bias.double(), dtype)
    base = rnd(M, N).to(dev())
    close(ops.linear(x, t, residual=True, out=base.clone()), base.double() + x.double() @ W.T, dtype, tol16=1e-3)
    # normalised rows, with a mean far from zero and a ragged true length
    n = K - 13
    xf, nw = (rnd(M, K) * 3 + 40).to(dev()), torch.zeros(K, device=dev())
    xf[:, n:] = 0
    nw[:n] = 1 + 0.5 * rnd(n).to(dev())
    h = torch.zeros(M, K, dtype=torch.float64, device=dev())
    h[:, :n] = plain.layer_norm(xf[:, :n].double(), nw[:n].double(), 1e-5)
    close(ops.linear(xf, t, norm=(nw, n, 1e-5)), h @ W.T, dtype, tol32=1e-4)
    rows = torch.tensor([M - 1, 0, M // 2], dtype=torch.int32, device=dev())
    cols = N - 5
    close(ops.linear(xf, t, norm=(nw, n, 1e-5), rows=rows, float_out=(cols, 0.3)), (h @ W.T)[rows.long(), :cols] * 0.3, dtype, tol32=1e-4)
    y = h @ W.T
    gate, up = y[:, 0::2].clamp(max=0.8), y[:, 1::2].clamp(-0.8, 0.8)
    close(ops.linear(xf, t, norm=(nw, n, 1e-5), glu=ops.GatedUnit.clamped(0.8)), gate * torch.sigmoid(1.702 * gate) * (up + 1), dtype, tol32=1e-4, tol16=3e-2)
    if K % 64 == 0:
        a, b = rnd(M, K // 2).to(dev()), rnd(M, K // 2).to(dev())
        close(ops.linear(a, t, x2=b, float_out=(N, 1.0)), torch.cat([a, b], 1).double() @ W.T, dtype)


@pytest.mark.parametrize("dtype", BOTH)
@pytest.mark.parametrize("M", [3, 70])
def test_linear_groups_and_head_gate(dtype, M):
    from vllmini_amd import hybrid_ops as ops

    g = torch.Generator().manual_seed(M)
    G, N, K, gap = 5, 64, 96, 160
    x = torch.randn(M, G * gap, generator=g).to(dtype).to(dev())
    w = (torch.randn(G, N, K, generator=g) / 10).to(torch.bfloat16).to(dev())
    gate = torch.randn(M, 32, generator=g).to(dtype).to(dev())
    out = torch.zeros(M, G * 80, dtype=dtype, device=dev())
    ops.linear(x, ops.MatrixTiles(w, dtype), x_gstride=gap, y_gstride=80, gate=gate[:, 3:], out=out)
    for i in range(G):
        want = x[:, i * gap:i * gap + K].double() @ w[i].double().T * torch.sigmoid(gate[:, 3 + i].double())[:, None]
        close(out[:, i * 80:i * 80 + N], want, dtype)
        assert not out[:, i * 80 + N:(i + 1) * 80].any()


@pytest.mark.parametrize("dtype", BOTH)
@pytest.mark.parametrize("n", [50, 96, 1500, 9001])
def test_elementwise_ends(dtype, n):
    from vllmini_amd import hybrid_ops as ops

    g = torch.Generator().manual_seed(n)
    ld = ops.pad32(n)
    x = torch.zeros(7, ld, device=dev())
    x[:, :n] = (torch.randn(7, n, generator=g) * 2 - 30).to(dev())
    add, w = torch.zeros(7, ld, dtype=dtype, device=dev()), torch.zeros(ld, device=dev())
    add[:, :n] = torch.randn(7, n, generator=g).to(dtype).to(dev())
    w[:n] = torch.randn(n, generator=g).to(dev())
    want = x.double() + add.double()
    h = ops.add_norm(x, add, (w, n, 1e-6), dtype)
    close(x, want, torch.float32)
    close(h[:, :n], plain.layer_norm(want[:, :n], w[:n].double(), 1e-6), dtype, tol32=1e-4)
    assert not h[:, n:].any()
    v = (torch.randn(7, 2 * ld, generator=g) * 2).to(dtype).to(dev())
    gate, up = v[:, 0::2].double().clamp(max=1.25), v[:, 1::2].double().clamp(-1.25, 1.25)
    close(ops.glu(v, ops.GatedUnit.clamped(1.25)), gate * torch.sigmoid(1.702 * gate) * (up + 1), dtype)
    table = torch.zeros(40, ld, dtype=torch.bfloat16, device=dev())
    table[:, :n] = torch.randn(40, n, generator=g).to(dev())
    ids = torch.tensor([0, 39, 7], device=dev())
    assert torch.equal(ops.embed(ids, table, n, 2.5), table[ids].float() * 2.5)
    lg = torch.randn(6, n, generator=g).to(dev())
    lg[2, 5] = lg[2, 31] = 9.0
    assert ops.argmax(lg).tolist() == lg.argmax(-1).tolist() and ops.argmax(lg)[2] == 5


# ---- the recurrent block ---------------------------------------------------------------------------------------------------------
def _rglru_weights(width, blocks, taps, seed):
    c = cases.config([cases.rglru(width, blocks, taps)], width=width)
    return cases.tensors(c, seed)


class _Rglru:
    """The kernel's operands for a width / block count, and the plain result for a whole sequence."""

    def __init__(self, width, blocks, taps, dtype, slots, seed=0):
        from vllmini_amd.hybrid_layers import Norm, RGLRU

        w = {k: v.to(dev()) for k, v in _rglru_weights(width, blocks, taps, seed).items()}
        self.w = {k[len("l0.mix."):]: v for k, v in w.items() if k.startswith("l0.mix.")}
        n = self.w
        self.layer = RGLRU(width=width, size=width, blocks=blocks, taps=taps, norm=Norm(w["l0.norm1"], (width + 31) // 32 * 32, 1e-5),
                           y=n["y"], y_b=n["y.b"], x=n["x"], x_b=n["x.b"], conv=n["conv"], conv_b=n["conv.b"], ra=n["ra"],
                           ra_b=n["ra.b"], ri=n["ri"], ri_b=n["ri.b"], lam=n["lam"], o=n["o"], dtype=dtype)
        self.width, self.blocks, self.dtype = width, blocks, dtype
        bw, bp = width // blocks, self.layer.width // blocks
        self.idx = (torch.arange(blocks)[:, None] * bp + torch.arange(bw)[None]).reshape(-1).to(dev())
        (s, _), (t, _) = self.layer.state_shapes()
        self.state = torch.full((slots, *s), 7.0, device=dev())              # what former owners left must not matter
        self.tail = torch.full((slots, *t), 5.0, dtype=dtype, device=dev())

    def inputs(self, T, seed):
        g = torch.Generator().manual_seed(seed)
        y, x = (torch.randn(T, self.width, generator=g).to(self.dtype).to(dev()) for _ in range(2))
        yx = torch.zeros(T, 2 * self.layer.width, dtype=self.dtype, device=dev())
        yx[:, self.idx], yx[:, self.layer.width + self.idx] = y, x
        return y, x, yx

    def plain(self, y, x):
        n = {k: v.double() for k, v in self.w.items()}
        u = plain.causal_conv(x.double(), n["conv"], n["conv.b"])
        if self.dtype == torch.bfloat16:
            u = u.to(torch.bfloat16).double()
        S, _ = plain.rglru_scan(u, plain.rglru_gate(u, n["ra"], n["ra.b"]), plain.rglru_gate(u, n["ri"], n["ri.b"]), n["lam"])
        return S * plain.gelu_tanh(y.double())

    def run(self, yx, step):
        from vllmini_amd import hybrid_ops as ops

        L = self.layer
        return ops.rglru(yx, step, conv_w=L.conv_w, conv_b=L.conv_b, gates=L.gates, gate_b=L.gate_b, decay=L.decay, blocks=L.blocks,
                         state=self.state, tail=self.tail)[:, self.idx]


@pytest.mark.parametrize("dtype", BOTH)
@pytest.mark.parametrize("width,blocks,taps", [(96, 3, 4), (40, 2, 1), (150, 1, 2), (600, 2, 7), (66, 11, 3)])
def test_recurrence_over_portions_of_every_size(dtype, width, blocks, taps):
    """Three sequences cut differently — whole, portions around the 64-row tile, two and three tokens, single tokens — in shared
    steps, the state in slots whose former contents are garbage."""
    T = 210
    k = _Rglru(width, blocks, taps, dtype, slots=5)
    seqs = [k.inputs(T, 10 + i) for i in range(3)]
    cuts = [[210], [63, 2, 64, 3, 1, 1, 65, 2, 9], [1] * 9 + [2, 3, 70, 1, 2, 123]]
    slots, at, flips = [4, 0, 2], [0] * 3, [0] * 3
    out = [[] for _ in range(3)]
    while any(at[i] < T for i in range(3)):
        live = [i for i in range(3) if at[i] < T]
        n = [cuts[i].pop(0) for i in live]
        yx = torch.cat([seqs[i][2][at[i]:at[i] + c] for i, c in zip(live, n)])
        step = layout(n, [at[i] for i in live], [[0]] * len(live), 64, [slots[i] for i in live], [flips[i] for i in live], pos_slots=False)
        got = k.run(yx, step)
        for i, c, g in zip(live, n, got.split(n)):
            out[i].append(g)
            at[i] += c
            flips[i] ^= 1
    for i in range(3):
        close(torch.cat(out[i]), k.plain(*seqs[i][:2]), dtype, tol32=3e-5, tol16=1.5e-2)


@pytest.mark.parametrize("dtype", BOTH)
def test_recurrence_decodes_like_it_prefills_and_skips_padding_rows(dtype):
    from vllmini_amd import hybrid_ops as ops

    k = _Rglru(96, 2, 4, dtype, slots=20)
    T, B = 20, 19
    seqs = [k.inputs(T, 50 + i) for i in range(B)]
    want = [k.plain(*s[:2]) for s in seqs]
    untouched = k.state[B].clone()
    for t in range(T):
        step = layout([1] * B, [t] * B, [[0]] * B, 64, flips=[t & 1] * B, pos_slots=False)
        f = dict(step.fields)
        f["tok_seq"] = torch.cat([f["tok_seq"], i32([-1, -1])])      # two padding rows, as a padded decode batch has
        f["tok_pos"], f["tok_slot"] = torch.cat([f["tok_pos"], i32([0, 0])]), torch.cat([f["tok_slot"], i32([-1, -1])])
        pad = ops.StepLayout(f, B + 2, B, 64, True, False, 1, t + 1)
        yx = torch.cat([s[2][t:t + 1] for s in seqs] + [torch.full((2, 2 * k.layer.width), float("nan"), dtype=dtype, device=dev())])
        got = k.run(yx, pad)
        assert not got[B:].any()
        for i in range(B):
            close(got[i], want[i][t], dtype, tol32=1e-4, tol16=3e-2)
    assert torch.equal(k.state[B], untouched)


def test_recurrence_keeps_a_long_memory_in_fp32():
    """Decays near one: after a thousand tokens without input the first token's trace is still there, to fp32 accuracy."""
    k = _Rglru(64, 2, 1, torch.bfloat16, slots=1)
    k.layer.decay.fill_(-1e-4)
    T = 1000
    yx = torch.zeros(T, 2 * k.layer.width, dtype=torch.bfloat16, device=dev())
    yx[:, k.idx] = 1.0
    yx[0, k.layer.width + k.idx] = 4.0
    k.layer.conv_b.zero_()
    k.layer.conv_w.fill_(1.0)
    k.layer.gate_b.zero_()
    k.layer.gates.zero_()
    got = k.run(yx, layout([T], [0], [[0]], 64, pos_slots=False)).double().cpu()
    a = np.exp(-1e-4 * 0.5)
    want = 4.0 * 0.5 * np.sqrt(1 - a * a) * a ** np.arange(T) * float(plain.gelu_tanh(torch.tensor(1.0, dtype=torch.float64)))
    assert np.abs(got.numpy() / want[:, None] - 1).max() < 5e-3          # (one bfloat16 rounding of the output)
    S = float(k.state[0, 0])
    assert S == pytest.approx(2.0 * np.sqrt(1 - a * a) * a ** (T - 1), rel=2e-5)


# ---- latent attention --------------------------------------------------------------------------------------------------------------
def _attend(dtype, H, rank, rot, counts, ctx, page, row_tiles=None, splits=1, spike=None, seed=0):
    from vllmini_amd import hybrid_ops as ops

    D, B = rank + rot, len(counts)
    g = torch.Generator().manual_seed(seed)
    total = [c + n for c, n in zip(ctx, counts)]
    per = [-(-t // page) for t in total]
    pages = torch.randperm(sum(per) + 3, generator=g).numpy()
    cache = torch.randn(len(pages), page, D, generator=g).to(dtype).to(dev())
    tables = np.zeros((B, max(per)), dtype=np.int64)
    at = 0
    for b in range(B):
        tables[b, :per[b]] = pages[at:at + per[b]]
        at += per[b]
    q = torch.randn(sum(counts), H, D, generator=g).to(dtype).to(dev())
    scale = 1.7 * D ** -0.5
    flat = cache.view(-1, D)
    row = lambda b, p: int(tables[b, p // page]) * page + p % page      # noqa: E731
    if spike is not None:      # query `t` of entry b meets a key of its own direction at position p: that score stands far out
        for b, t, p in spike:
            u = torch.randn(D, generator=g)
            u = u / u.norm()
            q[sum(counts[:b]) + t] = (u * (14 / scale) ** 0.5).to(dtype).to(dev())
            flat[row(b, p)] = (u * (14 / scale) ** 0.5).to(dtype).to(dev())
    step = layout(counts, ctx, tables, page)
    rt = ops.latent_row_tiles(D, row_tiles or 4, dtype)
    tiles = [(b, r) for b in range(B) for r in range(0, counts[b] * H, 16 * rt)]
    tiles.insert(1, (-1, -1))
    out = ops.latent_attention(q.view(-1, H * D), cache, step, i32(tiles), heads=H, rank=rank, rot=rot, scale=scale, row_tiles=rt,
                               splits=splits).view(-1, H, rank)
    want, at = [], 0
    for b in range(B):
        keys = flat[[row(b, p) for p in range(total[b])]].double()
        for t in range(counts[b]):
            s = q[at].double() @ keys[: ctx[b] + t + 1].T * scale
            want.append(torch.softmax(s, -1) @ keys[: ctx[b] + t + 1, :rank])
            at += 1
    return out, torch.stack(want)


@pytest.mark.parametrize("dtype", BOTH)
@pytest.mark.parametrize("H,rank,rot,page", [(1, 32, 32, 16), (3, 64, 32, 64), (7, 128, 32, 64), (20, 256, 64, 32), (16, 512, 64, 64),
                                             (5, 608, 32, 64), (40, 160, 96, 8)])
def test_latent_attention_over_pages(dtype, H, rank, rot, page):
    for counts, ctx in (([1], [0]), ([1, 1, 1], [63, 64, 200]), ([70, 1, 2], [0, 130, 62]), ([33], [95])):
        for rt in (1, 2, 4) if dtype == torch.bfloat16 else (1,):
            for sp in (1, 2, 5):
                got, want = _attend(dtype, H, rank, rot, counts, ctx, page, rt, sp)
                close(got, want, dtype, tol32=2e-5, tol16=1.5e-2)


@pytest.mark.parametrize("dtype", BOTH)
def test_latent_attention_sees_the_far_key_and_never_the_next_one(dtype):
    """One score stands out: at the very first token, at page borders, at the query's own position — and one past it, where it must
    not be seen."""
    n, ctx = 5, 700
    for p in (0, 1, 63, 64, 65, 127, 128, 447, 639, 640, ctx + 1, ctx + 2):
        got, want = _attend(dtype, 4, 64, 32, [n], [ctx], 64, splits=4, spike=[(0, 2, p)], seed=p)
        close(got, want, dtype)
        assert float(want[2].abs().max()) > 0.5
    got, want = _attend(dtype, 4, 64, 32, [n], [ctx], 64, splits=4, spike=[(0, 2, ctx + 3)], seed=1)      # the next token's key
    close(got, want, dtype)


@pytest.mark.parametrize("dtype", BOTH)
def test_latent_prep_normalises_rotates_and_writes_the_cache(dtype):
    from vllmini_amd import hybrid_ops as ops

    heads, dim, rot, rank, rot_n, rank_n, rot_true = 3, 32, 32, 64, 10, 50, 20
    g = torch.Generator().manual_seed(4)
    counts, ctx, page = [3, 1], [4000, 77], 16
    T = sum(counts)
    tables = np.arange(2 * 251).reshape(2, 251)[:, ::-1].copy()
    step = layout(counts, ctx, tables, page)
    ldp = heads * (dim + rot) + rank + rot + 32
    proj = torch.zeros(T, ldp)
    for h in range(heads + 1):
        at = h * (dim + rot) + dim if h < heads else heads * (dim + rot) + rank
        proj[:, at:at + rot_true] = torch.randn(T, rot_true, generator=g)
    proj[:, heads * (dim + rot):heads * (dim + rot) + rank_n] = 5 * torch.randn(T, rank_n, generator=g)
    proj = proj.to(dtype).to(dev())
    q = torch.full((T, heads * (rank + rot)), 3.0, dtype=dtype, device=dev())
    cache = torch.full((502, page, rank + rot), 9.0, dtype=dtype, device=dev())
    w = torch.zeros(rank, device=dev())
    w[:rank_n] = 1 + 0.3 * torch.randn(rank_n, generator=g).to(dev())
    freq = (500.0 ** (-2.0 * torch.arange(rot_n // 2, dtype=torch.float64) / rot_n)).to(dev())
    ops.latent_prep(proj, q, cache, step, norm_w=w, freq=freq, heads=heads, dim=dim, rot=rot, rank=rank, rot_n=rot_n, rank_n=rank_n, eps=1e-5)
    flat, P = cache.view(-1, rank + rot), proj.double().cpu()
    used = []
    for t in range(T):
        b, pos = (0, 4000 + t) if t < 3 else (1, 77)
        r = int(tables[b, pos // page]) * page + pos % page
        used.append(r)
        lat = heads * (dim + rot)
        close(flat[r, :rank_n], plain.rms_norm(P[t, lat:lat + rank_n], w[:rank_n].double().cpu(), 1e-5), dtype, tol16=6e-3)
        assert not flat[r, rank_n:rank].any()
        close(flat[r, rank:], plain.rotate(P[t, lat + rank:lat + rank + rot], pos, 500.0, rot_n), dtype, tol16=6e-3)
        for h in range(heads):
            s = h * (dim + rot) + dim
            close(q[t, h * (rank + rot) + rank:(h + 1) * (rank + rot)], plain.rotate(P[t, s:s + rot], pos, 500.0, rot_n), dtype, tol16=6e-3)
            assert (q[t, h * (rank + rot):h * (rank + rot) + rank] == 3).all()
    rest = torch.ones(flat.shape[0], dtype=torch.bool, device=dev())
    rest[used] = False
    assert (flat[rest] == 9).all()


# ---- the whole decoder -------------------------------------------------------------------------------------------------------------
_PLAIN = {}


def expected(name, toks):
    """Plain logits of a configuration's sequence (cached: several tests ask for prefixes of the same ones)."""
    key = (name, tuple(toks))
    if key not in _PLAIN:
        c = cases.CONFIGS[name]
        _PLAIN[key] = plain.forward(c, cases.tensors(c), toks)
    return _PLAIN[key]


def decoder(name, dtype, max_tokens=640, max_seqs=4, page=16, **kw):
    from vllmini_amd.hybrid_decoder import HybridDecoder
    from vllmini_amd.voduvik import VoduvikConfig, build_model

    c = cases.CONFIGS[name]
    m = build_model(VoduvikConfig.from_json(c), cases.tensors(c), dtype, dev())
    d = HybridDecoder(m, m.make_pool(max_tokens, max_seqs, page), **kw)
    g = torch.Generator(device=dev()).manual_seed(3)
    for t in d.pool.row_pages + d.pool.state:          # stale contents must never matter
        t.copy_(torch.empty(t.shape, device=dev()).uniform_(-4, 4, generator=g))
    return d


def logits_close(got, want, dtype, tol32=2e-4, tol16=0.12):
    got, want = got.double().cpu(), want.double().cpu()
    d = got - want
    d = d - d.mean(-1, keepdim=True)
    err = float((d.pow(2).mean(-1).sqrt() / want.std()).max())
    assert err <= (tol32 if dtype == torch.float32 else tol16), f"rms error / spread = {err:.3e}"


@pytest.mark.parametrize("dtype", BOTH)
@pytest.mark.parametrize("name", sorted(cases.CONFIGS))
def test_whole_prompt_and_the_stream_after_every_run(name, dtype):
    toks = cases.tokens(cases.CONFIGS[name], 90, 1)
    want, streams = expected(name, toks)
    d = decoder(name, dtype)
    d.pool.open(0)
    d.tap = []
    got = d.step([0], [toks], [list(range(90))])
    logits_close(got, want, dtype)
    assert len(d.tap) == len(streams)
    for a, b in zip(d.tap, streams):
        close(a, b, dtype, tol32=1e-4, tol16=8e-2)


@pytest.mark.parametrize("name", sorted(cases.CONFIGS))
def test_many_tokens_take_the_dense_path_to_the_same_logits(name, monkeypatch):
    from vllmini_amd import hybrid_layers

    monkeypatch.setattr(hybrid_layers, "DENSE_MIN_TOKENS", 1)
    toks = cases.tokens(cases.CONFIGS[name], 90, 1)
    for dtype in BOTH:
        d = decoder(name, dtype)
        d.pool.open(0)
        logits_close(d.step([0], [toks], [list(range(90))]), expected(name, toks)[0], dtype)


@pytest.mark.parametrize("dtype", BOTH)
@pytest.mark.parametrize("name", sorted(cases.CONFIGS))
def test_portions_single_tokens_and_neighbours_do_not_change_the_logits(name, dtype):
    """Unequal requests cut in every way, pages and slots given back and used again, requests left out of steps."""
    c = cases.CONFIGS[name]
    lens = [90, 40, 3, 1, 66, 90]
    toks = [cases.tokens(c, 90, 1)[:n] for n in lens]       # prefixes of one sequence: one plain run checks all of them
    want = expected(name, cases.tokens(c, 90, 1))[0]
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
    name, n = "mixed", 330
    toks = cases.tokens(cases.CONFIGS[name], n, 9)
    want = expected(name, toks)[0]
    d = decoder(name, dtype, page=32)
    first = d.prefill(0, toks[:1])
    got = torch.cat([first[None]] + [d.decode([0], torch.tensor([t], device=dev())).clone() for t in toks[1:]])
    logits_close(got, want, dtype, tol32=5e-4)


@pytest.mark.parametrize("vendor", [False, True], ids=["streaming", "vendor"])
def test_graph_replay_equals_eager_steps(vendor, monkeypatch):
    """Both ways a layer's products may run, captured; eager steps run between the replays."""
    from vllmini_amd import hybrid_layers

    if vendor:
        monkeypatch.setattr(hybrid_layers, "DENSE_MIN_TOKENS", 1)
    name = "mixed"
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


def test_step_refuses_what_does_not_fit():
    d = decoder("no_loop", torch.float32, max_tokens=64, max_seqs=2)
    d.pool.open(0)
    with pytest.raises(ValueError, match="token id"):
        d.step([0], [[1, 130]])
    with pytest.raises(ValueError, match="wanted places"):
        d.step([0], [[1, 2]], [[2]])
    with pytest.raises(RuntimeError, match="free blocks|blocks per layer"):
        d.step([0], [[1] * 65])
    assert d.pool.seq_len(0) == 0 and d.step([0], [[1, 2]], [[]]) is None
    with pytest.raises(RuntimeError):
        d.prefill_batch([1], [[1] * 100])
    assert 1 not in d.pool.allocated_blocks and d.pool.free_state_slots == 1


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
    return name, prompts, [_plain_greedy(name, p, 12) for p in prompts]


@pytest.mark.parametrize("kw", [{}, {"use_graph": True}, {"prefill_chunk": 7}, {"prefill_chunk": 16, "use_graph": True}, {"preempt_after": 4}],
                         ids=["plain", "graph", "chunks", "chunks+graph", "preempted"])
def test_greedy_generation_through_the_scheduler(kw, greedy_case):
    from vllmini_amd.scheduler import BatchScheduler

    name, prompts, want = greedy_case
    kw, blocks = dict(kw), 12
    after = kw.pop("preempt_after", 0)
    d = decoder(name, torch.float32, max_tokens=16 * blocks, max_seqs=3)
    sch = BatchScheduler(d, max_length=46, eos_token_id=-1, max_batch=3, sampler=lambda lg, generator=None: d.greedy(lg), **kw)
    ids = [sch.submit(p, max_new_tokens=12) for p in prompts]
    if after:                                          # a victim leaves for the host in mid-run and comes back by itself
        sch.run(max_steps=after)
        assert sch._make_room(exclude=()) and len(sch.swapped) == 1
    sch.run(max_steps=500)
    assert [sch.sequences[i] for i in ids] == want and not sch.pending() and not sch.rejected
    assert sch.stats["resumes"] == (1 if after else 0)
    assert len(d.pool.free_blocks) == blocks and d.pool.free_state_slots == 3


def test_swapped_out_sequences_continue_where_they_were():
    name = "mixed"
    c = cases.CONFIGS[name]
    d = decoder(name, torch.float32)
    toks = cases.tokens(c, 90, 1)
    want = expected(name, toks)[0]
    d.prefill(0, toks[:50])
    d.prefill(1, toks[:33])
    d.pool.swap_out(0)
    d.prefill(2, cases.tokens(c, 60, 8))               # takes the blocks and the slot that came free
    d.pool.free(1)
    assert d.pool.swap_in(0)
    got = torch.cat([d.step([0], [toks[50:70]], [list(range(20))])] + [d.decode([0], [t]) for t in toks[70:80]])
    logits_close(got, want[50:80], torch.float32)


def test_sampling_from_float_logits_stays_inside_the_top_k():
    from vllmini_amd.scheduler import sample_top_k

    lg = torch.randn(6, 203, device=dev())
    g = torch.Generator(device=dev()).manual_seed(0)
    top = lg.topk(4, -1).indices
    for _ in range(20):
        t = sample_top_k(lg, 4, 0.7, generator=g)
        assert ((top == t[:, None]).any(-1)).all()


def test_command_line_generation_and_trace_replay(tmp_path, greedy_case):
    name, prompts, want = greedy_case
    c = cases.CONFIGS[name]
    folder = cases.write_model(tmp_path / "model", c, cases.tensors(c))
    args = [a for p in prompts for a in ("--prompt-ids", ",".join(map(str, p)))]
    r = subprocess.run([sys.executable, "-m", "vllmini_amd", "generate", "--model", folder, "--dtype", "float32", "--max-new-tokens", "12",
                        "--prefill-chunk", "9", *args], capture_output=True, text=True, cwd=REPO, timeout=100)
    assert r.returncode == 0, r.stderr[-2000:]
    got = [json.loads(x) for x in r.stdout.splitlines()]
    assert [g["prompt"] + g["generated"] for g in got] == want
    out = tmp_path / "out"
    out.mkdir()
    toks = cases.tokens(c, 90, 1)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": toks[:40], "want": [0, 39]}, {"id": "b", "tokens": toks[:2], "want": []}], "end": []},
             {"step": 1, "entries": [{"id": "b", "tokens": toks[2:3], "want": []}], "end": ["a"]},
             {"step": 2, "entries": [{"id": "b", "tokens": toks[3:70], "want": [66]}, {"id": "c", "tokens": toks[:1], "want": [0]}], "end": ["b", "c"]}]
    r = subprocess.run([os.path.join(REPO, "bin", "trace_run"), "--model", folder, "--dtype", "float32", "--out", str(out), "--max-tokens", "256"],
                       input="\n".join(json.dumps(s) for s in steps) + "\n", capture_output=True, text=True, timeout=100)
    assert r.returncode == 0 and r.stdout.split("\n")[:3] == ["done 0", "done 1", "done 2"], r.stderr[-2000:]
    assert not (out / "1.f32").exists()
    ref = expected(name, toks)[0]
    read = lambda n: torch.from_numpy(np.fromfile(out / n, "<f4").reshape(-1, c["vocab"]))      # noqa: E731
    logits_close(read("0.f32"), ref[[0, 39]], torch.float32)
    logits_close(read("2.f32"), ref[[69, 0]], torch.float32)
