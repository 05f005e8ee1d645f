"""The Fetelorn design on the CPU: the plain restatement on its defining properties, configuration, builder, layouts, bias tables, pool."""
from __future__ import annotations

import ctypes
import math

import pytest
import torch

from oracle import fetelorn as plain
from tests import fetelorn_cases as cases


# ---- the oracle's own mechanisms -------------------------------------------------------------------------------------------------
def _rnd(*shape, seed=0):
    return torch.randn(*shape, generator=torch.Generator().manual_seed(seed), dtype=torch.float64)


def test_plain_delta_rule_recalls_and_overwrites():
    """Without decay and with full steps, a unit key reads back what was written under it last, whatever lies under orthogonal ones."""
    q, _ = torch.linalg.qr(_rnd(6, 6))
    keys = q.t()[[0, 1, 2, 1]][:, None]                   # token 3 writes under token 1's key again
    v = _rnd(4, 1, 5, seed=1)
    one = torch.ones(4, 1, 6, dtype=torch.float64)
    o, S = plain.delta_rule(keys, keys, v, one, torch.ones(4, 1, dtype=torch.float64))
    assert torch.allclose(o, v)                           # the read-out sees the token's own write
    assert torch.allclose(S[0].T @ keys[1, 0], v[3, 0]) and torch.allclose(S[0].T @ keys[0, 0], v[0, 0])
    o1, S1 = plain.delta_rule(keys[:2], keys[:2], v[:2], one[:2] * 0.5, torch.full((2, 1), 0.3, dtype=torch.float64))
    o2, S2 = plain.delta_rule(keys[2:], keys[2:], v[2:], one[2:] * 0.5, torch.full((2, 1), 0.3, dtype=torch.float64), state=S1)
    o3, S3 = plain.delta_rule(keys, keys, v, one * 0.5, torch.full((4, 1), 0.3, dtype=torch.float64))
    assert torch.allclose(torch.cat([o1, o2]), o3) and torch.allclose(S2, S3)


def test_plain_retention_is_a_decaying_sum():
    q, k, v, d = _rnd(7, 2, 4), _rnd(7, 2, 4, seed=1), _rnd(7, 2, 3, seed=2), torch.tensor([0.5, 1.0], dtype=torch.float64)
    o, _ = plain.retain(q, k, v, d)
    for t in range(7):
        for h in range(2):
            want = sum(d[h] ** (t - j) * (q[t, h] @ k[j, h]) * v[j, h] for j in range(t + 1))
            assert torch.allclose(o[t, h], want)
    turn = lambda x, p: plain.rotate(x, p, 300.0, 6)      # noqa: E731
    a, b = _rnd(10), _rnd(10, seed=4)
    assert float(turn(a, 9) @ turn(b, 4)) == pytest.approx(float(turn(a, 105) @ turn(b, 100)))
    assert torch.equal(turn(a, 31)[6:], a[6:]) and torch.equal(turn(a, 0), a)


def test_plain_attention_stays_in_its_chunk_and_counts_the_sink_once():
    q, k, v = _rnd(4, 6), _rnd(12, 2, 6, seed=1), _rnd(12, 2, 3, seed=2)
    rel, sink = _rnd(6, 4, seed=3), _rnd(4, seed=4)
    at = lambda i, kk=k, vv=v, s=sink, r=rel: plain.chunk_attend(q, kk, vv, i, 5, 0.3, r, 9.0, s)      # noqa: E731
    other = v.clone()
    other[:5] += 100
    other[8:] -= 100
    assert torch.equal(at(7, vv=other), at(7)) and not torch.equal(at(4, vv=other), at(4))
    # a single key (the first of a chunk): its weight is what the sink leaves
    w = torch.sigmoid((k[5].repeat_interleave(2, 0) * q).sum(-1) * 0.3 + rel[0] - sink)
    assert torch.allclose(at(5), w[:, None] * v[5].repeat_interleave(2, 0))
    far = rel.clone()
    far[plain.distance_bucket(2, 6, 9.0)] += 1e3           # two tokens back drowns everything else
    assert torch.allclose(at(8, r=far), v[6].repeat_interleave(2, 0))


@pytest.mark.parametrize("name", sorted(cases.CONFIGS))
def test_plain_forward_is_causal_and_its_faults_show(name):
    c = cases.CONFIGS[name]
    w, toks = cases.tensors(c), cases.tokens(c, 20)
    full, streams = plain.forward(c, w, toks)
    assert streams.shape[0] == len(c["layers"]) and torch.isfinite(full).all()
    part, _ = plain.forward(c, w, toks[:13])
    assert torch.allclose(part, full[:13], atol=1e-9)
    other, _ = plain.forward(c, w, [toks[0] ^ 1] + toks[1:])
    assert float((other[-1] - full[-1]).abs().max()) > 1e-4          # the first token still matters at the end
    for planted in ("rel", "sink", "left.g", "conv", "A_log", "dt_bias", "right.norm", "left.out", "norm1", "mlp.gate", "mix.g", "final.norm"):
        hit = [k for k in w if k.endswith(planted)]
        if hit:
            bad = dict(w)
            bad[hit[0]] = bad[hit[0]] * 0.5
            assert float((plain.forward(c, bad, toks)[0] - full).abs().max()) > 1e-3, planted


# ---- configuration and builder -----------------------------------------------------------------------------------------------------
def _config(c):
    from vllmini_amd.fetelorn import FetelornConfig

    return FetelornConfig.from_json(c)


@pytest.mark.parametrize("name", sorted(cases.CONFIGS))
def test_config_knows_every_tensor(name):
    have, want = _config(cases.CONFIGS[name]).tensor_shapes(), cases.shapes(cases.CONFIGS[name])
    assert set(have) == set(want)
    for k in want:
        assert len(have[k]) == len(want[k]) and all(a is None or a == b for a, b in zip(have[k], want[k])), k


def test_config_and_layers_refuse_what_the_design_does_not_have():
    from vllmini_amd.fetelorn import build_model
    from vllmini_amd.hybrid_ops import state_dim

    ret = cases.retention(2, 8, 8, 8, (0.5, 0.5))
    with pytest.raises(ValueError, match="unknown mixer"):
        _config(cases.config([{"type": "sliding", "mixer": {}, "mlp": None}]))
    with pytest.raises(ValueError, match="feed-forward"):
        _config(cases.config([{**ret, "mlp": {"kind": "experts", "ff": 8}}]))
    with pytest.raises(ValueError, match="key heads"):
        _config(cases.config([cases.parallel(cases.attention(3, 2, 8, 8, 1.0, 8, 9), cases.delta(1, 1, 8, 8, 1))]))
    for bad, text in ((cases.retention(2, 8, 8, 7, (0.5, 0.5)), "rotated"), (cases.retention(2, 8, 8, 8, (0.5,)), "decay"),
                      (cases.retention(2, 8, 8, 8, (0.5, 1.5)), "decay")):
        c = cases.config([bad])
        with pytest.raises(ValueError, match=text):
            build_model(_config(c), cases.tensors(c), torch.float32, "cpu")
    assert [state_dim(n) for n in (1, 32, 33, 100, 130, 200, 257)] == [32, 32, 64, 128, 192, 256, 512]
    with pytest.raises(ValueError, match="512"):
        state_dim(513)


def test_builder_refuses_missing_and_misshapen_tensors():
    from vllmini_amd.fetelorn import build_model

    c = cases.CONFIGS["chunks"]
    w, cfg = cases.tensors(c), _config(c)
    with pytest.raises(KeyError, match="l1.mix.left.sink"):
        build_model(cfg, {k: v for k, v in w.items() if k != "l1.mix.left.sink"}, torch.float32, "cpu")
    with pytest.raises(ValueError, match="l0.mix.right.b "):
        build_model(cfg, {**w, "l0.mix.right.b": w["l0.mix.right.b"][:-1]}, torch.float32, "cpu")
    with pytest.raises(ValueError, match="ranks"):
        build_model(cfg, {**w, "l0.mix.right.a1": w["l0.mix.right.a1"][:-1]}, torch.float32, "cpu")


def test_registry_serves_the_design_in_two_element_types(tmp_path):
    from vllmini_amd import registry

    c = cases.CONFIGS["mixed"]
    folder = cases.write_model(tmp_path / "m", c, cases.tensors(c))
    assert "Fetelorn" in registry.architectures() and registry.architecture_of(registry.read_config(folder)) == "Fetelorn"
    with pytest.raises(registry.UnsupportedDtype, match="Fetelorn"):
        registry.load_decoder(folder, dtype="float16", max_tokens=64, max_seqs=1, device="cpu")


def test_joined_projections_keep_the_products():
    """Tiles, padding, joining and interleaving only rearrange: what a block's two products read back as is the checkpoint's."""
    from vllmini_amd.fetelorn import build_model

    c = cases.CONFIGS["mixed"]
    w = {k: v.float() for k, v in cases.tensors(c).items()}
    runs = build_model(_config(c), cases.tensors(c), torch.float32, "cpu").runs
    E, blk = c["width"], runs[0].mixer
    d, z = blk.w_in.dense, blk.mixer.sizes
    H, dim, vd, ff = 3, 20, 24, 72
    for j, (n, true, padded) in enumerate((("q", dim, z["dim"]), ("k", dim, z["dim"]), ("v", vd, z["vdim"]), ("g", vd, z["vdim"]))):
        at = H * (min(j, 2) * z["dim"] + max(j - 2, 0) * z["vdim"])
        rows = d[at:at + H * padded, :E].view(H, padded, E)
        assert torch.equal(rows[:, :true], w[f"l0.mix.{n}"].view(H, true, E)) and not rows[:, true:].any()
    glu = d[blk.n_in:]
    assert torch.equal(glu[0:2 * ff:2, :E], w["l0.mlp.gate"]) and torch.equal(glu[1:2 * ff:2, :E], w["l0.mlp.up"]) and not d[:, E:].any()
    out = blk.w_out[0].dense
    assert torch.equal(out[:E, :H * z["vdim"]].reshape(E, H, -1)[:, :, :vd], w["l0.mix.o"].view(E, H, vd))
    assert torch.equal(out[:E, blk.n_mix:blk.n_mix + ff], w["l0.mlp.down"])
    two = runs[1].mixer                                   # two arms and the feed-forward: a product each
    assert [t.K for t in two.w_out] == [6 * 32, 4 * 64, 64] and two.n_mix == 6 * 32 + 4 * 64
    right = two.mixer.arms[1]
    assert torch.equal(right.conv_w[:, :2 * 32].t().reshape(2, 32, 3)[:, :24], w["l1.mix.right.q.conv"].view(2, 24, 3))
    assert right.sizes["kv_heads"] == 2 and right.channels == 2 * 2 * 32 + 4 * 64
    assert torch.equal(runs[2].mixer.w_out[0].dense[:E, :2 * 96].reshape(E, 2, 96)[:, :, :72], w["l2.mix.o"].view(E, 2, 72))


@pytest.mark.parametrize("buckets,far,n", [(16, 250.0, 700), (9, 64.0, 100), (2, 1.5, 40), (32, 1000.0, 5000), (6, 27.0, 60), (16, 128.0, 300)])
def test_bias_table_of_distances(buckets, far, n):
    from vllmini_amd.hybrid_layers import distance_buckets

    got = distance_buckets(n, buckets, far).tolist()
    half = buckets // 2
    for d, b in enumerate(got):
        x = None if d < half else math.log(d / half) / math.log(far / half) * (buckets - half)
        if x is not None and abs(x - round(x)) < 1e-7:      # on an edge: the row above it
            assert b == min(buckets - 1, half + round(x))
        else:
            assert b == plain.distance_bucket(d, buckets, far)
    assert got == sorted(got) and got[0] == 0 and (got[-1] == buckets - 1 or n <= far)
    with pytest.raises(ValueError, match="distance bias"):
        distance_buckets(9, 16, 8.0)
    assert distance_buckets(8, 16, 8.0).tolist() == list(range(8)) and distance_buckets(4, 1, 9.0).tolist() == [0] * 4


def test_pool_holds_pages_and_states_of_one_layer():
    from vllmini_amd.fetelorn import build_model

    c = cases.CONFIGS["mixed"]
    m = build_model(_config(c), cases.tensors(c), torch.bfloat16, "cpu")
    pool = m.make_pool(256, 3, 16)
    assert pool.page_rows == [2 * (32 + 32), 5 * (32 + 32)]
    assert [tuple(t.shape) for t in pool.state] == [(3, 3, 32, 32), (3, 4, 32, 64), (3, 2, 2, 2 * 2 * 32 + 4 * 64), (3, 2, 64, 96),
                                                    (3, 3, 32, 32), (3, 2, 3, 2 * 32 + 3 * 32)]
    assert [t.dtype for t in pool.state] == [torch.float32, torch.float32, torch.bfloat16, torch.float32, torch.float32, torch.bfloat16]


def test_entries_refuse_bad_arguments_without_touching_a_device():
    from vllmini_amd import hybrid_ops as h

    lib, step = h.load(), ctypes.byref(h.StepArgs())
    assert lib.vmi_hy_state(ctypes.byref(h.StateArgs()), step, None) == 1
    assert lib.vmi_hy_attention(ctypes.byref(h.GqaArgs()), step, None) == 1
    assert lib.vmi_hy_kv_prep(ctypes.byref(h.KvPrepArgs()), step, None) == 1
    assert lib.vmi_hy_rotations(None, 4, None, step, 0, None) == 1
    assert lib.vmi_hy_merge(None, None, 0, None, 0, None, 0, None, None, 1, 1, 4, 0.0, 0.5, 0, 0, None) == 1
    assert [h.attention_row_tiles(128, 128, n, torch.bfloat16) for n in (1, 2, 4)] == [1, 4, 4]
    assert h.attention_row_tiles(128, 128, 4, torch.float32) == 1 and h.attention_row_tiles(320, 64, 4, torch.bfloat16) == 1
    assert h.state_fuses(128, 128) and not h.state_fuses(128, 160) and h.state_fuses(256, 64) and not h.state_fuses(512, 64)
