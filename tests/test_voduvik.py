"""The Voduvik design on the CPU: the plain restatement against itself, configuration and checkpoint reading, the pool's portions
and state slots, portions of prompts in the scheduler, and the C-ABI of libvmi_hybrid.so."""
from __future__ import annotations

import ctypes
import os
import re
import subprocess

import numpy as np
import pytest
import torch

from oracle import voduvik as plain
from tests import voduvik_cases as cases

REPO = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))


# ---- the oracle's own mechanisms, checked on their defining properties ---------------------------------------------------------
def test_plain_rotation_turns_pairs_and_keeps_relative_angles():
    g = torch.Generator().manual_seed(0)
    q, k = (torch.randn(24, generator=g, dtype=torch.float64) for _ in range(2))
    dot = lambda p, j: float(plain.rotate(q, p, 700.0, 16) @ plain.rotate(k, j, 700.0, 16))      # noqa: E731
    assert dot(9, 4) == pytest.approx(dot(105, 100)) and dot(9, 4) != pytest.approx(dot(9, 5))
    assert torch.equal(plain.rotate(q, 31, 700.0, 16)[16:], q[16:]) and torch.equal(plain.rotate(q, 0, 700.0, 16), q)


def test_plain_convolution_and_recurrence_against_closed_forms():
    g = torch.Generator().manual_seed(1)
    x, w, b = torch.randn(9, 3, generator=g), torch.randn(3, 4, generator=g), torch.randn(3, generator=g)
    ref = torch.nn.functional.conv1d(torch.nn.functional.pad(x.t()[None], (3, 0)), w[:, None], b, groups=3)[0].t()
    assert torch.allclose(plain.causal_conv(x, w, b), ref, atol=1e-5)
    u, r, i = torch.ones(5, 2, dtype=torch.float64), torch.full((5, 2), 0.5, dtype=torch.float64), torch.ones(5, 2, dtype=torch.float64)
    lam = torch.tensor([-4.0, 1.0], dtype=torch.float64)
    a = torch.exp(-4 * torch.nn.functional.softplus(lam))
    S, last = plain.rglru_scan(u, r, i, lam)
    want = torch.stack([torch.sqrt(1 - a * a) * (1 - a ** n) / (1 - a) for n in range(1, 6)])
    assert torch.allclose(S, want) and torch.equal(last, S[-1])
    half, mid = plain.rglru_scan(u[:2], r[:2], i[:2], lam)
    rest, _ = plain.rglru_scan(u[2:], r[2:], i[2:], lam, state=mid)
    assert torch.allclose(torch.cat([half, rest]), S)


@pytest.mark.parametrize("name", sorted(cases.CONFIGS))
def test_plain_forward_is_causal_and_its_faults_show(name):
    c = cases.CONFIGS[name]
    w, toks = cases.tensors(c), cases.tokens(c, 24)
    full, streams = plain.forward(c, w, toks)
    assert streams.shape[0] == len(plain.layer_runs(c)) and torch.isfinite(full).all()
    part, _ = plain.forward(c, w, toks[:15])
    assert torch.allclose(part, full[:15], atol=1e-9)
    other, _ = plain.forward(c, w, [toks[0] ^ 1] + toks[1:])       # the first token still matters at the end: a lost state or key
    assert float((other[-1] - full[-1]).abs().max()) > 1e-3        # would show
    for planted in ("lam", "dkv.norm", "conv.b", "norm1", "mlp.gate", "loop.in"):       # so would any weight that is left out
        hit = [k for k in w if k.endswith(planted)]
        if hit:
            bad = dict(w)
            bad[hit[0]] = bad[hit[0]] * 0.5
            assert float((plain.forward(c, bad, toks)[0] - full).abs().max()) > 1e-2, planted


# ---- configuration, checkpoints, registry ----------------------------------------------------------------------------------------
@pytest.mark.parametrize("name", sorted(cases.CONFIGS))
def test_config_reads_every_size_and_orders_the_runs(name):
    from vllmini_amd.voduvik import VoduvikConfig

    c = cases.CONFIGS[name]
    cfg = VoduvikConfig.from_json(c)
    assert cfg.order() == plain.layer_runs(c)
    assert cfg.tensor_shapes() == cases.shapes(c)


def test_config_refuses_what_the_design_does_not_have():
    from vllmini_amd.voduvik import VoduvikConfig

    c = cases.config([{"type": "sliding", "mixer": {}, "mlp": None}])
    with pytest.raises(ValueError, match="unknown mixer"):
        VoduvikConfig.from_json(c)
    with pytest.raises(ValueError, match="feed-forward"):
        VoduvikConfig.from_json(cases.config([cases.rglru(32, 1, mlp={"kind": "experts", "ff": 8, "limit": 1.0})]))
    with pytest.raises(ValueError, match="loop"):
        VoduvikConfig.from_json(cases.config([cases.rglru(32, 1)], loop=(0, 2, 2)))


def test_safetensors_reader_round_trip_and_bounds(tmp_path):
    from vllmini_amd.weights import load_checkpoint, read_safetensors

    named = {"a": torch.randn(3, 5).to(torch.bfloat16), "b.c": torch.arange(7, dtype=torch.int32), "s": torch.randn(2, 1, 2)}
    cases.write_safetensors(tmp_path / "x.safetensors", named)
    got = load_checkpoint(str(tmp_path))
    assert set(got) == set(named)
    for k in named:
        assert got[k].dtype == named[k].dtype and torch.equal(got[k], named[k])
    raw = (tmp_path / "x.safetensors").read_bytes()
    (tmp_path / "cut.safetensors").write_bytes(raw[:-4])
    with pytest.raises(ValueError, match="extent"):
        read_safetensors(str(tmp_path / "cut.safetensors"))
    (tmp_path / "bad.safetensors").write_bytes((1 << 40).to_bytes(8, "little") + raw[8:])
    with pytest.raises(ValueError, match="header"):
        read_safetensors(str(tmp_path / "bad.safetensors"))


def test_registry_names_the_architecture_and_refuses_unknown_ones(tmp_path):
    from vllmini_amd import registry

    assert {"Voduvik", "GPT2LMHeadModel"} <= set(registry.architectures())
    assert registry.architecture_of({"architecture": "Voduvik"}) == "Voduvik"
    assert registry.architecture_of({"architectures": ["GPT2LMHeadModel"], "model_type": "gpt2"}) == "GPT2LMHeadModel"
    with pytest.raises(ValueError, match="no known architecture"):
        registry.architecture_of({"architecture": "Somethingelse"})
    folder = cases.write_model(tmp_path / "m", cases.CONFIGS["mixed"], cases.tensors(cases.CONFIGS["mixed"]))
    with pytest.raises(registry.UnsupportedDtype):
        registry.load_decoder(folder, dtype="float16", max_tokens=64, max_seqs=1, device="cpu")


def test_builder_refuses_missing_and_misshapen_tensors():
    from vllmini_amd.voduvik import VoduvikConfig, build_model

    c = cases.CONFIGS["no_loop"]
    w = cases.tensors(c)
    cfg = VoduvikConfig.from_json(c)
    with pytest.raises(KeyError, match="l1.mix.lam"):
        build_model(cfg, {k: v for k, v in w.items() if k != "l1.mix.lam"}, torch.float32, "cpu")
    with pytest.raises(ValueError, match="head"):
        build_model(cfg, {**w, "head": w["head"][:-1]}, torch.float32, "cpu")
    m = build_model(cfg, w, torch.float32, "cpu")
    assert len(m.runs) == 3 and m.head.w.N % 32 == 0


def test_padded_layouts_keep_the_products():
    """Tiles and padding only rearrange: the padded input projection of a latent-attention layer, read back, is the checkpoint's."""
    from vllmini_amd.voduvik import VoduvikConfig, build_model

    c = cases.CONFIGS["mixed"]
    w = cases.tensors(c)
    a = build_model(VoduvikConfig.from_json(c), w, torch.float32, "cpu").runs[1].mixer
    d = a.w_in.dense
    H, dim, rot, rank, E = 3, 20, 12, 40, c["width"]
    q = d[: H * (a.dim + a.rot), :E].view(H, a.dim + a.rot, E)
    assert torch.equal(q[:, :dim], w["l1.mix.q"].float().view(H, dim + rot, E)[:, :dim])
    assert torch.equal(q[:, a.dim:a.dim + rot], w["l1.mix.q"].float().view(H, dim + rot, E)[:, dim:])
    assert not q[:, dim:a.dim].any() and not q[:, a.dim + rot:].any() and not d[:, E:].any()
    at = H * (a.dim + a.rot)
    assert torch.equal(d[at:at + rank, :E], w["l1.mix.dkv"].float()[:rank])
    assert torch.equal(d[at + a.rank:at + a.rank + rot, :E], w["l1.mix.dkv"].float()[rank:])
    assert torch.equal(d[a.gate_at:a.gate_at + H, :E], w["l1.mix.g"].float())
    t = a.w_in.tiles[0]                                        # [N / 16][K / 32][kc][r][e]
    back = t.permute(0, 3, 1, 2, 4).reshape(a.w_in.N, a.w_in.K)
    assert torch.equal(back, d)


# ---- the pool ---------------------------------------------------------------------------------------------------------------------
def _pool(blocks=6, page=4, slots=2, per_seq=6):
    from vllmini_amd.kv_pool import PagedKVPool

    return PagedKVPool(blocks, 1, 8, page, per_seq, 1, device="cpu", page_rows=[8, 16], page_dtype=torch.float32,
                       state=[((5,), torch.float32)], state_slots=slots)


def test_pool_append_hands_out_positions_slots_and_parities():
    p = _pool()
    p.open(7)
    a = p.append([7], [3])
    assert a["ctx"].tolist() == [0] and a["pos"].tolist() == [0, 1, 2] and a["slots"][0].tolist() == [0, 1, 2] and a["parity"].tolist() == [0]
    p.open(9)
    b = p.append([9, 7], [5, 2])                             # 9 takes two blocks, 7 crosses into a second one
    assert b["ctx"].tolist() == [0, 3] and b["entry"].tolist() == [0] * 5 + [1] * 2 and b["pos"].tolist() == [0, 1, 2, 3, 4, 3, 4]
    assert b["slots"][0].tolist() == [4, 5, 6, 7, 8, 3, 12] and b["parity"].tolist() == [0, 1]
    assert b["state_slot"].tolist() == [1, 0] and p.seq_len(7) == 5 and p.free_state_slots == 0
    with pytest.raises(RuntimeError, match="free blocks"):
        p.open(11)
    assert 11 not in p.allocated_blocks
    before = (list(p.free_blocks), p._tables.copy(), p._seq_len.copy(), p._parity.copy())
    with pytest.raises(RuntimeError, match="No free blocks"):      # 9: 5 -> 17 tokens needs 3 blocks, 2 are left
        p.append([7, 9], [1, 12])
    assert list(p.free_blocks) == before[0] and all(np.array_equal(x, y) for x, y in zip(before[1:], (p._tables, p._seq_len, p._parity)))
    with pytest.raises(RuntimeError, match="blocks per layer"):
        p.append([7], [40])
    p.free(9)
    p.open(11)                                                 # pages and slots come round again
    c = p.append([11], [9])
    assert c["state_slot"].tolist() == [1] and set(p.allocated_blocks[11]) & {1, 2}
    with pytest.raises(ValueError):
        p.append([7, 7], [1, 1])
    assert p.row_pages[0].shape == (6, 4, 8) and p.row_pages[1].shape == (6, 4, 16) and p.state[0].shape == (2, 5)


def test_pool_append_agrees_with_the_decode_step_of_the_key_value_layout():
    from vllmini_amd.kv_pool import PagedKVPool

    a, b = (PagedKVPool(40, 2, 8, 4, 8, 3, device="cpu", allocate_tensors=False) for _ in range(2))
    a.allocate_for_prefill(0, 6)
    b.allocate_for_prefill(0, 6)
    for _ in range(7):
        ta, sa, la = a.decode_step_batch([0])
        r = b.append([0], [1])
        assert np.array_equal(ta, r["tables"]) and np.array_equal(sa, r["slots"]) and la.tolist() == (r["ctx"] + 1).tolist()


# ---- portions of prompts in the scheduler --------------------------------------------------------------------------------------------
class _Stand:
    """A decoder whose next token is a hash of the sequence: whatever the schedule, a request's tokens must come out the same."""

    def __init__(self, pool, vocab=50):
        self.pool, self.vocab, self.seen, self.steps = pool, vocab, {}, []

    def _logits(self, seq):
        out = torch.zeros(self.vocab)
        out[(sum((i + 1) * t for i, t in enumerate(seq)) * 31 + len(seq)) % self.vocab] = 1.0
        return out

    def step(self, ids, tokens, want):
        a = self.pool.append(ids, [len(t) for t in tokens])
        self.steps.append([len(t) for t in tokens])
        rows = []
        for s, t, w, ctx in zip(ids, tokens, want, a["ctx"]):
            seq = ([] if ctx == 0 else self.seen[s]) + [int(x) for x in t]
            assert len(seq) == ctx + len(t)
            self.seen[s] = seq
            rows += [self._logits(seq[: ctx + k + 1]) for k in w]
        return torch.stack(rows) if rows else None

    def prefill_batch(self, ids, prompts):
        for i in ids:
            self.pool.open(i)
        return self.step(ids, prompts, [[len(p) - 1] for p in prompts])

    paged_prefill = True

    def prefill(self, i, p):
        return self.prefill_batch([i], [p])[0]

    def decode(self, ids, tokens):
        return self.step(ids, [[int(t)] for t in tokens], [[0]] * len(ids))


def _generate(prompts, new, blocks, chunk, max_batch=3, slots=3):
    from vllmini_amd.kv_pool import PagedKVPool
    from vllmini_amd.scheduler import BatchScheduler, sample_greedy

    pool = PagedKVPool(blocks, 1, 8, 4, 40, 1, device="cpu", page_rows=[8], page_dtype=torch.float32, state_slots=slots,
                       allocate_tensors=False, host_blocks=100)
    dec = _Stand(pool)
    sch = BatchScheduler(dec, max_length=120, eos_token_id=-1, max_batch=max_batch, sampler=sample_greedy, prefill_chunk=chunk)
    ids = [sch.submit(p, max_new_tokens=n) for p, n in zip(prompts, new)]
    sch.run(max_steps=2000)
    assert not sch.pending() and len(pool.free_blocks) == blocks and pool.free_state_slots == slots
    return [sch.sequences[i] for i in ids], sch, dec


@pytest.mark.parametrize("chunk", [2, 5, 16])
@pytest.mark.parametrize("blocks", [60, 14])
def test_scheduler_runs_portions_beside_single_tokens(chunk, blocks):
    rng = np.random.default_rng(3)
    prompts = [rng.integers(0, 50, n).tolist() for n in (21, 1, 9, 30, 4, 17)]
    new = [6, 9, 3, 5, 12, 7]
    want, _, _ = _generate(prompts, new, 200, 0, max_batch=6, slots=6)
    got, sch, dec = _generate(prompts, new, blocks, chunk)
    assert got == want and not sch.rejected and not sch.evicted
    assert any(1 in s and max(s) > 1 for s in dec.steps), "no step mixed a portion with single tokens"
    assert max(sum(n for n in s if n > 1) for s in dec.steps) <= chunk


def test_scheduler_rejects_a_prompt_no_pool_can_hold_and_aborts_unfinished_ones():
    got, sch, _ = _generate([[1] * 90, [2, 3, 4]], [2, 2], 10, 8)
    assert list(sch.rejected) == [0] and len(got[1]) == 5
    from vllmini_amd.kv_pool import PagedKVPool
    from vllmini_amd.scheduler import BatchScheduler, sample_greedy

    pool = PagedKVPool(30, 1, 8, 4, 40, 1, device="cpu", page_rows=[8], state_slots=2, allocate_tensors=False)
    sch = BatchScheduler(_Stand(pool), max_length=100, eos_token_id=-1, sampler=sample_greedy, prefill_chunk=4)
    i = sch.submit([5] * 20, max_new_tokens=3)
    sch.step()
    assert sch.prefilling == {i: 4} and sch.abort(i) and len(pool.free_blocks) == 30 and not sch.pending()
    with pytest.raises(ValueError, match="step"):
        BatchScheduler(object(), max_length=4, eos_token_id=0, prefill_chunk=4)


# ---- the library's boundary ------------------------------------------------------------------------------------------------------
def test_hybrid_library_exports_its_header_and_nothing_else():
    from vllmini_amd import build, hybrid_ops

    path = build.build_hybrid()
    src = re.sub(r"/\*.*?\*/", "", open(os.path.join(REPO, "include", "vmi_hybrid.h")).read(), flags=re.S)
    declared = set(re.findall(r"\b(vmi_hy(?:brid)?_[a-z0-9_]+)\s*\(", src))
    assert declared == set(hybrid_ops.SIGNATURES)
    r = subprocess.run(["nm", "-D", "--defined-only", path], capture_output=True, text=True, check=True)
    funcs = {ln.split()[-1] for ln in r.stdout.splitlines() if ln.strip() and ln.split()[-2] in "TtWw"}
    assert funcs == declared, funcs ^ declared
    lib = hybrid_ops.load()
    assert lib.vmi_hybrid_abi_version() == hybrid_ops.ABI_VERSION and lib.vmi_hybrid_target_arch() == b"gfx950"


def test_hybrid_entries_refuse_bad_arguments_without_touching_a_device():
    from vllmini_amd import hybrid_ops as h

    lib = h.load()
    assert lib.vmi_hy_linear(ctypes.byref(h.LinearArgs()), None) == 1
    buf = (ctypes.c_char * 256)()
    p = (ctypes.addressof(buf) + 15) & ~15
    a = h.LinearArgs(x=p, w=p, y=p, M=1, N=16, K=40, groups=1, ldx=40, ldy=16)
    assert lib.vmi_hy_linear(ctypes.byref(a), None) == 2 and b"K % 32" in lib.vmi_hybrid_last_error()
    assert lib.vmi_hy_rglru(ctypes.byref(h.RglruArgs()), ctypes.byref(h.StepArgs()), None) == 1
    assert lib.vmi_hy_latent_attention(ctypes.byref(h.AttentionArgs()), ctypes.byref(h.StepArgs()), None) == 1
    assert lib.vmi_hy_latent_prep(ctypes.byref(h.PrepArgs()), ctypes.byref(h.StepArgs()), None) == 1
    with pytest.raises(RuntimeError, match="no CPU path"):
        h.argmax(torch.zeros(1, 4))
    # what a workgroup can hold: never more row tiles than fit beside 64 keys, fp32 one
    assert [h.latent_row_tiles(576, n, torch.bfloat16) for n in (1, 2, 4)] == [1, 2, 4]
    assert h.latent_row_tiles(576, 4, torch.float32) == 1 and h.latent_row_tiles(640, 4, torch.bfloat16) == 2
    assert h.latent_row_tiles(1000, 4, torch.bfloat16) == 1


def test_command_line_lists_models_and_parses_requests(capsys):
    from vllmini_amd.__main__ import _parser, main

    assert main(["models"]) == 0 and "Voduvik" in capsys.readouterr().out
    a = _parser().parse_args(["generate", "--model", "x", "--prompt-ids", "1,2", "--prompt-ids", "3", "--prefill-chunk", "8"])
    assert a.prompt_ids == ["1,2", "3"] and a.prefill_chunk == 8
    r = subprocess.run([os.path.join(REPO, "bin", "trace_run"), "--help"], capture_output=True, text=True)
    assert r.returncode == 0 and "--max-tokens" in r.stdout
