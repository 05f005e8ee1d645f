"""A decoder over hybrid_layers: recurrences, linear and softmax attention, in any order, some of them run several times.

The counterpart of GPT2PagedDecoder for models that are described by a list of layer runs (`HybridModel`): same pool
(kv_pool.PagedKVPool with row pages and state slots), same scheduler (prefill / prefill_batch / decode / greedy), one forward
pass for everything: `step()` takes, for any number of sequences, the next tokens of each — a whole prompt, a portion of one, one
sampled token — and runs them as one packed batch from the cache and state that earlier steps left.  decode() is the step in
which every portion is one token, replayed from a hipGraph when asked to.

Every layer RUN has its own cache / state: a layer inside a loop keeps one per pass.
"""
from __future__ import annotations

import dataclasses
from typing import Dict, List, Optional, Sequence, Union

import numpy as np
import torch

from . import hybrid_ops as ops
from .hybrid_layers import AttentionPlan, ClampedGLU, ConcatProjection, Head, LatentAttention, ParallelBlock, QueryTiling, Residual, RGLRU
from .kv_pool import PagedKVPool


@dataclasses.dataclass
class LayerRun:
    """One pass through one layer: an input projection in front of it (or None), its mixer, its feed-forward (or None; a
    ParallelBlock brings its own)."""
    mixer: Union[LatentAttention, RGLRU, ParallelBlock]
    mlp: Optional[ClampedGLU] = None
    enter: Optional[ConcatProjection] = None


@dataclasses.dataclass
class HybridModel:
    vocab_size: int
    width: int
    dtype: torch.dtype
    device: torch.device
    embed: torch.Tensor            # bfloat16 [vocab, width padded to 32]
    embed_scale: float
    runs: List[LayerRun]
    head: Head
    eos_token_id: int = -1         # (a design without one: generation ends at its length)

    def make_pool(self, max_tokens: int, max_seqs: int, page_size: int = 64, max_length: Optional[int] = None, **kw) -> PagedKVPool:
        """A pool for max_tokens tokens of live sequences (each rounded up to whole pages) and max_seqs sequences.  max_length:
        the longest a sequence may get (default: it may take the whole pool)."""
        blocks = max(1, max_tokens // page_size)
        per_seq = blocks if max_length is None else -(-max_length // page_size)
        rows = [n for r in self.runs for n in r.mixer.page_rows()]
        state = [s for r in self.runs for s in r.mixer.state_shapes()]
        return PagedKVPool(blocks, 1, max(rows, default=1), page_size, per_seq + 1, 1, device=self.device, max_seqs=max_seqs,
                           page_rows=rows, page_dtype=self.dtype, state=state, state_slots=max_seqs, **kw)


class HybridDecoder:
    MAX_STEP_TOKENS = 16384        # longer prompts run in several portions
    FILL_WORKGROUPS = {1: 512, 2: 256, 4: 256}     # by row tiles, what the chip holds at once: a step with fewer query tiles splits
                                                   # the keys of each over several workgroups
    KEY_TILE = 64

    def __init__(self, model: HybridModel, pool: PagedKVPool, pad_batch_to: int = 0):
        self.model, self.pool, self.device = model, pool, model.device
        if pool.page_rows is None:
            raise ValueError("HybridDecoder needs a pool with row pages (HybridModel.make_pool)")
        ops.load()
        self.pad_batch_to = int(pad_batch_to)
        self.paged_prefill = True                      # (prefill_batch is the one prefill there is)
        self._slots: List[tuple] = []                  # per run: its cache tensors, then its states
        ip = iter(pool.row_pages)
        st = iter(pool.state)
        for r in model.runs:
            self._slots.append((*(next(ip) for _ in r.mixer.page_rows()), *(next(st) for _ in r.mixer.state_shapes())))
        self._kinds: List[QueryTiling] = sorted({r.mixer.tiling() for r in model.runs} - {None})
        self.tap: Optional[List[torch.Tensor]] = None  # set to a list: the residual stream after every layer run is appended to it
        self._stage: List[list] = []                   # pinned staging buffers: [tensor, event]
        self._stage_i = 0
        self._sets: Dict[tuple, dict] = {}             # captured decode steps

    # ---- the step's layout -----------------------------------------------------------------------------------------------
    def _split_of(self, n_tiles: int, row_tiles: int, kind: QueryTiling, max_keys: int, T: int) -> int:
        n_tiles *= kind.sets
        if n_tiles > 128:
            return 1
        max_keys = min(max_keys, kind.chunk) if kind.chunk else max_keys
        want = min(self.FILL_WORKGROUPS[row_tiles] // max(n_tiles, 1), -(-max_keys // self.KEY_TILE))
        fit = (256 << 20) // max(1, T * kind.rep * kind.sets * (kind.width + 2) * 4)       # (bytes of the partial results)
        n = 1
        while 2 * n <= min(want, fit, 128):
            n *= 2
        return n

    def _layout(self, a: dict, counts: np.ndarray, rows: np.ndarray, T: int, B: int, table_ld: int, max_keys: int):
        """One int32 buffer with everything a step's kernels read, as named sections; T / B may exceed what is there (padding)."""
        n, b = int(counts.sum()), len(counts)
        starts = np.cumsum(counts) - counts
        sec: Dict[str, np.ndarray] = {}

        def put(name, size, values, fill):
            buf = np.full(size, fill, dtype=np.int32)
            buf[: len(values)] = values
            sec[name] = buf

        put("tok_seq", T, a["entry"], -1)
        put("tok_pos", T, a["pos"], 0)
        put("tok_slot", T, a["slots"][0], -1)
        put("q_start", B, starts, n)
        put("q_len", B, counts, 0)
        put("ctx", B, a["ctx"], 0)
        put("state_slot", B, a["state_slot"], 0)
        put("flip", B, a["parity"], 0)
        tab = np.zeros((B, table_ld), dtype=np.int32)
        w = min(table_ld, a["tables"].shape[2])
        tab[:b, :w] = np.maximum(a["tables"][0][:, :w], 0)
        sec["table"] = tab.reshape(-1)
        put("rows", max(len(rows), 1), rows, 0)
        plans = []
        for kind in self._kinds:
            rep, longest = kind.rep, int(counts.max()) * kind.rep
            rt = kind.row_tiles(4 if longest > 32 else 2 if longest > 16 else 1, self.model.dtype)
            per = -(-(counts * rep) // (16 * rt))
            ent = np.repeat(np.arange(b), per)
            first = (np.arange(int(per.sum())) - np.repeat(np.cumsum(per) - per, per)) * 16 * rt
            if b > 1 or len(first) > 1:       # longest first: the tail of the launch is short tiles
                keys = a["ctx"][ent] + (first + 16 * rt - 1) // rep
                order = np.argsort(-(keys % kind.chunk if kind.chunk else keys), kind="stable")
                ent, first = ent[order], first[order]
            nt = len(ent) + (B - b) * (-(-rep // (16 * rt)))
            t = np.full((nt, 2), -1, dtype=np.int32)
            t[: len(ent), 0], t[: len(ent), 1] = ent, first
            sec[f"tiles{len(plans)}"] = t.reshape(-1)
            plans.append((rt, self._split_of(nt, rt, kind, max_keys, T), nt))
        if (counts > 1).any():                # runs of rows for the linear-attention layers
            per = -(-counts // ops.CHUNK_ROWS)
            at = np.cumsum(per) - per
            put("chunk_start", B, at, 0)
            ent = np.repeat(np.arange(b), per)
            sec["chunks"] = np.stack([ent, (np.arange(int(per.sum())) - at[ent]) * ops.CHUNK_ROWS], axis=1).astype(np.int32).reshape(-1)
        offs, total = {}, 0
        for name, v in sec.items():
            offs[name] = (total, len(v))
            total += (len(v) + 3) // 4 * 4
        return sec, offs, total, plans

    def _upload(self, sec, offs, total: int, out: Optional[torch.Tensor] = None) -> torch.Tensor:
        """The sections into device memory with one asynchronous copy from pinned memory (a ring of four staging buffers)."""
        if out is None:
            out = torch.empty(total, dtype=torch.int32, device=self.device)
        if len(self._stage) < 4:
            self._stage.append([torch.empty(max(total, 1 << 14), dtype=torch.int32, pin_memory=True), None])
            i = len(self._stage) - 1
        else:
            i = self._stage_i = (self._stage_i + 1) % 4
        buf, ev = self._stage[i]
        if ev is not None:
            ev.synchronize()                    # its previous copy has run
        if buf.numel() < total:
            buf = self._stage[i][0] = torch.empty(2 * total, dtype=torch.int32, pin_memory=True)
        host = buf.numpy()
        for name, v in sec.items():
            host[offs[name][0]: offs[name][0] + len(v)] = v
        out.copy_(buf[:total], non_blocking=True)
        ev = torch.cuda.Event()
        ev.record()
        self._stage[i][1] = ev
        return out

    def _views(self, dev: torch.Tensor, offs, B: int, table_ld: int, plans):
        v = {k: dev[o: o + n] for k, (o, n) in offs.items()}
        v["table"] = v["table"].view(B, table_ld)
        if "chunks" in v:
            v["chunks"] = v["chunks"].view(-1, 2)
        plan = {kind: AttentionPlan(v[f"tiles{i}"].view(nt, 2), rt, sp) for i, (kind, (rt, sp, nt)) in enumerate(zip(self._kinds, plans))}
        return v, plan

    # ---- the forward pass --------------------------------------------------------------------------------------------------
    def _forward(self, ids: torch.Tensor, step: ops.StepLayout, plans, rows: Optional[torch.Tensor]) -> Optional[torch.Tensor]:
        m = self.model
        step.begin()
        x0 = ops.embed(ids, m.embed, m.width, m.embed_scale)
        loops = any(r.enter is not None for r in m.runs)
        res = Residual(x0.clone() if loops and m.runs[0].enter is None else x0, m.dtype)
        for r, held in zip(m.runs, self._slots):
            if r.enter is not None:
                r.enter.run(res, x0)
            r.mixer.run(res, step, plans, held)
            if r.mlp is not None:
                r.mlp.run(res, step)
            if self.tap is not None:
                self.tap.append(res.settle()[:, : m.width].clone())
        if rows is None:
            return None
        return m.head.run(res.settle(), rows)

    def _ids(self, tokens: Sequence) -> torch.Tensor:
        """The step's token ids on the device; host ids are range-checked here."""
        parts, host = [], []
        for t in tokens:
            if isinstance(t, torch.Tensor) and t.is_cuda:
                if host:
                    parts.append(torch.tensor(host, dtype=torch.int64))
                    host = []
                parts.append(t.reshape(-1).to(torch.int64))
            else:
                host.extend(int(x) for x in t)
        if host:
            parts.append(torch.tensor(host, dtype=torch.int64))
        for t in parts:
            if not t.is_cuda and t.numel() and (int(t.min()) < 0 or int(t.max()) >= self.model.vocab_size):
                raise ValueError(f"token id out of range (vocabulary of {self.model.vocab_size})")
        return torch.cat([t.to(self.device, non_blocking=True) for t in parts]) if len(parts) > 1 else parts[0].to(self.device)

    @torch.no_grad()
    def step(self, seq_ids: Sequence[int], tokens: Sequence, want: Optional[Sequence[Sequence[int]]] = None) -> Optional[torch.Tensor]:
        """tokens[i] (list or device tensor) are the next tokens of sequence seq_ids[i]; all of it is one batch.  Returns the
        logits (float32 [n, V]) at the wanted places — want[i]: places among tokens[i]; default: the last of each — entry by
        entry, or None when nothing is wanted.  Sequences are opened with pool.open() before their first step."""
        counts = np.asarray([len(t) for t in tokens], dtype=np.int64)
        starts = np.cumsum(counts) - counts
        if want is None:
            rows = starts + counts - 1
        else:
            for w, c in zip(want, counts):
                if any(not 0 <= int(k) < c for k in w):
                    raise ValueError("wanted places must lie inside their portion")
            rows = np.asarray([int(s) + int(k) for s, w in zip(starts, want) for k in w], dtype=np.int64)
        return self._run(seq_ids, counts, self._ids(tokens), rows)

    def _run(self, seq_ids: Sequence[int], counts: np.ndarray, ids: torch.Tensor, rows: np.ndarray) -> Optional[torch.Tensor]:
        T, B, starts = int(counts.sum()), len(counts), np.cumsum(counts) - counts
        if T > 65535:
            raise ValueError("a step holds at most 65535 tokens")
        a = self.pool.append(seq_ids, counts)
        keys = int((a["ctx"] + counts).max())
        ld = -(-keys // self.pool.block_size)
        sec, offs, total, plans = self._layout(a, counts, rows, T, B, ld, keys)
        v, plan = self._views(self._upload(sec, offs, total), offs, B, ld, plans)
        spans = bool((starts // ops.ROW_TILE != (starts + counts - 1) // ops.ROW_TILE).any())
        layout = ops.StepLayout(v, T, B, self.pool.block_size, bool((counts == 1).all()), spans, int(counts.max()), keys)
        return self._forward(ids, layout, plan, v["rows"] if len(rows) else None)

    # ---- what the scheduler calls -------------------------------------------------------------------------------------------
    def prefill(self, seq_id: int, input_ids: Sequence[int]) -> torch.Tensor:
        return self.prefill_batch([seq_id], [input_ids])[0]

    @torch.no_grad()
    def prefill_batch(self, seq_ids: Sequence[int], prompts: Sequence[Sequence[int]]) -> torch.Tensor:
        """Opens the sequences and runs their prompts, MAX_STEP_TOKENS at a time; last-token logits [n, V].  All or nothing."""
        if any(len(p) == 0 for p in prompts):
            raise ValueError("a prompt needs at least one token")
        opened: List[int] = []
        out: List[Optional[torch.Tensor]] = [None] * len(seq_ids)
        try:
            for s in seq_ids:
                self.pool.open(s)
                opened.append(s)
            done = [0] * len(prompts)
            while any(d < len(p) for d, p in zip(done, prompts)):
                room, ent = self.MAX_STEP_TOKENS, []
                for i, p in enumerate(prompts):
                    n = min(len(p) - done[i], room)
                    if n > 0:
                        ent.append((i, done[i], n))
                        room -= n
                last = [i for i, d, n in ent if d + n == len(prompts[i])]
                lg = self.step([seq_ids[i] for i, _, _ in ent], [list(prompts[i][d:d + n]) for i, d, n in ent],
                               [[n - 1] if i in last else [] for i, d, n in ent])
                for k, i in enumerate(last):
                    out[i] = lg[k]
                for i, d, n in ent:
                    done[i] = d + n
        except RuntimeError:
            for s in opened:
                self.pool.free(s)
            raise
        return torch.stack(out) if out else torch.empty((0, self.model.vocab_size), device=self.device)

    def _padded(self, B: int) -> int:
        m = self.pad_batch_to
        return B if not m or B % m == 0 else (B // m + 1) * m

    @torch.no_grad()
    def decode(self, seq_ids: Sequence[int], input_ids, use_graph: bool = False) -> torch.Tensor:
        """One token per sequence; logits [B, V].  use_graph: the launches are replayed from a hipGraph, captured once per
        (padded batch size, number of key splits)."""
        B = len(seq_ids)
        ids = input_ids.reshape(-1).to(self.device, torch.int64) if isinstance(input_ids, torch.Tensor) else self._ids([list(input_ids)])
        if not use_graph:
            return self._run(seq_ids, np.ones(B, dtype=np.int64), ids, np.arange(B))
        Bp, MB = self._padded(B), self.pool.max_blocks_per_seq
        counts = np.ones(B, dtype=np.int64)
        a = self.pool.append(seq_ids, counts)
        keys = int(a["ctx"].max()) + 1
        bucket = 2 * self.KEY_TILE
        while bucket < keys:
            bucket *= 2
        sec, offs, total, plans = self._layout(a, counts, np.arange(Bp), Bp, Bp, MB, bucket)
        key = (Bp, tuple(plans))
        hit = self._sets.get(key)
        if hit is None:
            hit = self._sets[key] = {"meta": torch.zeros(total, dtype=torch.int32, device=self.device),
                                     "ids": torch.zeros(Bp, dtype=torch.int64, device=self.device), "graph": None}
        self._upload(sec, offs, total, hit["meta"])
        hit["ids"][:B].copy_(ids, non_blocking=True)
        if hit["graph"] is None:
            v, plan = self._views(hit["meta"], offs, Bp, MB, plans)
            layout = ops.StepLayout(v, Bp, Bp, self.pool.block_size, True, False, 1, bucket)
            # capturing launches nothing; what needs a first run outside a capture is the kernels' LDS allowance and the library,
            # so the step's FIRST execution is eager and it is its result that is returned — a step must not run twice, the
            # recurrent state would advance twice
            out = self._forward(hit["ids"], layout, plan, v["rows"])
            first = out[:B].clone()
            s = torch.cuda.Stream(self.device)
            s.wait_stream(torch.cuda.current_stream(self.device))
            graph = torch.cuda.CUDAGraph()
            with torch.cuda.graph(graph, stream=s):
                out = self._forward(hit["ids"], layout, plan, v["rows"])
            hit["graph"], hit["out"], hit["keep"] = graph, out, (layout, plan)
            return first
        hit["graph"].replay()
        return hit["out"][:B]

    def greedy(self, logits: torch.Tensor) -> torch.Tensor:
        return ops.argmax(logits)
