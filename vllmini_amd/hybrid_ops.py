"""Operators of libvmi_hybrid.so (include/vmi_hybrid.h): what decoders that mix recurrences, linear and softmax attention are made of.

Thin ctypes wrappers over csrc/hybrid_*.hip that check operands on the host (devices, dtypes, shapes, strides — a kernel never
sees sizes that do not fit its buffers) and launch on torch's current stream.  There is no torch fallback: a missing library or
an unsupported shape raises.  Two element types: torch.bfloat16 (what models are served in) and torch.float32 (every product in
full 32 bits).

    linear            y = epilogue(prologue(x) W^T): norm / concatenation in front, residual add / gated unit / head gate behind
    embed, add_norm, merge, glu, argmax
    rglru             causal convolution + block-diagonal gates + gated linear recurrence + gelu(y) product
    latent_prep       RMS norm of the latent, rotary parts, cache write
    latent_attention  softmax attention in the latent space over the paged cache
    linear_state      linear attention with a matrix state per head: retention, the gated delta rule
    kv_prep           RMS norms of q and k, cache write
    attention         grouped-query softmax attention over the paged cache: chunks, bias by distance, sink, output gate

StepLayout describes the tokens of one step to the latter ones.
"""
from __future__ import annotations

import ctypes
import os
import threading
from typing import NamedTuple, Optional, Tuple

import torch

from . import build as _build

ABI_VERSION = 2
DTYPES = {torch.bfloat16: 0, torch.float32: 1}
X_ROWS, X_NORM, X_CONCAT = 0, 1, 2
E_STORE, E_RESIDUAL, E_FLOAT, E_GLU, E_GATED, E_STORE_GLU = 0, 1, 2, 3, 4, 5
RETENTION, DELTA = 0, 1
ACTS = {"sigmoid": 0, "silu": 1}
CHUNK_ROWS = 16     # rows of a chunk of the linear-attention kernels
STATE_DIMS = (32, 64, 96, 128, 192, 256, 512)       # key dimensions they are built for

_vp, _i32, _i64, _f32 = ctypes.c_void_p, ctypes.c_int32, ctypes.c_int64, ctypes.c_float


def _struct(name, fields):
    return type(name, (ctypes.Structure,), {"_fields_": [(n, t) for t, names in fields for n in names.split()]})


LinearArgs = _struct("LinearArgs", [(_vp, "x x2 rows norm_w w bias gate y y2"), (_i64, "ldx ldy ldg ldy2 x_gstride y_gstride"),
                                    (_i32, "M N K groups norm_n n_out n_split rms"), (_f32, "eps scale glu_alpha glu_up"),
                                    (_i32, "x_kind epilogue dtype device")])
StepArgs = _struct("StepArgs", [(_vp, "tok_seq tok_pos tok_slot q_start q_len ctx state_slot flip table chunks chunk_start"),
                                (_i32, "T B table_ld page_size n_chunks")])
RglruArgs = _struct("RglruArgs", [(_vp, "yx out conv_w conv_b gates gate_b decay state tail scratch carry"), (_i64, "ldx ldo"),
                                  (_i32, "width blocks taps single spans dtype device")])
PrepArgs = _struct("PrepArgs", [(_vp, "proj q cache norm_w freq"), (_i64, "ldp"), (_i32, "heads dim rot rank rot_n rank_n"),
                                (_f32, "eps"), (_i32, "dtype device")])
AttentionArgs = _struct("AttentionArgs", [(_vp, "q cache out tiles partial"), (_i32, "heads rank rot n_tiles row_tiles splits"),
                                          (_f32, "scale"), (_i32, "dtype device")])
StateArgs = _struct("StateArgs", [(_vp, "proj beta z conv_w rate dt_bias decay log2_decay turns state tail o scratch out gate norm_w"),
                                  (_i64, "ldp ldz ldo ldg"),
                                  (_i32, "heads kv_heads dim vdim dim_n vdim_n taps rot_n kind single act"), (_f32, "eps"),
                                  (_i32, "dtype device")])
KvPrepArgs = _struct("KvPrepArgs", [(_vp, "proj q cache"), (_i64, "ldp"), (_i32, "heads kv_heads dim vdim dim_n"), (_f32, "eps"),
                                    (_i32, "dtype device")])
GqaArgs = _struct("GqaArgs", [(_vp, "q cache out bias sink gate tiles partial"), (_i64, "ldo ldg"),
                              (_i32, "heads kv_heads dim vdim bias_n chunk n_tiles row_tiles splits"), (_f32, "scale"),
                              (_i32, "dtype device")])

SIGNATURES = {
    "vmi_hy_linear": (ctypes.c_int, [ctypes.POINTER(LinearArgs), _vp]),
    "vmi_hy_embed": (ctypes.c_int, [_vp, _vp, _vp, _i32, _i32, _i32, _i32, _f32, _i32, _vp]),
    "vmi_hy_add_norm": (ctypes.c_int, [_vp, _vp, _i64, _vp, _vp, _i32, _i32, _i32, _f32, _i32, _i32, _i32, _vp]),
    "vmi_hy_merge": (ctypes.c_int, [_vp, _vp, _i64, _vp, _i64, _vp, _i64, _vp, _vp, _i32, _i32, _i32, _f32, _f32, _i32, _i32, _vp]),
    "vmi_hy_glu": (ctypes.c_int, [_vp, _i64, _vp, _i64, _i32, _i32, _f32, _f32, _f32, _i32, _i32, _vp]),
    "vmi_hy_rotations": (ctypes.c_int, [_vp, _i32, _vp, ctypes.POINTER(StepArgs), _i32, _vp]),
    "vmi_hy_state_scratch": (_i64, [_i32, _i32, _i32]),
    "vmi_hy_state_fuses": (_i32, [_i32, _i32]),
    "vmi_hy_state": (ctypes.c_int, [ctypes.POINTER(StateArgs), ctypes.POINTER(StepArgs), _vp]),
    "vmi_hy_kv_prep": (ctypes.c_int, [ctypes.POINTER(KvPrepArgs), ctypes.POINTER(StepArgs), _vp]),
    "vmi_hy_attention_row_tiles": (_i32, [_i32, _i32, _i32, _i32]),
    "vmi_hy_attention": (ctypes.c_int, [ctypes.POINTER(GqaArgs), ctypes.POINTER(StepArgs), _vp]),
    "vmi_hy_concat": (ctypes.c_int, [_vp, _vp, _vp, _i32, _i32, _i32, _i32, _vp]),
    "vmi_hy_argmax": (ctypes.c_int, [_vp, _i64, _i32, _i32, _vp, _i32, _vp]),
    "vmi_hy_rglru": (ctypes.c_int, [ctypes.POINTER(RglruArgs), ctypes.POINTER(StepArgs), _vp]),
    "vmi_hy_latent_prep": (ctypes.c_int, [ctypes.POINTER(PrepArgs), ctypes.POINTER(StepArgs), _vp]),
    "vmi_hy_latent_row_tiles": (_i32, [_i32, _i32, _i32]),
    "vmi_hy_latent_attention": (ctypes.c_int, [ctypes.POINTER(AttentionArgs), ctypes.POINTER(StepArgs), _vp]),
    "vmi_hybrid_last_error": (ctypes.c_char_p, []),
    "vmi_hybrid_abi_version": (_i32, []),
    "vmi_hybrid_target_arch": (ctypes.c_char_p, []),
}

_lock = threading.Lock()
_lib = None


class HybridLibraryError(RuntimeError):
    """libvmi_hybrid.so is missing / stale / does not match the header."""


def load() -> ctypes.CDLL:
    global _lib
    if _lib is None:
        with _lock:
            if _lib is None:
                path = _build.HYBRID_LIB_PATH
                if not os.path.exists(path):
                    raise HybridLibraryError(f"{path} not found: build it with `python -m vllmini_amd.build` (or `make hybrid`)")
                try:
                    lib = ctypes.CDLL(path)
                except OSError as e:
                    raise HybridLibraryError(f"cannot load {path}: {e}") from e
                for name, (restype, argtypes) in SIGNATURES.items():
                    try:
                        fn = getattr(lib, name)
                    except AttributeError as e:
                        raise HybridLibraryError(f"{path} does not export {name}") from e
                    fn.restype, fn.argtypes = restype, argtypes
                if lib.vmi_hybrid_abi_version() != ABI_VERSION:
                    raise HybridLibraryError(f"{path}: ABI {lib.vmi_hybrid_abi_version()}, expected {ABI_VERSION}")
                _lib = lib
    return _lib


def _check(rc: int) -> None:
    if rc != 0:
        raise RuntimeError(load().vmi_hybrid_last_error().decode("utf-8", "replace"))


def _need(cond: bool, what: str) -> None:
    if not cond:
        raise RuntimeError(what)


def _ptr(t: Optional[torch.Tensor]):
    return None if t is None else t.data_ptr()


def _on(t: torch.Tensor) -> Tuple[int, int]:
    _need(t.device.type == "cuda", "hybrid_ops: there is no CPU path")
    idx = t.device.index if t.device.index is not None else torch.cuda.current_device()
    return idx, torch.cuda.current_stream(t.device).cuda_stream


def pad32(n: int) -> int:
    return (n + 31) // 32 * 32


def state_dim(n: int) -> int:
    """The key dimension that the linear-attention kernels are built for and that holds n."""
    for d in STATE_DIMS:
        if n <= d:
            return d
    raise ValueError(f"key dimensions beyond {STATE_DIMS[-1]} are not built")


class GatedUnit(NamedTuple):
    """g' sigmoid(alpha g') (u' + up) with g' = min(g, limit), u' = u clamped to +- limit."""
    limit: float
    alpha: float
    up: float

    @classmethod
    def clamped(cls, limit: float) -> "GatedUnit":
        return cls(float(limit), 1.702, 1.0)


SILU_UNIT = GatedUnit(float("inf"), 1.0, 0.0)      # silu(g) u
NormArgs = Tuple       # weight, true columns, eps, and whether it is an RMS norm (default: a layer norm)


def _rms(norm: Optional[NormArgs]) -> int:
    return int(norm is not None and len(norm) > 3 and norm[3])


class MatrixTiles:
    """Linear weights [N, K] (or a group of them, [G, N, K]) as the tiles the kernels stream, zero-padded to N % 32 == K % 32 == 0:
    tiles[g][s][t][kc * 16 + r][e] = w[g][16 s + r][32 t + 8 kc + e].  `dense=True` keeps the padded [N, K] as well (steps of many
    tokens go through the vendor's matrix product)."""

    def __init__(self, weight: torch.Tensor, dtype: torch.dtype, dense: bool = False):
        w = weight if weight.dim() == 3 else weight[None]
        G, N, K = w.shape
        self.groups, self.N, self.K = G, pad32(N), pad32(K)
        p = torch.zeros((G, self.N, self.K), dtype=dtype, device=w.device)
        p[:, :N, :K] = w.to(dtype)
        self.tiles = p.view(G, self.N // 16, 16, self.K // 32, 4, 8).permute(0, 1, 3, 4, 2, 5).contiguous()
        self.dense = p[0].contiguous() if dense and G == 1 else None


def linear(x: torch.Tensor, w: MatrixTiles, *, norm: Optional[NormArgs] = None, x2: Optional[torch.Tensor] = None,
           rows: Optional[torch.Tensor] = None, bias: Optional[torch.Tensor] = None, out: Optional[torch.Tensor] = None,
           residual: bool = False, float_out: Optional[Tuple[int, float]] = None, glu: Optional[GatedUnit] = None,
           glu_from: int = -1, glu_out: Optional[torch.Tensor] = None, gate: Optional[torch.Tensor] = None, x_gstride: int = 0,
           y_gstride: int = 0) -> torch.Tensor:
    """One linear layer over the rows of x.
        input     x [M, K] of the element type | norm=(weight, n, eps, rms): x float32, normed over its first n columns, optionally
                  of `rows` only | x2: x and x2 float32 side by side
        output    element type (+ bias) | residual=True: out (float32) += | float_out=(columns, scale): float32 | glu: the
                  gated unit of interleaved (gate, up) columns | gate [M, groups ...]: times sigmoid of the group's column |
                  glu and glu_from=n, glu_out: columns below n as they are, the gated unit of the others into glu_out
        groups    group g reads x at column g * x_gstride, writes out at column g * y_gstride"""
    lib = load()
    device, stream = _on(x)
    T = w.tiles.dtype
    kind = X_NORM if norm is not None else X_CONCAT if x2 is not None else X_ROWS
    epi = E_RESIDUAL if residual else E_FLOAT if float_out else (E_GLU if glu_out is None else E_STORE_GLU) if glu is not None else E_GATED if gate is not None else E_STORE
    M = int(rows.numel()) if rows is not None else int(x.shape[0])
    K, N = w.K, w.N
    span = (w.groups - 1) * x_gstride + (K // 2 if kind == X_CONCAT else K)
    _need(x.dim() == 2 and x.stride(1) == 1 and x.shape[1] >= span and x.dtype == (T if kind == X_ROWS else torch.float32),
          f"hybrid_ops.linear: x {tuple(x.shape)} {x.dtype} does not hold {w.groups} x {K} columns")
    if x2 is not None:
        _need(x2.shape == x.shape and x2.stride() == x.stride() and x2.dtype == torch.float32 and x2.device == x.device,
              "hybrid_ops.linear: x2 must match x")
    if norm is not None:
        _need(norm[0].dtype == torch.float32 and norm[0].numel() >= K and 0 < norm[1] <= K, "hybrid_ops.linear: norm weight float32 [K]")
    if rows is not None:
        _need(kind == X_NORM and rows.dtype == torch.int32 and rows.is_contiguous(), "hybrid_ops.linear: rows int32, with norm")
    if bias is not None:
        _need(bias.dtype == torch.float32 and bias.numel() >= N, "hybrid_ops.linear: bias float32 [N]")
    if gate is not None:
        _need(gate.dtype == T and gate.shape[0] == M and gate.stride(1) == 1 and gate.shape[1] >= w.groups, "hybrid_ops.linear: gate")
    if epi == E_STORE_GLU:
        _need(0 <= glu_from <= N and glu_from % 16 == 0 and glu_out.dtype == T and glu_out.dim() == 2 and glu_out.stride(1) == 1
              and glu_out.shape[0] == M and glu_out.shape[1] >= (N - glu_from) // 2 and glu_out.device == x.device
              and w.groups == 1, "hybrid_ops.linear: glu_out")
    cols = float_out[0] if epi == E_FLOAT else N // 2 if epi == E_GLU else glu_from if epi == E_STORE_GLU else (w.groups - 1) * y_gstride + N
    odt = torch.float32 if epi in (E_RESIDUAL, E_FLOAT) else T
    if out is None:
        out = torch.empty((M, cols), dtype=odt, device=x.device)
    _need(out.dim() == 2 and out.shape[0] == M and out.shape[1] >= cols and out.stride(1) == 1 and out.dtype == odt
          and out.data_ptr() != x.data_ptr(), f"hybrid_ops.linear: out {tuple(out.shape)} {out.dtype} for {M} x {cols}")
    a = LinearArgs(x=x.data_ptr(), x2=_ptr(x2), rows=_ptr(rows), norm_w=norm[0].data_ptr() if norm else None, w=w.tiles.data_ptr(),
                   bias=_ptr(bias), gate=_ptr(gate), y=out.data_ptr(), y2=_ptr(glu_out), ldx=x.stride(0), ldy=out.stride(0),
                   ldg=gate.stride(0) if gate is not None else 0, ldy2=glu_out.stride(0) if glu_out is not None else 0, x_gstride=x_gstride, y_gstride=y_gstride, M=M, N=N, K=K,
                   groups=w.groups, norm_n=norm[1] if norm else 0, n_out=float_out[0] if float_out else 0,
                   n_split=max(glu_from, 0), rms=_rms(norm), eps=norm[2] if norm else 0.0,
                   scale=float_out[1] if float_out else glu.limit if glu is not None else 1.0,
                   glu_alpha=glu.alpha if glu is not None else 0.0, glu_up=glu.up if glu is not None else 0.0,
                   x_kind=kind, epilogue=epi, dtype=DTYPES[T], device=device)
    _check(lib.vmi_hy_linear(ctypes.byref(a), stream))
    return out


def embed(ids: torch.Tensor, table: torch.Tensor, width: int, scale: float) -> torch.Tensor:
    """float32 [T, ld] = table[ids] * scale, zero past `width` (table bfloat16 [vocab, ld])."""
    device, stream = _on(ids)
    _need(ids.dtype == torch.int64 and ids.dim() == 1 and ids.is_contiguous() and table.dtype == torch.bfloat16
          and table.is_contiguous() and table.device == ids.device, "hybrid_ops.embed: int64 ids, bfloat16 table on one device")
    T, ld = ids.numel(), table.shape[1]
    x = torch.empty((T, ld), dtype=torch.float32, device=ids.device)
    _check(load().vmi_hy_embed(ids.data_ptr(), table.data_ptr(), x.data_ptr(), T, width, ld, table.shape[0], float(scale), device, stream))
    return x


def add_norm(x: torch.Tensor, add: Optional[torch.Tensor], norm: Optional[NormArgs], dtype: torch.dtype) -> Optional[torch.Tensor]:
    """x += add (if given), then the norm of x in `dtype` (if asked for)."""
    device, stream = _on(x)
    T, ld = x.shape
    _need(x.dtype == torch.float32 and x.is_contiguous(), "hybrid_ops.add_norm: x float32, contiguous")
    if add is not None:
        _need(add.shape[0] == T and add.shape[1] >= ld and add.stride(1) == 1 and add.dtype == dtype, "hybrid_ops.add_norm: add")
    out = None
    if norm is not None:
        _need(norm[0].dtype == torch.float32 and norm[0].numel() >= ld, "hybrid_ops.add_norm: norm weight float32 [ld]")
        out = torch.empty((T, ld), dtype=dtype, device=x.device)
    _check(load().vmi_hy_add_norm(x.data_ptr(), _ptr(add), add.stride(0) if add is not None else 0, norm[0].data_ptr() if norm else None,
                                  _ptr(out), T, norm[1] if norm else ld, ld, norm[2] if norm else 0.0, _rms(norm), DTYPES[dtype],
                                  device, stream))
    return out


def merge(x: torch.Tensor, a: torch.Tensor, wa: torch.Tensor, b: torch.Tensor, wb: torch.Tensor, add: Optional[torch.Tensor], *, n: int,
          eps: float, scale: float) -> None:
    """x += scale (RMS norm of a + RMS norm of b) + add, in place; x float32 [T, ld], norms over n columns."""
    device, stream = _on(x)
    T, ld = x.shape
    _need(x.dtype == torch.float32 and x.is_contiguous() and 0 < n <= ld, "hybrid_ops.merge: x float32, contiguous")
    for t in (a, b) if add is None else (a, b, add):
        _need(t.dtype == a.dtype and t.shape[0] == T and t.shape[1] >= ld and t.stride(1) == 1 and t.device == x.device, "hybrid_ops.merge: branches")
    for t in (wa, wb):
        _need(t.dtype == torch.float32 and t.numel() >= ld and t.is_contiguous(), "hybrid_ops.merge: weights float32 [ld]")
    _check(load().vmi_hy_merge(x.data_ptr(), a.data_ptr(), a.stride(0), b.data_ptr(), b.stride(0), _ptr(add),
                               add.stride(0) if add is not None else 0, wa.data_ptr(), wb.data_ptr(), T, n, ld, eps, scale,
                               DTYPES[a.dtype], device, stream))


def glu(x: torch.Tensor, unit: GatedUnit, out: Optional[torch.Tensor] = None) -> torch.Tensor:
    """The gated unit of interleaved (gate, up) columns: [T, 2 n] -> [T, n]."""
    device, stream = _on(x)
    T, n = x.shape[0], x.shape[1] // 2
    _need(x.dim() == 2 and x.stride(1) == 1 and x.dtype in DTYPES, "hybrid_ops.glu: rows of unit stride")
    if out is None:
        out = torch.empty((T, n), dtype=x.dtype, device=x.device)
    _need(out.shape == (T, n) and out.stride(1) == 1 and out.dtype == x.dtype, "hybrid_ops.glu: out [T, n]")
    for t in range(0, T, 65535):      # (a launch's grid holds that many rows)
        m = min(65535, T - t)
        _check(load().vmi_hy_glu(x[t:].data_ptr(), x.stride(0), out[t:].data_ptr(), out.stride(0), m, n, unit.limit, unit.alpha, unit.up,
                                 DTYPES[x.dtype], device, stream))
    return out


def concat(x: torch.Tensor, x2: torch.Tensor, dtype: torch.dtype) -> torch.Tensor:
    """(x | x2) of two float32 [T, n] tensors, in `dtype`."""
    device, stream = _on(x)
    _need(x.shape == x2.shape and x.is_contiguous() and x2.is_contiguous() and x.dtype == x2.dtype == torch.float32
          and x2.device == x.device, "hybrid_ops.concat: two contiguous float32 tensors of one shape")
    T, n = x.shape
    out = torch.empty((T, 2 * n), dtype=dtype, device=x.device)
    _check(load().vmi_hy_concat(x.data_ptr(), x2.data_ptr(), out.data_ptr(), T, n, DTYPES[dtype], device, stream))
    return out


def argmax(logits: torch.Tensor) -> torch.Tensor:
    device, stream = _on(logits)
    _need(logits.dim() == 2 and logits.dtype == torch.float32 and logits.stride(1) == 1, "hybrid_ops.argmax: float32 [B, V]")
    out = torch.empty((logits.shape[0],), dtype=torch.int64, device=logits.device)
    _check(load().vmi_hy_argmax(logits.data_ptr(), logits.stride(0), logits.shape[0], logits.shape[1], out.data_ptr(), device, stream))
    return out


ROW_TILE = 64      # rows of a tile of the recurrence's kernel


class StepLayout:
    """The tokens of a step on the device: `fields` maps the names of vmi_hy_step to int32 tensors; `single`: every portion is one
    token; `spans`: some portion crosses a row tile."""

    def __init__(self, fields: dict, T: int, B: int, page_size: int, single: bool, spans: bool, max_len: int, max_keys: int):
        for name in ("tok_seq", "tok_pos", "tok_slot"):
            _need(fields[name].dtype == torch.int32 and fields[name].numel() >= T and fields[name].is_contiguous(), f"StepLayout: {name}")
        for name in ("q_start", "q_len", "ctx", "state_slot", "flip"):
            _need(fields[name].dtype == torch.int32 and fields[name].numel() >= B and fields[name].is_contiguous(), f"StepLayout: {name}")
        tab = fields["table"]
        _need(tab.dtype == torch.int32 and tab.dim() == 2 and tab.shape[0] >= B and tab.is_contiguous(), "StepLayout: table")
        chunks = fields.get("chunks")      # [n, 2], with chunk_start [B]: steps whose portions are longer than a token, where a layer asks
        if chunks is not None:
            _need(chunks.dtype == torch.int32 and chunks.dim() == 2 and chunks.shape[1] == 2 and chunks.is_contiguous(), "StepLayout: chunks")
            _need(fields["chunk_start"].dtype == torch.int32 and fields["chunk_start"].numel() >= B, "StepLayout: chunk_start")
        self.n_chunks = 0 if chunks is None else int(chunks.shape[0])
        self.fields = fields      # (keeps the tensors alive)
        self.T, self.B, self.single, self.spans = T, B, single, spans
        self.max_len, self.max_keys = max_len, max_keys      # longest portion, most keys any token sees
        self.args = StepArgs(**{k: fields[k].data_ptr() for k in ("tok_seq", "tok_pos", "tok_slot", "q_start", "q_len", "ctx",
                                                                  "state_slot", "flip", "table")},
                             chunks=_ptr(chunks), chunk_start=_ptr(fields.get("chunk_start")), n_chunks=self.n_chunks, T=T, B=B, table_ld=tab.shape[1], page_size=page_size)
        self.ref = ctypes.byref(self.args)
        self._turns: dict = {}

    def begin(self) -> None:
        """A forward pass over this layout starts: what earlier passes derived from its positions is void (a captured pass has to
        derive it again)."""
        self._turns.clear()

    def rotations(self, freq: torch.Tensor, key) -> torch.Tensor:
        """float32 [T, n, 2]: cos and sin of position times frequency; one launch per pass for all layers that name the same key."""
        if key not in self._turns:
            device, stream = _on(freq)
            _need(freq.dtype == torch.float64 and freq.is_contiguous(), "StepLayout.rotations: float64 frequencies")
            out = torch.empty((self.T, freq.numel(), 2), dtype=torch.float32, device=freq.device)
            if freq.numel():
                _check(load().vmi_hy_rotations(freq.data_ptr(), freq.numel(), out.data_ptr(), self.ref, device, stream))
            self._turns[key] = out
        return self._turns[key]


def rglru(yx: torch.Tensor, step: StepLayout, *, conv_w: torch.Tensor, conv_b: torch.Tensor, gates: torch.Tensor, gate_b: torch.Tensor,
          decay: torch.Tensor, blocks: int, state: torch.Tensor, tail: Optional[torch.Tensor]) -> torch.Tensor:
    """yx [T, 2 width] -> [T, width]; state float32 [slots, width] and tail [slots, 2, taps - 1, width] are updated."""
    device, stream = _on(yx)
    T, width, taps = step.T, state.shape[1], conv_w.shape[0]
    bw = width // blocks
    _need(yx.shape == (T, 2 * width) and yx.is_contiguous() and width % blocks == 0 and conv_w.shape == (taps, width)
          and conv_b.numel() == width and gates.numel() == 2 * blocks * bw * bw and gates.dtype == yx.dtype and gate_b.numel() == 2 * width
          and decay.numel() == width and state.dtype == torch.float32 and state.is_contiguous(), "hybrid_ops.rglru: operand sizes")
    for t in (conv_w, conv_b, gate_b, decay):
        _need(t.dtype == torch.float32 and t.is_contiguous(), "hybrid_ops.rglru: float32 constants")
    if taps > 1:
        _need(tail is not None and tail.shape == (state.shape[0], 2, taps - 1, width) and tail.dtype == yx.dtype and tail.is_contiguous(),
              "hybrid_ops.rglru: tail [slots, 2, taps - 1, width]")
    out = torch.empty((T, width), dtype=yx.dtype, device=yx.device)
    scratch = carry = None
    if not step.single:
        scratch = torch.empty((2, T, width), dtype=torch.float32, device=yx.device)
        carry = torch.empty((-(-T // ROW_TILE), width), dtype=torch.float32, device=yx.device)
    a = RglruArgs(yx=yx.data_ptr(), out=out.data_ptr(), conv_w=conv_w.data_ptr(), conv_b=conv_b.data_ptr(), gates=gates.data_ptr(),
                  gate_b=gate_b.data_ptr(), decay=decay.data_ptr(), state=state.data_ptr(), tail=_ptr(tail) if taps > 1 else None,
                  scratch=_ptr(scratch), carry=_ptr(carry), ldx=yx.stride(0), ldo=width, width=width, blocks=blocks, taps=taps,
                  single=int(step.single), spans=int(step.spans), dtype=DTYPES[yx.dtype], device=device)
    _check(load().vmi_hy_rglru(ctypes.byref(a), step.ref, stream))
    return out


def latent_prep(proj: torch.Tensor, q: torch.Tensor, cache: torch.Tensor, step: StepLayout, *, norm_w: torch.Tensor, freq: torch.Tensor,
                heads: int, dim: int, rot: int, rank: int, rot_n: int, rank_n: int, eps: float) -> None:
    device, stream = _on(proj)
    D = rank + rot
    _need(proj.shape[0] == step.T and proj.shape[1] >= heads * (dim + rot) + D and proj.stride(1) == 1 and q.dtype == proj.dtype
          and q.shape == (step.T, heads * D) and q.is_contiguous() and cache.dtype == proj.dtype and cache.shape[-1] == D
          and cache.is_contiguous() and norm_w.numel() == rank and norm_w.dtype == torch.float32 and freq.dtype == torch.float64
          and freq.numel() == rot_n // 2, "hybrid_ops.latent_prep: operand sizes")
    a = PrepArgs(proj=proj.data_ptr(), q=q.data_ptr(), cache=cache.data_ptr(), norm_w=norm_w.data_ptr(), freq=freq.data_ptr(),
                 ldp=proj.stride(0), heads=heads, dim=dim, rot=rot, rank=rank, rot_n=rot_n, rank_n=rank_n, eps=eps,
                 dtype=DTYPES[proj.dtype], device=device)
    _check(load().vmi_hy_latent_prep(ctypes.byref(a), step.ref, stream))


def latent_row_tiles(row_dim: int, want: int, dtype: torch.dtype) -> int:
    return int(load().vmi_hy_latent_row_tiles(row_dim, want, DTYPES[dtype]))


def latent_attention(q: torch.Tensor, cache: torch.Tensor, step: StepLayout, tiles: torch.Tensor, *, heads: int, rank: int, rot: int,
                     scale: float, row_tiles: int, splits: int) -> torch.Tensor:
    """q [T, heads * (rank + rot)] -> [T, heads * rank] over the cache's pages."""
    device, stream = _on(q)
    _need(q.shape == (step.T, heads * (rank + rot)) and q.is_contiguous() and cache.dtype == q.dtype and cache.dim() == 3
          and cache.shape[1] == step.args.page_size and cache.shape[2] == rank + rot and cache.is_contiguous()
          and tiles.dtype == torch.int32 and tiles.dim() == 2 and tiles.shape[1] == 2 and tiles.is_contiguous(),
          "hybrid_ops.latent_attention: operand sizes")
    out = torch.empty((step.T, heads * rank), dtype=q.dtype, device=q.device)
    partial = torch.empty((splits, step.T * heads, rank + 2), dtype=torch.float32, device=q.device) if splits > 1 else None
    a = AttentionArgs(q=q.data_ptr(), cache=cache.data_ptr(), out=out.data_ptr(), tiles=tiles.data_ptr(), partial=_ptr(partial),
                      heads=heads, rank=rank, rot=rot, n_tiles=tiles.shape[0], row_tiles=row_tiles, splits=splits, scale=scale,
                      dtype=DTYPES[q.dtype], device=device)
    _check(load().vmi_hy_latent_attention(ctypes.byref(a), step.ref, stream))
    return out


def state_fuses(dim: int, vdim: int) -> bool:
    """Whether a step of single tokens finishes its rows (norm and output gate) by itself."""
    return bool(load().vmi_hy_state_fuses(dim, vdim))


def linear_state(proj: torch.Tensor, step: StepLayout, *, kind: int, heads: int, kv_heads: int, dim: int, vdim: int, dim_n: int,
                 vdim_n: int, state: torch.Tensor, gate: torch.Tensor, act: str, eps: float, out: torch.Tensor,
                 norm_w: Optional[torch.Tensor] = None, turns: Optional[torch.Tensor] = None, decay: Optional[torch.Tensor] = None,
                 log2_decay: Optional[torch.Tensor] = None, beta: Optional[torch.Tensor] = None, z: Optional[torch.Tensor] = None,
                 conv_w: Optional[torch.Tensor] = None, rate: Optional[torch.Tensor] = None, dt_bias: Optional[torch.Tensor] = None,
                 tail: Optional[torch.Tensor] = None) -> None:
    """Linear attention with a matrix state: proj [T, q | k | v ...] -> out [T, heads vdim], every head over its root mean square,
    times norm_w and the activated gate; state float32 [slots, heads, dim, vdim] (and tail) are updated."""
    device, stream = _on(proj)
    who, T, C, dt = "hybrid_ops.linear_state: ", step.T, 2 * kv_heads * dim + heads * vdim, proj.dtype
    _need(proj.shape[0] == T and proj.shape[1] >= C and proj.stride(1) == 1 and dt in DTYPES, who + "proj")
    _need(state.dim() == 4 and state.shape[1:] == (heads, dim, vdim) and state.dtype == torch.float32 and state.is_contiguous(), who + "state")
    _need(out.shape == (T, heads * vdim) and out.stride(1) == 1 and out.dtype == dt and gate.shape == (T, heads * vdim)
          and gate.stride(1) == 1 and gate.dtype == dt, who + "out, gate")
    _need(norm_w is None or (norm_w.dtype == torch.float32 and norm_w.numel() == vdim), who + "norm weight float32 [vdim]")
    taps = 0
    if kind == DELTA:
        taps = conv_w.shape[0]
        _need(conv_w.shape == (taps, C) and rate.numel() == heads and dt_bias.numel() == heads * dim and beta.dtype == dt
              and beta.shape == (T, heads) and beta.stride() == (proj.stride(0), 1) and z.dtype == dt and z.shape == (T, heads * dim)
              and z.stride(1) == 1, who + "gates")
        for t in (conv_w, rate, dt_bias):
            _need(t.dtype == torch.float32 and t.is_contiguous(), who + "float32 constants")
        _need(taps == 1 or (tail is not None and tail.shape == (state.shape[0], 2, taps - 1, C) and tail.dtype == dt
                            and tail.is_contiguous()), who + "tail [slots, 2, taps - 1, channels]")
    else:
        _need(turns.dtype == torch.float32 and turns.dim() == 3 and turns.shape[0] == T and 2 * turns.shape[1] <= dim
              and turns.is_contiguous() and decay.numel() == log2_decay.numel() == heads
              and decay.dtype == log2_decay.dtype == torch.float32, who + "turns, decay")
    lib, single = load(), step.single
    o = scratch = None
    if not single:
        _need(step.n_chunks > 0, who + "the step's layout has no chunks")
        scratch = torch.empty(step.n_chunks * heads * lib.vmi_hy_state_scratch(kind, dim, vdim), dtype=torch.float32, device=proj.device)
    elif not state_fuses(dim, vdim):
        o = torch.empty((T, heads * vdim), dtype=torch.float32, device=proj.device)
    a = StateArgs(proj=proj.data_ptr(), beta=_ptr(beta), z=_ptr(z), conv_w=_ptr(conv_w), rate=_ptr(rate), dt_bias=_ptr(dt_bias),
                  decay=_ptr(decay), log2_decay=_ptr(log2_decay), turns=_ptr(turns), state=state.data_ptr(),
                  tail=_ptr(tail) if taps > 1 else None, o=_ptr(o), scratch=_ptr(scratch), out=out.data_ptr(),
                  gate=gate.data_ptr(), norm_w=_ptr(norm_w), ldp=proj.stride(0), ldz=z.stride(0) if z is not None else 0,
                  ldo=out.stride(0), ldg=gate.stride(0), heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, dim_n=dim_n, vdim_n=vdim_n,
                  taps=taps, rot_n=2 * turns.shape[1] if turns is not None else 0, kind=kind, single=int(single), act=ACTS[act], eps=eps,
                  dtype=DTYPES[dt], device=device)
    _check(lib.vmi_hy_state(ctypes.byref(a), step.ref, stream))


def kv_prep(proj: torch.Tensor, q: torch.Tensor, cache: torch.Tensor, step: StepLayout, *, heads: int, kv_heads: int, dim: int, vdim: int,
            dim_n: int, eps: float) -> None:
    """proj [T, q | k | v ...]: q and k over their root mean square, q to q, k and v to the cache."""
    device, stream = _on(proj)
    _need(proj.shape[0] == step.T and proj.shape[1] >= (heads + kv_heads) * dim + kv_heads * vdim and proj.stride(1) == 1
          and q.shape == (step.T, heads * dim) and q.is_contiguous() and q.dtype == proj.dtype and cache.dtype == proj.dtype
          and cache.shape[-1] == kv_heads * (dim + vdim) and cache.is_contiguous(), "hybrid_ops.kv_prep: operand sizes")
    a = KvPrepArgs(proj=proj.data_ptr(), q=q.data_ptr(), cache=cache.data_ptr(), ldp=proj.stride(0), heads=heads, kv_heads=kv_heads,
                   dim=dim, vdim=vdim, dim_n=dim_n, eps=eps, dtype=DTYPES[proj.dtype], device=device)
    _check(load().vmi_hy_kv_prep(ctypes.byref(a), step.ref, stream))


def attention_row_tiles(dim: int, vdim: int, want: int, dtype: torch.dtype) -> int:
    return int(load().vmi_hy_attention_row_tiles(dim, vdim, want, DTYPES[dtype]))


def attention(q: torch.Tensor, cache: torch.Tensor, step: StepLayout, tiles: torch.Tensor, *, heads: int, kv_heads: int, dim: int,
              vdim: int, scale: float, row_tiles: int, splits: int, out: torch.Tensor, chunk: int = 0, bias: Optional[torch.Tensor] = None,
              sink: Optional[torch.Tensor] = None, gate: Optional[torch.Tensor] = None) -> None:
    """q [T, heads dim] -> out [T, heads vdim] over the cache's pages; bias [heads, distances] and sink [heads] times log2(e)."""
    device, stream = _on(q)
    who = "hybrid_ops.attention: "
    _need(q.shape == (step.T, heads * dim) and q.is_contiguous() and cache.dtype == q.dtype and cache.dim() == 3
          and cache.shape[1] == step.args.page_size and cache.shape[2] == kv_heads * (dim + vdim) and cache.is_contiguous()
          and tiles.dtype == torch.int32 and tiles.dim() == 2 and tiles.shape[1] == 2 and tiles.is_contiguous()
          and out.shape == (step.T, heads * vdim) and out.stride(1) == 1 and out.dtype == q.dtype, who + "operand sizes")
    _need(bias is None or (bias.dtype == torch.float32 and bias.dim() == 2 and bias.shape[0] == heads and bias.is_contiguous()), who + "bias")
    _need(sink is None or (sink.dtype == torch.float32 and sink.numel() == heads), who + "sink")
    _need(gate is None or (gate.dtype == q.dtype and gate.shape == (step.T, heads) and gate.stride(1) == 1), who + "gate")
    partial = torch.empty((splits, step.T * heads, vdim + 2), dtype=torch.float32, device=q.device) if splits > 1 else None
    a = GqaArgs(q=q.data_ptr(), cache=cache.data_ptr(), out=out.data_ptr(), bias=_ptr(bias), sink=_ptr(sink), gate=_ptr(gate),
                tiles=tiles.data_ptr(), partial=_ptr(partial), ldo=out.stride(0), ldg=gate.stride(0) if gate is not None else 0,
                heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, bias_n=bias.shape[1] if bias is not None else 0, chunk=chunk,
                n_tiles=tiles.shape[0], row_tiles=row_tiles, splits=splits, scale=scale, dtype=DTYPES[q.dtype], device=device)
    _check(load().vmi_hy_attention(ctypes.byref(a), step.ref, stream))
