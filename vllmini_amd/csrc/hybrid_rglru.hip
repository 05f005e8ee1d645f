// The recurrent block between its projections (include/vmi_hybrid.h): causal convolution -> block-diagonal gates -> gated linear
// recurrence -> product with gelu(y).
//
// The packed tokens are cut into row tiles of BM consecutive rows, whatever entries they belong to.  A workgroup takes one row
// tile x up to 64 channels of one gate block: the convolution of the block's channels goes to LDS (element type), both gate
// matrices run on the matrix cores (A = gate rows = channels, B = u rows = tokens, fp32 accumulation), and everything behind the
// product is fp32: r, i, log a = decay * r, a, b = sqrt(1 - a^2) * i * u.  A token that opens an entry's portion folds the state
// of its slot in at once (b += a * S, a = 0), so one uniform walk S = a S + b, P = a P over the tile serves any mix of entries:
// P is zero from an opening token on and the product of the decays in front of one — only the rows of a tile's LEADING segment
// (a portion that began in an earlier tile) are unfinished, by P * (the carry into the tile).  Batches whose portions all fit
// their tiles — every decode step — are one launch; otherwise a second kernel runs the carries from tile to tile and a third
// finishes the leading rows.
//
// The convolution's tail (the last taps - 1 inputs of a sequence) has two halves: a step reads half `flip` and writes the other
// one, so no workgroup can overwrite what another still reads.
#include "hybrid_common.hpp"

namespace vmi_hybrid {

constexpr int CT = 64;      // channels of a workgroup
constexpr int KCH = 256;    // channels of u in LDS at a time
constexpr int MAX_TAPS = 16;

struct RowMeta {
  int seq, qs, len, ctx, slot, flip, first, last;
};

template <typename T, int BM>
struct Lds {
  static constexpr int LDU = KCH + 16 / (int)sizeof(T), LDA = CT + 4;
  T u[BM * LDU];
  float a[BM * LDA];
  float b[BM * LDA];
  float end[2][4][CT];
  RowMeta meta[BM];
};

// convolution of 8 channels for the token of row m.  TAPS = 0: any number of taps; else exactly that many, every load issued
// without a condition around it (taps before the start read a valid row and count zero), so that all of them are in flight
template <typename T, int TAPS>
__device__ __forceinline__ f32x8 conv8(const vmi_hy_rglru_args& p, const RowMeta& r, int t, int c) {
  f32x8 acc = load8(p.conv_b + c);
  const T* in = static_cast<const T*>(p.yx) + p.width + c;
  const int taps = TAPS ? TAPS : p.taps, pos = r.ctx + t - r.qs;
  // tail entries: positions ctx - (taps - 1) .. ctx - 1
  const T* tail = static_cast<const T*>(p.tail) + ((int64_t)r.slot * 2 + r.flip) * (taps - 1) * p.width + c;
  auto tap = [&](int j) {
    const int back = taps - 1 - j;
    const T* src = t - back >= r.qs ? in + (int64_t)(t - back) * p.ldx
                   : pos >= back    ? tail + (int64_t)(pos - back - (r.ctx - (taps - 1))) * p.width
                                    : in + (int64_t)t * p.ldx;
    const V8<T> v = load8(src);
    const f32x8 w = load8(p.conv_w + (int64_t)j * p.width + c);
    const bool on = pos >= back;
#pragma unroll
    for (int e = 0; e < 8; ++e) acc[e] = fmaf(w[e], on ? (float)v[e] : 0.f, acc[e]);
  };
  if constexpr (TAPS > 0) {
#pragma unroll
    for (int j = 0; j < TAPS; ++j) tap(j);
  } else {
    for (int j = 0; j < taps; ++j) tap(j);
  }
  return acc;
}

template <typename T>
__device__ __forceinline__ void store_out8(const vmi_hy_rglru_args& p, int t, int c, const f32x8& s, const f32x8& y) {
  f32x8 o;
#pragma unroll
  for (int e = 0; e < 8; ++e) o[e] = s[e] * gelu_tanh(y[e]);
  *reinterpret_cast<V8<T>*>(static_cast<T*>(p.out) + (int64_t)t * p.ldo + c) = from_f32<T>(o);
}

template <typename T, int BM, int TAPS>
__global__ __launch_bounds__(256, 2) void rglru_tile_kernel(const vmi_hy_rglru_args p, const vmi_hy_step s) {
  constexpr int MT = BM / 16;
  extern __shared__ __attribute__((aligned(16))) unsigned char smem[];
  auto& L = *reinterpret_cast<Lds<T, BM>*>(smem);
  constexpr int LDU = Lds<T, BM>::LDU, LDA = Lds<T, BM>::LDA;
  const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6), kc = lane >> 4, r16 = lane & 15;
  const int bw = p.width / p.blocks, per = (bw + CT - 1) / CT;
  const int blk = blockIdx.x / per, cin = (blockIdx.x % per) * CT;   // gate block, first channel inside it
  const int t0 = blockIdx.y * BM, rows = min(BM, s.T - t0);
  const int nch = min(CT, bw - cin), c0 = blk * bw + cin;            // channels of this workgroup (a multiple of 32)

  if (tid < BM) {
    RowMeta r{-1, 0, 0, 0, 0, 0, 0, 0};
    if (tid < rows) r.seq = s.tok_seq[t0 + tid];
    if (r.seq >= 0) {
      r.qs = s.q_start[r.seq];
      r.len = s.q_len[r.seq];
      r.ctx = s.ctx[r.seq];
      r.slot = s.state_slot[r.seq];
      r.flip = s.flip[r.seq];
      r.first = t0 + tid == r.qs;
      r.last = t0 + tid == r.qs + r.len - 1;
    }
    L.meta[tid] = r;
  }

  // gate products over the block's channels, KCH of them in LDS at a time
  f32x4 ar[MT], ai[MT];
#pragma unroll
  for (int mi = 0; mi < MT; ++mi) ar[mi] = ai[mi] = f32x4{0.f, 0.f, 0.f, 0.f};
  const bool wvalid = wave * 16 < nch;
  const int64_t gsz = (int64_t)bw * bw, nks = bw >> 5;
  const T* wr = static_cast<const T*>(p.gates) + blk * gsz + ((int64_t)((cin >> 4) + wave) * nks * 64 + lane) * 8;
  const T* wi = wr + p.blocks * gsz;
  // requested now, used behind the products
  const int cl = wave * 16 + 4 * kc;
  f32x4 br, bi, dec, S0[MT];
  if (wvalid) {
    br = *reinterpret_cast<const f32x4*>(p.gate_b + c0 + cl);
    bi = *reinterpret_cast<const f32x4*>(p.gate_b + p.width + c0 + cl);
    dec = *reinterpret_cast<const f32x4*>(p.decay + c0 + cl);
  }
  __syncthreads();   // meta is there
#pragma unroll
  for (int mi = 0; mi < MT; ++mi) {
    const RowMeta& r = L.meta[mi * 16 + r16];
    S0[mi] = f32x4{0.f, 0.f, 0.f, 0.f};
    if (wvalid && r.seq >= 0 && r.first && r.ctx > 0) S0[mi] = *reinterpret_cast<const f32x4*>(p.state + (int64_t)r.slot * p.width + c0 + cl);
  }
  constexpr int YU = (BM * (CT / 8) + 255) / 256;   // this thread's units of the output: y
  V8<T> yv[YU];
#pragma unroll
  for (int i = 0; i < YU; ++i) {
    const int m = (tid + i * 256) / (CT / 8), k = ((tid + i * 256) % (CT / 8)) * 8;
    yv[i] = load8(static_cast<const T*>(p.yx) + (int64_t)(t0 + min(m, rows - 1)) * p.ldx + c0 + min(k, nch - 8));
  }
  for (int k0 = 0; k0 < bw; k0 += KCH) {
    const int kn = min(KCH, bw - k0);
    // few rows: the chunk's gate tiles are in flight while u is computed (many rows: those registers are worth a second workgroup)
    constexpr bool AHEAD = BM == 16;
    V8<T> fr[AHEAD ? KCH / 32 : 1], fi[AHEAD ? KCH / 32 : 1];
    if constexpr (AHEAD) {
#pragma unroll
      for (int k = 0; k < KCH / 32; ++k) {
        const int64_t at = (int64_t)((k0 >> 5) + min(k, (kn >> 5) - 1)) * 512;
        if (wvalid) fr[k] = load8(wr + at), fi[k] = load8(wi + at);
      }
    }
    if (k0 > 0) __syncthreads();   // the previous chunk has been read
    auto conv_row = [&](int m, int k) {
      const RowMeta& r = L.meta[m];
      if (r.seq >= 0 && k < kn) *reinterpret_cast<V8<T>*>(L.u + m * LDU + k) = from_f32<T>(conv8<T, TAPS>(p, r, t0 + m, blk * bw + k0 + k));
      else if (k < kn) *reinterpret_cast<V8<T>*>(L.u + m * LDU + k) = zero8<T>();
    };
    if constexpr (BM == 64 && TAPS > 0) {
      // eight channels of eight consecutive rows: inside one portion, past its first taps, the rows share their inputs
      const int k = (tid % (KCH / 8)) * 8, m0 = (tid / (KCH / 8)) * 8;
      const RowMeta &ra = L.meta[m0], &rb = L.meta[m0 + 7];
      if (k < kn && ra.seq >= 0 && ra.seq == rb.seq && t0 + m0 - (TAPS - 1) >= ra.qs) {
        const int c = blk * bw + k0 + k;
        const T* in = static_cast<const T*>(p.yx) + (int64_t)(t0 + m0 - (TAPS - 1)) * p.ldx + p.width + c;
        V8<T> v[TAPS + 7];
        f32x8 w[TAPS];
#pragma unroll
        for (int j = 0; j < TAPS + 7; ++j) v[j] = load8(in + (int64_t)j * p.ldx);
#pragma unroll
        for (int j = 0; j < TAPS; ++j) w[j] = load8(p.conv_w + (int64_t)j * p.width + c);
        const f32x8 b = load8(p.conv_b + c);
#pragma unroll
        for (int m = 0; m < 8; ++m) {
          f32x8 acc = b;
#pragma unroll
          for (int j = 0; j < TAPS; ++j)
#pragma unroll
            for (int e = 0; e < 8; ++e) acc[e] = fmaf(w[j][e], (float)v[m + j][e], acc[e]);
          *reinterpret_cast<V8<T>*>(L.u + (m0 + m) * LDU + k) = from_f32<T>(acc);
        }
      } else {
#pragma unroll 1
        for (int m = 0; m < 8; ++m) conv_row(m0 + m, k);
      }
    } else {
#pragma unroll 2
      for (int u = tid; u < BM * (KCH / 8); u += 256) conv_row(u / (KCH / 8), (u % (KCH / 8)) * 8);
    }
    __syncthreads();
    if (wvalid) {
      auto product = [&](int k, const V8<T>& a, const V8<T>& b) {
#pragma unroll
        for (int mi = 0; mi < MT; ++mi) {
          const V8<T> fu = load8(L.u + (mi * 16 + r16) * LDU + k * 32 + 8 * kc);
          mma(ar[mi], a, fu);
          mma(ai[mi], b, fu);
        }
      };
      if constexpr (AHEAD) {
#pragma unroll
        for (int k = 0; k < KCH / 32; ++k)
          if (k < kn >> 5) product(k, fr[k], fi[k]);
      } else {
#pragma unroll 2
        for (int k = 0; k < kn >> 5; ++k)
          product(k, load8(wr + (int64_t)((k0 >> 5) + k) * 512), load8(wi + (int64_t)((k0 >> 5) + k) * 512));
      }
    }
  }
  // the workgroup's own channels of u: into b, from LDS or (a block of several chunks) computed again
  const bool held = bw <= KCH;
  if (held) __syncthreads();
  for (int u = tid; u < BM * (CT / 8); u += 256) {
    const int m = u / (CT / 8), k = (u % (CT / 8)) * 8;
    const RowMeta& r = L.meta[m];
    f32x8 v;
#pragma unroll
    for (int e = 0; e < 8; ++e) v[e] = 0.f;
    if (held && k < nch) v = to_f32<T>(load8(L.u + m * LDU + cin + k));
    else if (r.seq >= 0 && k < nch) v = to_f32<T>(from_f32<T>(conv8<T, TAPS>(p, r, t0 + m, c0 + k)));   // rounded as the gates saw it
    *reinterpret_cast<f32x8*>(L.b + m * LDA + k) = v;
  }
  __syncthreads();
  if (wvalid) {
#pragma unroll
    for (int mi = 0; mi < MT; ++mi) {
      const int m = mi * 16 + r16;
      const RowMeta& r = L.meta[m];
      const f32x4 u = *reinterpret_cast<const f32x4*>(L.b + m * LDA + cl);
      f32x4 a, b;
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        const float la = dec[e] * sigmoid(ar[mi][e] + br[e]);
        a[e] = exp_hw(la);
        b[e] = __builtin_amdgcn_sqrtf(one_minus_exp(-2.f * la, a[e] * a[e])) * sigmoid(ai[mi][e] + bi[e]) * u[e];
        if (r.seq < 0) a[e] = 1.f, b[e] = 0.f;
        if (r.first) {
          b[e] = fmaf(a[e], S0[mi][e], b[e]);
          a[e] = 0.f;
        }
      }
      *reinterpret_cast<f32x4*>(L.a + m * LDA + cl) = a;
      *reinterpret_cast<f32x4*>(L.b + m * LDA + cl) = b;
    }
  }
  __syncthreads();
  const bool lead0 = L.meta[0].seq >= 0 && !L.meta[0].first;   // the tile opens inside a portion
  if (!p.single) {   // the walk, in place (b becomes S, a becomes P): a wave takes a quarter of the rows, a lane a channel
    constexpr int RW = BM / 4;
    float* pa = L.a + wave * RW * LDA + lane;
    float* pb = L.b + wave * RW * LDA + lane;
    if (lane < nch) {
      float S = 0.f, P = wave == 0 ? (lead0 ? 1.f : 0.f) : 1.f;
#pragma unroll 8
      for (int m = 0; m < RW; ++m) {
        const float a = pa[m * LDA], b = pb[m * LDA];
        S = fmaf(a, S, b);
        P *= a;
        pb[m * LDA] = S;
        pa[m * LDA] = P;
      }
      L.end[0][wave][lane] = S;
      L.end[1][wave][lane] = P;
    }
    __syncthreads();
    if (lane < nch && wave > 0) {   // what the quarters before this one hand over
      float S = L.end[0][0][lane], P = L.end[1][0][lane];
      for (int w = 1; w < wave; ++w) {
        S = fmaf(L.end[1][w][lane], S, L.end[0][w][lane]);
        P *= L.end[1][w][lane];
      }
#pragma unroll 8
      for (int m = 0; m < RW; ++m) {
        pb[m * LDA] = fmaf(pa[m * LDA], S, pb[m * LDA]);
        pa[m * LDA] *= P;
      }
    }
  }
  __syncthreads();
  const int lead_end = lead0 ? min(rows, L.meta[0].qs + L.meta[0].len - t0) : 0;   // rows of the leading segment
#pragma unroll
  for (int i = 0; i < YU; ++i) {
    const int u = tid + i * 256, m = u / (CT / 8), k = (u % (CT / 8)) * 8;
    if (m >= rows || k >= nch) continue;
    const RowMeta& r = L.meta[m];
    const f32x8 S = *reinterpret_cast<const f32x8*>(L.b + m * LDA + k);
    const int t = t0 + m, c = c0 + k;
    if (r.seq < 0) {
      *reinterpret_cast<V8<T>*>(static_cast<T*>(p.out) + (int64_t)t * p.ldo + c) = zero8<T>();
      continue;
    }
    const bool lead = m < lead_end;
    if (lead || (m == BM - 1 && !r.last)) {   // unfinished, or what the next tile's carry starts from
      *reinterpret_cast<f32x8*>(p.scratch + (int64_t)t * p.width + c) = S;
      *reinterpret_cast<f32x8*>(p.scratch + ((int64_t)s.T + t) * p.width + c) = *reinterpret_cast<const f32x8*>(L.a + m * LDA + k);
    }
    if (lead) continue;
    store_out8<T>(p, t, c, S, to_f32<T>(yv[i]));
    if (r.last) *reinterpret_cast<f32x8*>(p.state + (int64_t)r.slot * p.width + c) = S;
  }
  // the convolution tail of entries that end in this tile, into its other half
  const int nt = p.taps - 1;
  for (int u = tid; u < rows * nt * (CT / 8); u += 256) {
    const int k = (u % (CT / 8)) * 8, e = u / (CT / 8) % nt, m = u / (CT / 8) / nt, c = c0 + k;
    const RowMeta& r = L.meta[m];
    if (k >= nch || r.seq < 0 || !r.last) continue;
    const T* from = static_cast<const T*>(p.tail) + ((int64_t)r.slot * 2 + r.flip) * nt * p.width;
    T* to = static_cast<T*>(p.tail) + ((int64_t)r.slot * 2 + (r.flip ^ 1)) * nt * p.width;
    const int pos = r.ctx + r.len - nt + e;   // the position this entry stands for
    V8<T> v = zero8<T>();
    if (pos >= r.ctx) v = load8(static_cast<const T*>(p.yx) + (int64_t)(r.qs + pos - r.ctx) * p.ldx + p.width + c);
    else if (pos >= 0) v = load8(from + (int64_t)(pos - (r.ctx - nt)) * p.width + c);
    *reinterpret_cast<V8<T>*>(to + (int64_t)e * p.width + c) = v;
  }
}

// carries from tile to tile of the entries that span tiles: one thread per (entry, channel)
__global__ __launch_bounds__(64) void rglru_carry_kernel(const vmi_hy_rglru_args p, const vmi_hy_step s) {
  constexpr int BM = 64;
  const int c = blockIdx.x * 64 + threadIdx.x, q = blockIdx.y;
  if (c >= p.width || s.q_len[q] <= 0) return;
  const int qs = s.q_start[q], qe = qs + s.q_len[q];
  const int first = qs / BM, last = (qe - 1) / BM;
  if (first == last) return;
  const float* S = p.scratch + c;
  const float* P = p.scratch + (int64_t)s.T * p.width + c;
  float carry = S[(int64_t)(first * BM + BM - 1) * p.width];
  constexpr int U = 8;
  for (int k = first + 1; k <= last; k += U) {
    float sv[U], pv[U];
#pragma unroll
    for (int i = 0; i < U; ++i) {
      const int64_t row = min((k + i) * BM + BM, qe) - 1;
      sv[i] = k + i <= last ? S[row * p.width] : 0.f;
      pv[i] = k + i <= last ? P[row * p.width] : 0.f;
    }
#pragma unroll
    for (int i = 0; i < U; ++i) {
      if (k + i <= last) {
        p.carry[(int64_t)(k + i) * p.width + c] = carry;
        carry = fmaf(pv[i], carry, sv[i]);
      }
    }
  }
  p.state[(int64_t)s.state_slot[q] * p.width + c] = carry;
}

// the rows of leading segments: S + P * carry
template <typename T>
__global__ __launch_bounds__(256) void rglru_finish_kernel(const vmi_hy_rglru_args p, const vmi_hy_step s) {
  constexpr int BM = 64;
  const int t = blockIdx.y, c = (blockIdx.x * 256 + threadIdx.x) * 8;
  const int q = s.tok_seq[t];
  if (c >= p.width || q < 0) return;
  const int tile = t / BM;
  if (s.q_start[q] >= tile * BM) return;
  const f32x8 S = load8(p.scratch + (int64_t)t * p.width + c), P = load8(p.scratch + ((int64_t)s.T + t) * p.width + c);
  const f32x8 k = load8(p.carry + (int64_t)tile * p.width + c);
  f32x8 o;
#pragma unroll
  for (int e = 0; e < 8; ++e) o[e] = fmaf(P[e], k[e], S[e]);
  store_out8<T>(p, t, c, o, to_f32<T>(load8(static_cast<const T*>(p.yx) + (int64_t)t * p.ldx + c)));
}

template <typename T, int BM, int TAPS>
static int launch_tile(const vmi_hy_rglru_args& p, const vmi_hy_step& s, hipStream_t st) {
  auto* fn = rglru_tile_kernel<T, BM, TAPS>;
  if (int rc = allow_lds(fn, sizeof(Lds<T, BM>), "vmi_hy_rglru")) return rc;
  const int bw = p.width / p.blocks;
  hipLaunchKernelGGL(fn, dim3(p.blocks * ((bw + CT - 1) / CT), (s.T + BM - 1) / BM), dim3(256), sizeof(Lds<T, BM>), st, p, s);
  return launched("vmi_hy_rglru");
}

template <typename T>
static int run_rglru(const vmi_hy_rglru_args& p, const vmi_hy_step& s, hipStream_t st) {
  if (p.single) return p.taps == 4 ? launch_tile<T, 16, 4>(p, s, st) : launch_tile<T, 16, 0>(p, s, st);
  if (int rc = p.taps == 4 ? launch_tile<T, 64, 4>(p, s, st) : launch_tile<T, 64, 0>(p, s, st)) return rc;
  if (!p.spans) return VMI_HY_OK;
  hipLaunchKernelGGL(rglru_carry_kernel, dim3((p.width + 63) / 64, s.B), dim3(64), 0, st, p, s);
  hipLaunchKernelGGL(rglru_finish_kernel<T>, dim3((p.width / 8 + 255) / 256, s.T), dim3(256), 0, st, p, s);
  return launched("vmi_hy_rglru");
}

}  // namespace vmi_hybrid

using namespace vmi_hybrid;

extern "C" int vmi_hy_rglru(const vmi_hy_rglru_args* a, const vmi_hy_step* s, void* stream) {
  static const char* who = "vmi_hy_rglru";
  if (!a || !s || !a->yx || !a->out || !a->conv_w || !a->conv_b || !a->gates || !a->gate_b || !a->decay || !a->state ||
      (a->taps > 1 && !a->tail) || !s->tok_seq || !s->q_start || !s->q_len || !s->ctx || !s->state_slot || !s->flip || s->T <= 0 ||
      s->B <= 0 || a->width <= 0 || a->blocks <= 0 || a->taps < 1 || (a->spans && (!a->scratch || !a->carry)))
    return fail(VMI_HY_E_ARG, who, "null pointer or non-positive size");
  if (a->width % a->blocks || ((a->width / a->blocks) & 31) || (a->ldx & 7) || (a->ldo & 7) || a->taps > MAX_TAPS || s->T > 65535 * 16 ||
      (a->spans && s->T > 65535))
    return fail(VMI_HY_E_SHAPE, who, "needs blocks of a multiple of 32 channels, rows of a multiple of 8 elements, at most 16 taps");
  if (!a->single && !a->spans && !a->scratch) return fail(VMI_HY_E_ARG, who, "portions need scratch");
  DeviceScope dev(a->device);
  if (!dev.ok) return fail(VMI_HY_E_HIP, who, "hipSetDevice failed");
  hipStream_t st = static_cast<hipStream_t>(stream);
  return a->dtype == VMI_HY_BF16 ? run_rglru<b16>(*a, *s, st) : run_rglru<float>(*a, *s, st);
}
