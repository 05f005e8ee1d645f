// Grouped-query softmax attention over a paged cache (include/vmi_hybrid.h): chunked masks, a bias by distance, a sink in the
// denominator, an output gate per head.  A cache row holds [key | value] of every key head side by side.
//
// Query rows are (token, head of the group) pairs of one key head, so a key tile read from the pages serves the whole group; a
// workgroup walks the keys its rows can see in tiles: from the first row's chunk start to the last row's token.  A tile comes into
// LDS once, requested one tile ahead and held in registers meanwhile, with the biases of the distances that occur in it; the value
// operand is read column-wise from the same LDS rows.  Scores, softmax and sums are fp32; the sink opens the running maximum and sum.
//   gqa_kernel       16 rows (steps of few tokens): wave w scores the 16 keys 16 w .., statistics meet in LDS, then wave w adds the
//                    value columns w, w + 4, ... (tiles of 16)
//   gqa_rows_kernel  64 rows (portions of prompts, bfloat16): every wave owns 16 of them, so only the key tile is shared
// Tiles too few for the chip have their keys dealt to `splits` workgroups.
#include "hybrid_softmax.hpp"

namespace vmi_hybrid {

// distances that the rows of a tile (R of them, rep to a token) can have to the keys of one tile
__host__ __device__ inline int bias_window(int KT, int R, int rep) { return KT + (R + rep - 1) / rep; }

template <typename T, int KT>
inline size_t gqa_lds(int dim, int vdim, int rep, bool bias) {
  constexpr int PAD = pad_of<T>();
  return ((size_t)KT * (dim + vdim + PAD) + (size_t)16 * (dim + PAD) + (size_t)16 * (KT + PAD)) * sizeof(T) + (size_t)4 * 16 * 4 +
         (bias ? (size_t)rep * bias_window(KT, 16, rep) * 4 : 0);
}

// What a workgroup needs to know about its query tile and keys, the same in both kernels
struct QueryTile {
  int e, r0, split, g, rep, ctx, nrows, tok0, h0, first, kv_end, kt0, kt1;
  __device__ __forceinline__ QueryTile(const vmi_hy_attention_args& p, const vmi_hy_step& s, int R, int KT)
      : e(p.tiles[2 * blockIdx.x]), r0(p.tiles[2 * blockIdx.x + 1]), split(blockIdx.y), g(blockIdx.z), rep(p.heads / p.kv_heads), nrows(0) {
    if (e < 0) return;
    ctx = s.ctx[e];
    nrows = min(R, s.q_len[e] * rep - r0);
    tok0 = s.q_start[e];
    h0 = g * rep;
    first = ctx + r0 / rep;   // position of the first row
    const int kv_begin = p.chunk > 0 ? first / p.chunk * p.chunk : 0;
    kv_end = ctx + (r0 + max(nrows, 1) - 1) / rep + 1;
    const int tb = kv_begin / KT, nkt = (kv_end + KT - 1) / KT - tb, tps = (nkt + p.splits - 1) / p.splits;
    kt0 = tb + split * tps;
    kt1 = min(tb + nkt, kt0 + tps);
  }
  // row m: token tok0 + (r0 + m) / rep, head h0 + (r0 + m) % rep; partial results lie by (token, head)
  __device__ __forceinline__ float* part(const vmi_hy_attention_args& p, const vmi_hy_step& s, int m) const {
    return p.partial + (((int64_t)split * s.T + tok0 + (r0 + m) / rep) * p.heads + h0 + (r0 + m) % rep) * (p.vdim + 2);
  }
  // a split without keys (split 0 always has some): its parts weigh nothing
  __device__ __forceinline__ bool empty(const vmi_hy_attention_args& p, const vmi_hy_step& s, int tid) const {
    if (kt0 < kt1) return false;
    if (tid < nrows) {
      float* o = part(p, s, tid);
      o[p.vdim] = -1e30f;
      o[p.vdim + 1] = 0.f;
    }
    return true;
  }
};

// The keys of a tile on their way from the pages to LDS, and the biases of its distances.  The page of a tile is known one tile
// before it is requested, keys past the end repeat the last one and columns past the row its last ones: no lane-wise condition stands
// around a load.  KT keys, U 8-element units of a row per thread.
template <typename T, int KT, int U>
struct KeyTile {
  static constexpr int TPK = 256 / KT, BU = 2;
  const T* cache;
  const int* tab;
  const float* bg;
  int64_t ldc;
  int D, kj, kcol, page_size, kv_end, next_page, BW, bn, first, bias_n;
  V8<T> kr[U];
  float br[BU];
  __device__ __forceinline__ int key_of(int kt) const { return min(kt * KT + kj, kv_end - 1); }
  __device__ __forceinline__ float bias_at(int kt, int u) const {   // entry (hh, w): head hh, distance first - (last key of the tile) + w
    const int hh = u / BW, w = u - hh * BW;
    return bg[(int64_t)hh * bias_n + min(max(first - (kt * KT + KT - 1) + w, 0), bias_n - 1)];
  }
  __device__ __forceinline__ void load(int page, int kt) {
    const T* src = cache + ((int64_t)page * page_size + key_of(kt) % page_size) * ldc;
    if (bn) {
#pragma unroll
      for (int i = 0; i < BU; ++i) br[i] = bias_at(kt, min((int)threadIdx.x + 256 * i, bn - 1));
    }
#pragma unroll
    for (int i = 0; i < U; ++i) kr[i] = load8(src + min(kcol + i * TPK * 8, D - 8));
  }
  __device__ __forceinline__ void open(const vmi_hy_attention_args& p, const vmi_hy_step& s, const QueryTile& q, int R) {
    D = p.dim + p.vdim;
    cache = static_cast<const T*>(p.cache) + (int64_t)q.g * D;
    ldc = (int64_t)p.kv_heads * D;
    tab = s.table + (int64_t)q.e * s.table_ld;
    kj = threadIdx.x / TPK;
    kcol = (threadIdx.x % TPK) * 8;
    page_size = s.page_size;
    kv_end = q.kv_end;
    first = q.first;
    bias_n = p.bias_n;
    BW = bias_window(KT, R, q.rep);
    bn = p.bias ? q.rep * BW : 0;
    bg = p.bias + (int64_t)q.h0 * p.bias_n;
    load(tab[key_of(q.kt0) / page_size], q.kt0);
    next_page = tab[key_of(min(q.kt0 + 1, q.kt1 - 1)) / page_size];
  }
  // tile kt into LDS; the one behind it is requested
  __device__ __forceinline__ void step(T* ks, float* bl, int ldk, int kt, int kt1) {
#pragma unroll
    for (int i = 0; i < U; ++i)   // (a clamped column is written again with the same values)
      *reinterpret_cast<V8<T>*>(ks + kj * ldk + min(kcol + i * TPK * 8, D - 8)) = kr[i];
    if (bn) {
#pragma unroll
      for (int i = 0; i < BU; ++i) bl[min((int)threadIdx.x + 256 * i, bn - 1)] = br[i];
      for (int u = threadIdx.x + 256 * BU; u < bn; u += 256) bl[u] = bias_at(kt, u);
    }
    if (kt + 1 < kt1) {
      load(next_page, kt + 1);
      next_page = tab[key_of(min(kt + 2, kt1 - 1)) / page_size];
    }
  }
};

// NT value tiles (of 16 columns) per wave
template <typename T, int KT, int NT, int U>
__global__ __launch_bounds__(256) void gqa_kernel(const vmi_hy_attention_args p, const vmi_hy_step s) {
  constexpr int R = 16, PAD = pad_of<T>(), LDP = KT + PAD, SW = KT / 16;   // SW waves score
  extern __shared__ __attribute__((aligned(16))) unsigned char smem[];
  const int dim = p.dim, vdim = p.vdim, LDK = dim + vdim + PAD, LDQ = dim + PAD;
  T* ks = reinterpret_cast<T*>(smem);              // [KT][LDK]
  T* qs = ks + (size_t)KT * LDK;                   // [R][LDQ]
  T* ps = qs + (size_t)R * LDQ;                    // [R][LDP]
  float* sx = reinterpret_cast<float*>(ps + (size_t)R * LDP);   // [4][R]
  float* bl = sx + 4 * R;                          // [rep][window]: the bias of the distances that occur in a tile
  const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6), kc = lane >> 4, r16 = lane & 15;
  const QueryTile q(p, s, R, KT);
  if (q.nrows <= 0 || q.empty(p, s, tid)) return;
  KeyTile<T, KT, U> keys;
  keys.open(p, s, q, R);
  for (int u = tid; u < R * (dim >> 3); u += 256) {
    const int m = u / (dim >> 3), k = (u - m * (dim >> 3)) * 8, row = q.r0 + min(m, q.nrows - 1);
    *reinterpret_cast<V8<T>*>(qs + m * LDQ + k) =
        load8(static_cast<const T*>(p.q) + ((int64_t)(q.tok0 + row / q.rep) * p.heads + q.h0 + row % q.rep) * dim + k);
  }
  f32x4 o[NT];
  float mrun[4], lrun[4];
  int lim[4], low[4], boff[4];   // last and first key row m sees, its place in the bias window
#pragma unroll
  for (int nt = 0; nt < NT; ++nt) o[nt] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
  for (int r = 0; r < 4; ++r) {
    const int row = q.r0 + min(4 * kc + r, q.nrows - 1), hh = row % q.rep;
    mrun[r] = -1e30f;
    lrun[r] = 0.f;
    if (p.sink && q.split == 0) {   // counted once: by one lane of the first split
      mrun[r] = p.sink[q.h0 + hh];
      lrun[r] = wave == 0 && r16 == 0 ? 1.f : 0.f;
    }
    lim[r] = q.ctx + row / q.rep;
    low[r] = p.chunk > 0 ? lim[r] / p.chunk * p.chunk : 0;
    boff[r] = hh * keys.BW + lim[r] - q.first + KT - 1 - (wave * 16 + r16);
  }
  const float sc2 = p.scale * 1.4426950408889634f;   // scores in units of log 2
  const int n16 = vdim >> 4;

  for (int kt = q.kt0; kt < q.kt1; ++kt) {
    keys.step(ks, bl, LDK, kt, q.kt1);
    __syncthreads();
    f32x4 sc = f32x4{0.f, 0.f, 0.f, 0.f};
    if (SW == 4 || wave < SW) {
      const T* krow = ks + (wave * 16 + r16) * LDK + 8 * kc;
      const T* qrow = qs + r16 * LDQ + 8 * kc;
      f32x4 odd = f32x4{0.f, 0.f, 0.f, 0.f};   // (two chains of sums)
      int k = 0;
      for (; k + 64 <= dim; k += 64) {
        mma(sc, load8(qrow + k), load8(krow + k));
        mma(odd, load8(qrow + k + 32), load8(krow + k + 32));
      }
      if (k < dim) mma(sc, load8(qrow + k), load8(krow + k));
      sc += odd;
      const int key = kt * KT + wave * 16 + r16;
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const float b = keys.bn ? bl[boff[r]] : 0.f;
        sc[r] = key <= lim[r] && key >= low[r] ? fmaf(sc[r], sc2, b) : -INFINITY;
        const float v = max16(sc[r]);
        if (r16 == 0) sx[wave * R + 4 * kc + r] = v;
      }
    }
    __syncthreads();
    float alpha[4];
    f32x4 mx = *reinterpret_cast<const f32x4*>(sx + 4 * kc);
#pragma unroll
    for (int w = 1; w < SW; ++w) {
      const f32x4 v = *reinterpret_cast<const f32x4*>(sx + w * R + 4 * kc);
#pragma unroll
      for (int r = 0; r < 4; ++r) mx[r] = fmaxf(mx[r], v[r]);
    }
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const float mn = fmaxf(mrun[r], mx[r]);
      alpha[r] = exp2_hw(mrun[r] - mn);
      mrun[r] = mn;
      lrun[r] *= alpha[r];
      if (SW == 4 || wave < SW) {
        const T pr = (T)exp2_hw(sc[r] - mn);
        lrun[r] += (float)pr;   // (what is summed is what multiplies the values)
        ps[(4 * kc + r) * LDP + wave * 16 + r16] = pr;
      }
    }
#pragma unroll
    for (int nt = 0; nt < NT; ++nt)
#pragma unroll
      for (int r = 0; r < 4; ++r) o[nt][r] *= alpha[r];
    __syncthreads();
#pragma unroll
    for (int k = 0; k < KT; k += 32) {
      const V8<T> pf = load8(ps + r16 * LDP + k + 8 * kc);
#pragma unroll
      for (int nt = 0; nt < NT; ++nt) {
        const int dt = min(wave + 4 * nt, n16 - 1);   // (past the last one: computed, not stored)
        mma(o[nt], pf, column8(ks, LDK, k + 8 * kc, dim + dt * 16, r16));
      }
    }
    __syncthreads();
  }

  // the rows' sums: over the 16 keys a lane group held, then over the waves
#pragma unroll
  for (int r = 0; r < 4; ++r) {
    const float v = sum16(lrun[r]);
    if (r16 == 0) sx[wave * R + 4 * kc + r] = v;
  }
  __syncthreads();
#pragma unroll
  for (int r = 0; r < 4; ++r) {
    const int m = 4 * kc + r;
    if (m >= q.nrows) continue;
    const float l = sx[m] + sx[R + m] + sx[2 * R + m] + sx[3 * R + m];
    if (p.splits == 1) {
      const int64_t t = q.tok0 + (q.r0 + m) / q.rep;
      const int h = q.h0 + (q.r0 + m) % q.rep;
      const float gate = p.gate ? sigmoid((float)static_cast<const T*>(p.gate)[t * p.ldg + h]) : 1.f, inv = gate / l;
      T* out = static_cast<T*>(p.out) + t * p.ldo + (int64_t)h * vdim + r16;
#pragma unroll
      for (int nt = 0; nt < NT; ++nt) {
        const int dt = wave + 4 * nt;
        if (dt < n16) out[dt * 16] = (T)(o[nt][r] * inv);
      }
    } else {
      float* out = q.part(p, s, m);
#pragma unroll
      for (int nt = 0; nt < NT; ++nt) {
        const int dt = wave + 4 * nt;
        if (dt < n16) out[dt * 16 + r16] = o[nt][r];
      }
      if (wave == 0 && r16 == 0) {
        out[vdim] = mrun[r];
        out[vdim + 1] = l;
      }
    }
  }
}

inline size_t gqa_rows_lds(int dim, int vdim, int rep, bool bias) {
  return ((size_t)64 * (dim + vdim + 8) + (size_t)64 * 72) * 2 + (bias ? (size_t)rep * bias_window(64, 64, rep) * 4 : 0);
}

// NK k-steps (of 32) of a query row, NV value tiles (of 16 columns)
template <int NK, int NV, int U>
__global__ __launch_bounds__(256, NV <= 8 ? 2 : 1) void gqa_rows_kernel(const vmi_hy_attention_args p, const vmi_hy_step s) {
  constexpr int R = 64, KT = 64, LDP = KT + 8;
  extern __shared__ __attribute__((aligned(16))) unsigned char smem[];
  const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6), kc = lane >> 4, r16 = lane & 15;
  const int dim = p.dim, vdim = p.vdim, LDK = dim + vdim + 8;
  b16* ks = reinterpret_cast<b16*>(smem);          // [64][LDK]
  b16* ps = ks + (size_t)KT * LDK + wave * 16 * LDP;   // [16][LDP], this wave's
  float* bl = reinterpret_cast<float*>(ks + (size_t)KT * LDK + 64 * LDP);
  const QueryTile q(p, s, R, KT);
  if (q.nrows <= 0 || q.empty(p, s, tid)) return;
  KeyTile<b16, KT, U> keys;
  keys.open(p, s, q, R);
  const int m0 = wave * 16;   // (rows past the last one repeat it and are not stored)
  b16x8 qr[NK];
  {
    const int row = q.r0 + min(m0 + r16, q.nrows - 1);
    const b16* src = static_cast<const b16*>(p.q) + ((int64_t)(q.tok0 + row / q.rep) * p.heads + q.h0 + row % q.rep) * dim + 8 * kc;
#pragma unroll
    for (int k = 0; k < NK; ++k) qr[k] = load8(src + min(32 * k, dim - 32));
  }
  f32x4 o[NV];
  float mrun[4], lrun[4];
  int lim[4], low[4], boff[4];   // last and first key row m sees, its place in the bias window
#pragma unroll
  for (int nt = 0; nt < NV; ++nt) o[nt] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
  for (int r = 0; r < 4; ++r) {
    const int row = q.r0 + min(m0 + 4 * kc + r, q.nrows - 1), hh = row % q.rep;
    mrun[r] = -1e30f;
    lrun[r] = 0.f;
    if (p.sink && q.split == 0) {   // counted once: by one lane of the first split
      mrun[r] = p.sink[q.h0 + hh];
      lrun[r] = r16 == 0 ? 1.f : 0.f;
    }
    lim[r] = q.ctx + row / q.rep;
    low[r] = p.chunk > 0 ? lim[r] / p.chunk * p.chunk : 0;
    boff[r] = hh * keys.BW + lim[r] - q.first + KT - 1 - r16;
  }
  const float sc2 = p.scale * 1.4426950408889634f;   // scores in units of log 2
  // what the wave's rows see, all of them and any of them: tiles outside need no look at single keys
  const int lim0 = q.ctx + (q.r0 + min(m0, q.nrows - 1)) / q.rep, lim1 = q.ctx + (q.r0 + min(m0 + 15, q.nrows - 1)) / q.rep;
  const int low0 = p.chunk > 0 ? lim0 / p.chunk * p.chunk : 0, low1 = p.chunk > 0 ? lim1 / p.chunk * p.chunk : 0;
  const int n16 = vdim >> 4, nk = dim >> 5;

  for (int kt = q.kt0; kt < q.kt1; ++kt) {
    keys.step(ks, bl, LDK, kt, q.kt1);
    __syncthreads();
    const int key0 = kt * KT;
    if (key0 <= lim1 && key0 + KT > low0) {
      f32x4 sc[4];
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        sc[j] = f32x4{0.f, 0.f, 0.f, 0.f};
        const b16* krow = ks + (j * 16 + r16) * LDK + 8 * kc;
#pragma unroll
        for (int k = 0; k < NK; ++k)
          if (NK <= 4 || k < nk) mma(sc[j], qr[k], k < nk ? load8(krow + 32 * k) : zero8<b16>());
      }
      const bool whole = key0 + KT - 1 <= lim0 && key0 >= low1;
      f32x4 mx;
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        float v = -INFINITY;
#pragma unroll
        for (int j = 0; j < 4; ++j) {
          const float b = keys.bn ? bl[boff[r] - 16 * j] : 0.f;
          sc[j][r] = fmaf(sc[j][r], sc2, b);
          if (!whole) {
            const int key = key0 + j * 16 + r16;
            sc[j][r] = key <= lim[r] && key >= low[r] ? sc[j][r] : -INFINITY;
          }
          v = fmaxf(v, sc[j][r]);
        }
        mx[r] = max16(v);
      }
      float alpha[4];
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const float mn = fmaxf(mrun[r], mx[r]);
        alpha[r] = exp2_hw(mrun[r] - mn);
        mrun[r] = mn;
        lrun[r] *= alpha[r];
#pragma unroll
        for (int j = 0; j < 4; ++j) {
          const b16 pr = (b16)exp2_hw(sc[j][r] - mn);
          lrun[r] += (float)pr;   // (what is summed is what multiplies the values)
          ps[(4 * kc + r) * LDP + j * 16 + r16] = pr;
        }
      }
#pragma unroll
      for (int nt = 0; nt < NV; ++nt)
#pragma unroll
        for (int r = 0; r < 4; ++r) o[nt][r] *= alpha[r];
#pragma unroll
      for (int k = 0; k < KT; k += 32) {
        const b16x8 pf = load8(ps + r16 * LDP + k + 8 * kc);
#pragma unroll
        for (int nt = 0; nt < NV; ++nt)
          if (nt < n16) mma(o[nt], pf, column8(ks, LDK, k + 8 * kc, dim + nt * 16, r16));
      }
    }
    __syncthreads();
  }
#pragma unroll
  for (int r = 0; r < 4; ++r) {
    const float l = sum16(lrun[r]);
    const int m = m0 + 4 * kc + r;
    if (m >= q.nrows) continue;
    if (p.splits == 1) {
      const int64_t t = q.tok0 + (q.r0 + m) / q.rep;
      const int h = q.h0 + (q.r0 + m) % q.rep;
      const float gate = p.gate ? sigmoid((float)static_cast<const b16*>(p.gate)[t * p.ldg + h]) : 1.f, inv = gate / l;
      b16* out = static_cast<b16*>(p.out) + t * p.ldo + (int64_t)h * vdim + r16;
#pragma unroll
      for (int nt = 0; nt < NV; ++nt)
        if (nt < n16) out[nt * 16] = (b16)(o[nt][r] * inv);
    } else {
      float* out = q.part(p, s, m);
#pragma unroll
      for (int nt = 0; nt < NV; ++nt)
        if (nt < n16) out[nt * 16 + r16] = o[nt][r];
      if (r16 == 0) {
        out[vdim] = mrun[r];
        out[vdim + 1] = l;
      }
    }
  }
}

// q and k over their root mean square, k and v into the cache; one workgroup per token, 16 lanes per head
template <typename T>
__global__ __launch_bounds__(256) void kv_prep_kernel(const vmi_hy_kv_prep_args p, const vmi_hy_step s) {
  const int t = blockIdx.x, tid = threadIdx.x, l = tid & 15, D = p.dim + p.vdim;
  if (s.tok_seq[t] < 0) return;
  const int64_t slot = s.tok_slot[t];
  const T* row = static_cast<const T*>(p.proj) + (int64_t)t * p.ldp;
  T* crow = slot >= 0 ? static_cast<T*>(p.cache) + slot * p.kv_heads * D : nullptr;
  for (int u = tid >> 4; u < p.heads + p.kv_heads; u += 16) {
    const T* src = row + (int64_t)u * p.dim;
    float ss = 0.f;
    for (int k = l * 8; k < p.dim; k += 128) {
      const f32x8 v = to_f32<T>(load8(src + k));
#pragma unroll
      for (int e = 0; e < 8; ++e) ss = fmaf(v[e], v[e], ss);
    }
    ss = sum16(ss);
    const float r = 1.f / sqrtf(ss / (float)p.dim_n + p.eps);
    T* dst = u < p.heads ? static_cast<T*>(p.q) + ((int64_t)t * p.heads + u) * p.dim : crow ? crow + (int64_t)(u - p.heads) * D : nullptr;
    if (!dst) continue;
    for (int k = l * 8; k < p.dim; k += 128) {
      f32x8 v = to_f32<T>(load8(src + k));
#pragma unroll
      for (int e = 0; e < 8; ++e) v[e] *= r;
      *reinterpret_cast<V8<T>*>(dst + k) = from_f32<T>(v);
    }
  }
  if (!crow) return;
  const T* v = row + (int64_t)(p.heads + p.kv_heads) * p.dim;
  for (int u = tid * 8; u < p.kv_heads * p.vdim; u += 2048) {
    const int g = u / p.vdim, k = u - g * p.vdim;
    *reinterpret_cast<V8<T>*>(crow + (int64_t)g * D + p.dim + k) = load8(v + u);
  }
}

template <typename T>
static int launched_gqa(const vmi_hy_attention_args& p, const vmi_hy_step& s, hipStream_t st) {
  if (p.splits > 1) launch_combine<T>(Combine{p.partial, p.out, p.gate, s.tok_seq, p.ldo, p.ldg, s.T, p.heads, p.vdim, p.splits}, st);
  return launched("vmi_hy_attention");
}

template <typename T, int KT, int NT, int U>
static int launch_gqa(const vmi_hy_attention_args& p, const vmi_hy_step& s, hipStream_t st) {
  auto* fn = gqa_kernel<T, KT, NT, U>;
  const size_t lds = gqa_lds<T, KT>(p.dim, p.vdim, p.heads / p.kv_heads, p.bias != nullptr);
  if (int rc = allow_lds(fn, lds, "vmi_hy_attention")) return rc;
  hipLaunchKernelGGL(fn, dim3(p.n_tiles, p.splits, p.kv_heads), dim3(256), lds, st, p, s);
  return launched_gqa<T>(p, s, st);
}

template <int NK, int NV, int U>
static int launch_gqa_rows(const vmi_hy_attention_args& p, const vmi_hy_step& s, hipStream_t st) {
  auto* fn = gqa_rows_kernel<NK, NV, U>;
  const size_t lds = gqa_rows_lds(p.dim, p.vdim, p.heads / p.kv_heads, p.bias != nullptr);
  if (int rc = allow_lds(fn, lds, "vmi_hy_attention")) return rc;
  hipLaunchKernelGGL(fn, dim3(p.n_tiles, p.splits, p.kv_heads), dim3(256), lds, st, p, s);
  return launched_gqa<b16>(p, s, st);
}

template <typename T, int KT>
static int gqa_width(const vmi_hy_attention_args& p, const vmi_hy_step& s, hipStream_t st) {
  const int units = (p.dim + p.vdim + 2048 / KT - 1) / (2048 / KT);   // of 8 elements of a cache row, per thread
  constexpr int H = 64 / KT;                                          // (tiles of 32 keys: twice the threads per key)
  if (p.vdim <= 128 && units * H <= 4) return launch_gqa<T, KT, 2, 4 / H>(p, s, st);
  if (p.vdim <= 128 && units * H <= 8) return launch_gqa<T, KT, 2, 8 / H>(p, s, st);
  if (p.vdim <= 256 && units * H <= 8) return launch_gqa<T, KT, 4, 8 / H>(p, s, st);
  if (p.vdim <= 512 && units * H <= 16) return launch_gqa<T, KT, 8, 16 / H>(p, s, st);
  if constexpr (sizeof(T) == 2 || KT == 32)
    if (p.vdim <= 512 && units * H <= 32) return launch_gqa<T, KT, 8, 32 / H>(p, s, st);
  return fail(VMI_HY_E_SHAPE, "vmi_hy_attention", "heads this large are not built");
}

// row tiles of 16 that a workgroup takes: 4 (a wave each) where more than one is wanted and the kernel is built for it
static int gqa_row_tiles(int dim, int vdim, int want, int dtype) {
  return dtype == VMI_HY_BF16 && want >= 2 && dim <= 256 && vdim <= 256 ? 4 : 1;
}

template <typename T>
static int run_gqa(const vmi_hy_attention_args& p, const vmi_hy_step& s, hipStream_t st) {
  if (p.row_tiles != 1 && p.row_tiles != gqa_row_tiles(p.dim, p.vdim, 4, p.dtype))
    return fail(VMI_HY_E_ARG, "vmi_hy_attention", "row_tiles is what vmi_hy_attention_row_tiles returns");
  if constexpr (sizeof(T) == 2) {
    if (p.row_tiles == 4) {
      if (p.dim <= 128 && p.vdim <= 128) return launch_gqa_rows<4, 8, 8>(p, s, st);
      return launch_gqa_rows<8, 16, 16>(p, s, st);
    }
  }
  const bool wide = gqa_lds<T, 64>(p.dim, p.vdim, p.heads / p.kv_heads, p.bias != nullptr) <= LDS_PER_CU &&
                    (sizeof(T) == 2 || p.dim + p.vdim <= 512);
  return wide ? gqa_width<T, 64>(p, s, st) : gqa_width<T, 32>(p, s, st);
}

}  // namespace vmi_hybrid

using namespace vmi_hybrid;

extern "C" {

int vmi_hy_kv_prep(const vmi_hy_kv_prep_args* a, const vmi_hy_step* s, void* stream) {
  static const char* who = "vmi_hy_kv_prep";
  if (!a || !s || !a->proj || !a->q || !a->cache || !s->tok_seq || !s->tok_slot || s->T <= 0 || a->heads <= 0 || a->kv_heads <= 0 ||
      a->heads % a->kv_heads || a->dim <= 0 || a->vdim <= 0 || a->dim_n <= 0 || a->dim_n > a->dim)
    return fail(VMI_HY_E_ARG, who, "null pointer or a size out of range");
  if ((a->dim & 31) || (a->vdim & 31) || (a->ldp & 7) || ((uintptr_t)a->proj & 15))
    return fail(VMI_HY_E_SHAPE, who, "needs sizes that are multiples of 32 and aligned rows");
  DeviceScope dev(a->device);
  if (!dev.ok) return fail(VMI_HY_E_HIP, who, "hipSetDevice failed");
  hipStream_t st = static_cast<hipStream_t>(stream);
  if (a->dtype == VMI_HY_BF16)
    hipLaunchKernelGGL(kv_prep_kernel<b16>, dim3(s->T), dim3(256), 0, st, *a, *s);
  else
    hipLaunchKernelGGL(kv_prep_kernel<float>, dim3(s->T), dim3(256), 0, st, *a, *s);
  return launched(who);
}

int32_t vmi_hy_attention_row_tiles(int32_t dim, int32_t vdim, int32_t want, int32_t dtype) { return gqa_row_tiles(dim, vdim, want, dtype); }

int vmi_hy_attention(const vmi_hy_attention_args* a, const vmi_hy_step* s, void* stream) {
  static const char* who = "vmi_hy_attention";
  if (!a || !s || !a->q || !a->cache || !a->out || !a->tiles || !s->tok_seq || !s->q_start || !s->q_len || !s->ctx || !s->table ||
      s->T <= 0 || s->table_ld <= 0 || s->page_size <= 0 || a->heads <= 0 || a->kv_heads <= 0 || a->heads % a->kv_heads || a->dim <= 0 ||
      a->vdim <= 0 || a->n_tiles <= 0 || a->splits <= 0 || a->splits > 128 || (a->splits > 1 && !a->partial) || a->chunk < 0 ||
      (a->bias && a->bias_n <= 0) || a->kv_heads > 65535)
    return fail(VMI_HY_E_ARG, who, "null pointer or a size out of range");
  if ((a->dim & 31) || (a->vdim & 31)) return fail(VMI_HY_E_SHAPE, who, "needs sizes that are multiples of 32");
  DeviceScope dev(a->device);
  if (!dev.ok) return fail(VMI_HY_E_HIP, who, "hipSetDevice failed");
  hipStream_t st = static_cast<hipStream_t>(stream);
  return a->dtype == VMI_HY_BF16 ? run_gqa<b16>(*a, *s, st) : run_gqa<float>(*a, *s, st);
}

}  // extern "C"
