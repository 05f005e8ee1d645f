// Grouped-query softmax attention over a paged cache (include/vmi_hybrid.h): chunked masks, a bias by distance, a sink in the
// denominator, an output gate per head.  A cache row holds [key | value] of every key head side by side.
//
// A workgroup takes 16 * RT query rows of one key head — (token, head of the group) pairs, so a key tile read from the pages serves
// the whole group — and walks the keys its rows can see in tiles of KT: from the first row's chunk start to the last row's token.
// A tile comes into LDS once (requested one tile ahead, held in registers meanwhile): wave w scores the 16 keys 16 w .., statistics
// meet in LDS, then wave w adds value columns w, w + 4, ... (tiles of 16), read column-wise.  Scores, softmax and sums are fp32; the
// sink opens the running maximum and sum.  Tiles too few for the chip have their keys dealt to `splits` workgroups.
#include "hybrid_softmax.hpp"

namespace vmi_hybrid {

// distances that the rows of a tile (R of them, rep to a token) can have to the keys of one tile
__host__ __device__ inline int bias_window(int KT, int R, int rep) { return KT + (R + rep - 1) / rep; }

template <typename T, int KT, int RT>
inline size_t gqa_lds(int dim, int vdim, int rep, bool bias) {
  constexpr int PAD = pad_of<T>();
  return ((size_t)KT * (dim + vdim + PAD) + (size_t)16 * RT * (dim + PAD) + (size_t)16 * RT * (KT + PAD)) * sizeof(T) +
         (size_t)4 * 16 * RT * 4 + (bias ? (size_t)rep * bias_window(KT, 16 * RT, rep) * 4 : 0);
}

// RT row tiles, NT value tiles (of 16 columns) per wave, U 8-element units of a cache row per thread
template <typename T, int KT, int RT, int NT, int U>
__global__ __launch_bounds__(256) void gqa_kernel(const vmi_hy_attention_args p, const vmi_hy_step s) {
  constexpr int R = 16 * RT, TPK = 256 / KT, PAD = pad_of<T>(), LDP = KT + PAD, SW = KT / 16;   // SW waves score
  extern __shared__ __attribute__((aligned(16))) unsigned char smem[];
  const int dim = p.dim, vdim = p.vdim, D = dim + vdim, LDK = D + PAD, LDQ = dim + PAD;
  T* ks = reinterpret_cast<T*>(smem);              // [KT][LDK]
  T* qs = ks + (size_t)KT * LDK;                   // [R][LDQ]
  T* ps = qs + (size_t)R * LDQ;                    // [R][LDP]
  float* sx = reinterpret_cast<float*>(ps + (size_t)R * LDP);   // [4][R]
  float* bl = sx + 4 * R;                          // [rep][window]: the bias of the distances that occur in a tile
  const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6), kc = lane >> 4, r16 = lane & 15;
  const int e = p.tiles[2 * blockIdx.x], r0 = p.tiles[2 * blockIdx.x + 1], split = blockIdx.y, g = blockIdx.z;
  if (e < 0) return;
  const int rep = p.heads / p.kv_heads, ctx = s.ctx[e];
  const int nrows = min(R, s.q_len[e] * rep - r0);
  if (nrows <= 0) return;
  const int tok0 = s.q_start[e], h0 = g * rep;
  const int first = ctx + r0 / rep;                                        // position of the first row
  const int kv_begin = p.chunk > 0 ? first / p.chunk * p.chunk : 0, kv_end = ctx + (r0 + nrows - 1) / rep + 1;
  const int tb = kv_begin / KT, nkt = (kv_end + KT - 1) / KT - tb, tps = (nkt + p.splits - 1) / p.splits;
  const int kt0 = tb + split * tps, kt1 = min(tb + nkt, kt0 + tps);
  // row m: token tok0 + (r0 + m) / rep, head h0 + (r0 + m) % rep; partial results lie by (token, head)
  auto part_of = [&](int m) {
    return p.partial + (((int64_t)split * s.T + tok0 + (r0 + m) / rep) * p.heads + h0 + (r0 + m) % rep) * (vdim + 2);
  };
  if (kt0 >= kt1) {   // (splits > 1 only: split 0 always has keys)
    if (tid < nrows) {
      float* part = part_of(tid);
      part[vdim] = -1e30f;
      part[vdim + 1] = 0.f;
    }
    return;
  }
  const T* cache = static_cast<const T*>(p.cache) + (int64_t)g * D;
  const int64_t ldc = (int64_t)p.kv_heads * D;
  const int* tab = s.table + (int64_t)e * s.table_ld;
  const int kj = tid / TPK, kcol = (tid % TPK) * 8;   // this thread's key of a tile, first column
  // (as in the latent kernel: the page of a tile is known one tile before it is requested, keys past the end repeat the last one and
  //  columns past the row its last ones, so no lane-wise condition stands around a load)
  auto key_of = [&](int kt) { return min(kt * KT + kj, kv_end - 1); };
  V8<T> kr[U];
  auto load_tile = [&](int page, int kt) {
    const T* src = cache + ((int64_t)page * s.page_size + key_of(kt) % s.page_size) * ldc;
#pragma unroll
    for (int i = 0; i < U; ++i) kr[i] = load8(src + min(kcol + i * TPK * 8, D - 8));
  };
  load_tile(tab[key_of(kt0) / s.page_size], kt0);
  int next_page = tab[key_of(min(kt0 + 1, kt1 - 1)) / s.page_size];
  for (int u = tid; u < R * (dim >> 3); u += 256) {
    const int m = u / (dim >> 3), k = (u - m * (dim >> 3)) * 8, row = r0 + min(m, nrows - 1);
    *reinterpret_cast<V8<T>*>(qs + m * LDQ + k) =
        load8(static_cast<const T*>(p.q) + ((int64_t)(tok0 + row / rep) * p.heads + h0 + row % rep) * dim + k);
  }
  // the window's entry (hh, w): head hh, distance first - (last key of the tile) + w
  const int BW = bias_window(KT, R, rep), bn = p.bias ? rep * BW : 0;
  const float* bg = p.bias + (int64_t)h0 * p.bias_n;
  auto bias_at = [&](int kt, int u) {
    const int hh = u / BW, w = u - hh * BW;
    return bg[(int64_t)hh * p.bias_n + min(max(first - (kt * KT + KT - 1) + w, 0), p.bias_n - 1)];
  };
  constexpr int BU = 2;   // of a window, per thread, requested with the tile's keys
  float br[BU] = {};
  auto load_bias = [&](int kt) {
#pragma unroll
    for (int i = 0; i < BU; ++i)
      if (bn) br[i] = bias_at(kt, min(tid + 256 * i, bn - 1));
  };
  load_bias(kt0);

  f32x4 o[RT][NT];
  float mrun[RT][4], lrun[RT][4];
  int lim[RT][4], low[RT][4], boff[RT][4];   // last and first key row m sees, its bias row
#pragma unroll
  for (int rt = 0; rt < RT; ++rt) {
#pragma unroll
    for (int nt = 0; nt < NT; ++nt) o[rt][nt] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int row = r0 + min(rt * 16 + 4 * kc + r, nrows - 1), hh = row % rep;
      mrun[rt][r] = -1e30f;
      lrun[rt][r] = 0.f;
      if (p.sink && split == 0) {   // counted once: by one lane of the first split
        mrun[rt][r] = p.sink[h0 + hh];
        lrun[rt][r] = wave == 0 && r16 == 0 ? 1.f : 0.f;
      }
      lim[rt][r] = ctx + row / rep;
      low[rt][r] = p.chunk > 0 ? lim[rt][r] / p.chunk * p.chunk : 0;
      boff[rt][r] = hh * BW + lim[rt][r] - first;
    }
  }
  const float sc2 = p.scale * 1.4426950408889634f;   // scores in units of log 2

  for (int kt = kt0; kt < kt1; ++kt) {
#pragma unroll
    for (int i = 0; i < U; ++i)   // (a clamped column is written again with the same values)
      *reinterpret_cast<V8<T>*>(ks + kj * LDK + min(kcol + i * TPK * 8, D - 8)) = kr[i];
    if (bn) {
#pragma unroll
      for (int i = 0; i < BU; ++i) bl[min(tid + 256 * i, bn - 1)] = br[i];   // (a clamped entry is written again with the same value)
      for (int u = tid + 256 * BU; u < bn; u += 256) bl[u] = bias_at(kt, u);
    }
    if (kt + 1 < kt1) {
      load_bias(kt + 1);
      load_tile(next_page, kt + 1);
      next_page = tab[key_of(min(kt + 2, kt1 - 1)) / s.page_size];
    }
    __syncthreads();
    f32x4 sc[RT];
#pragma unroll
    for (int rt = 0; rt < RT; ++rt) sc[rt] = f32x4{0.f, 0.f, 0.f, 0.f};
    if (SW == 4 || wave < SW) {
      const T* krow = ks + (wave * 16 + r16) * LDK + 8 * kc;
      const T* qrow = qs + r16 * LDQ + 8 * kc;
#pragma unroll 2
      for (int k = 0; k < dim; k += 32) {
        const V8<T> kf = load8(krow + k);
#pragma unroll
        for (int rt = 0; rt < RT; ++rt) mma(sc[rt], load8(qrow + rt * 16 * LDQ + k), kf);
      }
      const int key = kt * KT + wave * 16 + r16;
#pragma unroll
      for (int rt = 0; rt < RT; ++rt) {
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const float b = bn ? bl[boff[rt][r] + KT - 1 - (wave * 16 + r16)] : 0.f;
          sc[rt][r] = key <= lim[rt][r] && key >= low[rt][r] ? fmaf(sc[rt][r], sc2, b) : -INFINITY;
          const float v = max16(sc[rt][r]);
          if (r16 == 0) sx[wave * R + rt * 16 + 4 * kc + r] = v;
        }
      }
    }
    __syncthreads();
    float alpha[RT][4];
#pragma unroll
    for (int rt = 0; rt < RT; ++rt) {
      f32x4 mx = *reinterpret_cast<const f32x4*>(sx + rt * 16 + 4 * kc);
#pragma unroll
      for (int w = 1; w < SW; ++w) {
        const f32x4 v = *reinterpret_cast<const f32x4*>(sx + w * R + rt * 16 + 4 * kc);
#pragma unroll
        for (int r = 0; r < 4; ++r) mx[r] = fmaxf(mx[r], v[r]);
      }
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const float mn = fmaxf(mrun[rt][r], mx[r]);
        alpha[rt][r] = exp2_hw(mrun[rt][r] - mn);
        mrun[rt][r] = mn;
        lrun[rt][r] *= alpha[rt][r];
        if (SW == 4 || wave < SW) {
          const T pr = (T)exp2_hw(sc[rt][r] - mn);
          lrun[rt][r] += (float)pr;   // (what is summed is what multiplies the values)
          ps[(rt * 16 + 4 * kc + r) * LDP + wave * 16 + r16] = pr;
        }
      }
    }
#pragma unroll
    for (int rt = 0; rt < RT; ++rt)
#pragma unroll
      for (int nt = 0; nt < NT; ++nt)
#pragma unroll
        for (int r = 0; r < 4; ++r) o[rt][nt][r] *= alpha[rt][r];
    __syncthreads();
    const int n16 = vdim >> 4;
#pragma unroll
    for (int k = 0; k < KT; k += 32) {
      V8<T> pf[RT];
#pragma unroll
      for (int rt = 0; rt < RT; ++rt) pf[rt] = load8(ps + (rt * 16 + r16) * LDP + k + 8 * kc);
#pragma unroll
      for (int nt = 0; nt < NT; ++nt) {
        const int dt = min(wave + 4 * nt, n16 - 1);   // (past the last one: computed, not stored)
        const V8<T> vf = column8(ks, LDK, k + 8 * kc, dim + dt * 16, r16);
#pragma unroll
        for (int rt = 0; rt < RT; ++rt) mma(o[rt][nt], pf[rt], vf);
      }
    }
    __syncthreads();
  }

  // the rows' sums: over the 16 keys a lane group held, then over the waves
#pragma unroll
  for (int rt = 0; rt < RT; ++rt)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const float v = sum16(lrun[rt][r]);
      if (r16 == 0) sx[wave * R + rt * 16 + 4 * kc + r] = v;
    }
  __syncthreads();
  const int n16 = vdim >> 4;
#pragma unroll
  for (int rt = 0; rt < RT; ++rt) {
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int m = rt * 16 + 4 * kc + r;
      if (m >= nrows) continue;
      const float l = sx[m] + sx[R + m] + sx[2 * R + m] + sx[3 * R + m];
      if (p.splits == 1) {
        const int64_t t = tok0 + (r0 + m) / rep;
        const int h = h0 + (r0 + m) % rep;
        const float gate = p.gate ? sigmoid((float)static_cast<const T*>(p.gate)[t * p.ldg + h]) : 1.f, inv = gate / l;
        T* out = static_cast<T*>(p.out) + t * p.ldo + (int64_t)h * vdim + r16;
#pragma unroll
        for (int nt = 0; nt < NT; ++nt) {
          const int dt = wave + 4 * nt;
          if (dt < n16) out[dt * 16] = (T)(o[rt][nt][r] * inv);
        }
      } else {
        float* out = part_of(m);
#pragma unroll
        for (int nt = 0; nt < NT; ++nt) {
          const int dt = wave + 4 * nt;
          if (dt < n16) out[dt * 16 + r16] = o[rt][nt][r];
        }
        if (wave == 0 && r16 == 0) {
          out[vdim] = mrun[rt][r];
          out[vdim + 1] = l;
        }
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

template <typename T, int KT, int RT, int NT, int U>
static int launch_gqa(const vmi_hy_attention_args& p, const vmi_hy_step& s, hipStream_t st) {
  auto* fn = gqa_kernel<T, KT, RT, NT, U>;
  const size_t lds = gqa_lds<T, KT, RT>(p.dim, p.vdim, p.heads / p.kv_heads, p.bias != nullptr);
  if (int rc = allow_lds(fn, lds, "vmi_hy_attention")) return rc;
  hipLaunchKernelGGL(fn, dim3(p.n_tiles, p.splits, p.kv_heads), dim3(256), lds, st, p, s);
  if (p.splits > 1) launch_combine<T>(Combine{p.partial, p.out, p.gate, s.tok_seq, p.ldo, p.ldg, s.T, p.heads, p.vdim, p.splits}, st);
  return launched("vmi_hy_attention");
}

template <typename T, int KT, int RT>
static int gqa_width(const vmi_hy_attention_args& p, const vmi_hy_step& s, hipStream_t st) {
  const int units = (p.dim + p.vdim + 2048 / KT - 1) / (2048 / KT);   // of 8 elements of a cache row, per thread
  constexpr int H = 64 / KT;                                          // (tiles of 32 keys: twice the threads per key)
  if (p.vdim <= 128 && units * H <= 4) return launch_gqa<T, KT, RT, 2, 4 / H>(p, s, st);
  if (p.vdim <= 128 && units * H <= 8) return launch_gqa<T, KT, RT, 2, 8 / H>(p, s, st);
  if (p.vdim <= 256 && units * H <= 8) return launch_gqa<T, KT, RT, 4, 8 / H>(p, s, st);
  if constexpr (RT <= 2)
    if (p.vdim <= 512 && units * H <= 16) return launch_gqa<T, KT, RT, 8, 16 / H>(p, s, st);
  if constexpr (RT == 1)
    if (p.vdim <= 512 && units * H <= 32) return launch_gqa<T, KT, RT, 8, 32 / H>(p, s, st);
  return fail(VMI_HY_E_SHAPE, "vmi_hy_attention", "heads this large are not built");
}

// the most row tiles (1, 2, 4; at most `want`) a workgroup takes beside a tile of 64 keys; fp32 is built for one
static int gqa_row_tiles(int dim, int vdim, int want, int dtype) {
  if (dtype == VMI_HY_BF16) {
    if (want >= 4 && dim + vdim <= 256) return 4;
    if (want >= 2 && dim + vdim <= 512 && vdim <= 512) return 2;
  }
  return 1;
}

template <typename T>
static int run_gqa(const vmi_hy_attention_args& p, const vmi_hy_step& s, hipStream_t st) {
  if (p.row_tiles > gqa_row_tiles(p.dim, p.vdim, 4, p.dtype) || (p.row_tiles != 1 && p.row_tiles != 2 && p.row_tiles != 4))
    return fail(VMI_HY_E_ARG, "vmi_hy_attention", "row_tiles is at most what vmi_hy_attention_row_tiles returns");
  if constexpr (sizeof(T) == 2) {
    if (p.row_tiles == 4) return gqa_width<T, 64, 4>(p, s, st);
    if (p.row_tiles == 2) return gqa_width<T, 64, 2>(p, s, st);
  }
  return gqa_lds<T, 64, 1>(p.dim, p.vdim, p.heads / p.kv_heads, p.bias != nullptr) <= LDS_PER_CU ? gqa_width<T, 64, 1>(p, s, st) : gqa_width<T, 32, 1>(p, s, st);
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
