// Latent attention over a paged cache of latents (include/vmi_hybrid.h): the queries are taken into the latent space (the key
// up-projection is folded into them), so a cache row [rank | rot] is at once the key of ALL heads and, its first `rank` columns,
// their value: one page read serves every head, and the rows of a query tile are (token, head) pairs.
//
// A workgroup takes 16 * RT query rows and walks its keys in tiles of KT cache rows.  A tile comes from the pages into LDS once
// (requested one tile ahead, held in registers meanwhile) and is used three ways: wave w scores the 16 keys 16 w ..; softmax
// statistics meet in LDS; then wave w adds the value columns w, w + 4, ... (tiles of 16) of all rows, the value operand read
// column-wise from the same LDS rows (ds_read_b64_tr_b16).  Scores, softmax and accumulators are fp32.  A sequence whose rows do
// not fill the chip has its keys dealt to `splits` workgroups, whose unnormalised parts a second kernel adds up.
#include "hybrid_softmax.hpp"

namespace vmi_hybrid {

template <typename T, int KT, int RT>
inline size_t attention_lds(int D) {
  return ((size_t)(KT + 16 * RT) * (D + pad_of<T>()) + (size_t)16 * RT * (KT + pad_of<T>())) * sizeof(T) + (size_t)4 * 16 * RT * 4;
}

// RT row tiles, NT value tiles (of 16 columns) per wave, U 16-byte-element units of a cache row per thread
// EXACT: a row has exactly that many (its length is known to the compiler: loops over it unroll, and with one row tile the query
// stays in registers, which leaves LDS for a second workgroup)
template <typename T, int KT, int RT, int NT, int U, bool EXACT>
__global__ __launch_bounds__(256, EXACT && RT == 1 ? 2 : 1) void latent_attention_kernel(const vmi_hy_latent_attention_args p, const vmi_hy_step s) {
  constexpr int R = 16 * RT, TPK = 256 / KT, PAD = pad_of<T>(), LDP = KT + PAD, SW = KT / 16;   // SW waves score
  extern __shared__ __attribute__((aligned(16))) unsigned char smem[];
  constexpr bool QREG = EXACT && RT == 1 && sizeof(T) == 2;
  const int D = EXACT ? U * TPK * 8 : p.rank + p.rot, LDK = D + PAD;
  T* ks = reinterpret_cast<T*>(smem);              // [KT][LDK]
  T* qs = ks + (size_t)KT * LDK;                   // [R][LDK]
  T* ps = qs + (QREG ? 0 : (size_t)R * LDK);       // [R][LDP]
  float* sx = reinterpret_cast<float*>(ps + (size_t)R * LDP);   // [4][R]
  const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6), kc = lane >> 4, r16 = lane & 15;
  const int e = p.tiles[2 * blockIdx.x], r0 = p.tiles[2 * blockIdx.x + 1], split = blockIdx.y;
  if (e < 0) return;
  const int H = p.heads, ctx = s.ctx[e];
  const int nrows = min(R, s.q_len[e] * H - r0);
  if (nrows <= 0) return;
  const int64_t grow0 = (int64_t)s.q_start[e] * H + r0;          // row of q / out
  const int kv_end = ctx + (r0 + nrows - 1) / H + 1;
  const int nkt = (kv_end + KT - 1) / KT, tps = (nkt + p.splits - 1) / p.splits;
  const int kt0 = split * tps, kt1 = min(nkt, kt0 + tps);
  const int n16 = p.rank >> 4, d0 = (int)blockIdx.z * (NT * 4);   // this workgroup's value tiles: d0 + wave + 4 nt
  float* part = p.partial ? p.partial + ((int64_t)split * s.T * H + grow0) * (p.rank + 2) : nullptr;
  if (kt0 >= kt1) {   // (splits > 1 only: split 0 always has keys)
    if (blockIdx.z == 0 && tid < nrows) {
      part[(int64_t)tid * (p.rank + 2) + p.rank] = -1e30f;
      part[(int64_t)tid * (p.rank + 2) + p.rank + 1] = 0.f;
    }
    return;
  }

  const T* cache = static_cast<const T*>(p.cache);
  const int* tab = s.table + (int64_t)e * s.table_ld;
  const int kj = tid / TPK, kcol = (tid % TPK) * 8;   // this thread's key of a tile, first column
  // The page number of a tile is read one tile before the tile itself, and not touched before that tile is requested: loads
  // complete in order, so an earlier use would wait for everything requested in between.  Keys past the end read the last one's
  // row and columns past the row its last ones: nothing lane-wise stands around a load, all of a tile's are in flight together.
  auto key_of = [&](int kt) { return min(kt * KT + kj, kv_end - 1); };
  V8<T> kr[U];
  auto load_tile = [&](int page, int kt) {
    const T* src = cache + ((int64_t)page * s.page_size + key_of(kt) % s.page_size) * D;
#pragma unroll
    for (int i = 0; i < U; ++i) kr[i] = load8(src + min(kcol + i * TPK * 8, D - 8));
  };
  load_tile(tab[key_of(kt0) / s.page_size], kt0);
  int next_page = tab[key_of(min(kt0 + 1, kt1 - 1)) / s.page_size];

  constexpr int QK = QREG ? U * TPK / 4 : 1;   // k-steps of a row
  V8<T> qr[QK];
  if constexpr (QREG) {   // (rows past the last one repeat it and are not stored)
#pragma unroll
    for (int k = 0; k < QK; ++k) qr[k] = load8(static_cast<const T*>(p.q) + (grow0 + min(r16, nrows - 1)) * D + k * 32 + 8 * kc);
  } else {
    for (int u = tid; u < R * (D >> 3); u += 256) {
      const int m = u / (D >> 3), k = (u - m * (D >> 3)) * 8;
      *reinterpret_cast<V8<T>*>(qs + m * LDK + k) = m < nrows ? load8(static_cast<const T*>(p.q) + (grow0 + m) * D + k) : zero8<T>();
    }
  }

  f32x4 o[RT][NT];
  float mrun[RT][4], lrun[RT][4];
  int lim[RT][4];   // last key row m sees
#pragma unroll
  for (int rt = 0; rt < RT; ++rt) {
#pragma unroll
    for (int nt = 0; nt < NT; ++nt) o[rt][nt] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      mrun[rt][r] = -1e30f;
      lrun[rt][r] = 0.f;
      lim[rt][r] = ctx + (r0 + rt * 16 + 4 * kc + r) / H;
    }
  }
  const float sc2 = p.scale * 1.4426950408889634f;   // scores in units of log 2

  for (int kt = kt0; kt < kt1; ++kt) {
#pragma unroll
    for (int i = 0; i < U; ++i)   // (a clamped column is written again with the same values)
      *reinterpret_cast<V8<T>*>(ks + kj * LDK + min(kcol + i * TPK * 8, D - 8)) = kr[i];
    if (kt + 1 < kt1) {
      load_tile(next_page, kt + 1);
      next_page = tab[key_of(min(kt + 2, kt1 - 1)) / s.page_size];
    }
    __syncthreads();
    f32x4 sc[RT];
#pragma unroll
    for (int rt = 0; rt < RT; ++rt) sc[rt] = f32x4{0.f, 0.f, 0.f, 0.f};
    if (SW == 4 || wave < SW) {
      const T* krow = ks + (wave * 16 + r16) * LDK + 8 * kc;
      const T* qrow = qs + r16 * LDK + 8 * kc;
      if constexpr (QREG) {
        f32x4 odd = f32x4{0.f, 0.f, 0.f, 0.f};   // (two chains of sums)
#pragma unroll
        for (int k = 0; k < QK; ++k) mma(k & 1 ? odd : sc[0], qr[k], load8(krow + k * 32));
        sc[0] += odd;
      } else if constexpr (EXACT) {
#pragma unroll
        for (int k = 0; k < U * TPK * 8; k += 32) {
          const V8<T> kf = load8(krow + k);
#pragma unroll
          for (int rt = 0; rt < RT; ++rt) mma(sc[rt], load8(qrow + rt * 16 * LDK + k), kf);
        }
      } else {
#pragma unroll 2
        for (int k = 0; k < D; k += 32) {
          const V8<T> kf = load8(krow + k);
#pragma unroll
          for (int rt = 0; rt < RT; ++rt) mma(sc[rt], load8(qrow + rt * 16 * LDK + k), kf);
        }
      }
      const int key = kt * KT + wave * 16 + r16;
#pragma unroll
      for (int rt = 0; rt < RT; ++rt) {
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          sc[rt][r] = key <= lim[rt][r] ? sc[rt][r] * sc2 : -INFINITY;   // (keys past kv_end are past every row's limit)
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
        if (SW == 4 || wave < SW) {
          const T pr = (T)exp2_hw(sc[rt][r] - mn);
          lrun[rt][r] = fmaf(lrun[rt][r], alpha[rt][r], (float)pr);   // (what is summed is what multiplies the values)
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
#pragma unroll
    for (int k = 0; k < KT; k += 32) {
      V8<T> pf[RT];
#pragma unroll
      for (int rt = 0; rt < RT; ++rt) pf[rt] = load8(ps + (rt * 16 + r16) * LDP + k + 8 * kc);
#pragma unroll
      for (int nt = 0; nt < NT; ++nt) {
        const int dt = min(d0 + wave + 4 * nt, n16 - 1);   // (past the last one: computed, not stored)
        const V8<T> vf = column8(ks, LDK, k + 8 * kc, dt * 16, r16);
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
#pragma unroll
  for (int rt = 0; rt < RT; ++rt) {
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int m = rt * 16 + 4 * kc + r;
      if (m >= nrows) continue;
      const float l = sx[m] + sx[R + m] + sx[2 * R + m] + sx[3 * R + m];
      if (p.splits == 1) {
        const float inv = 1.f / l;
        T* out = static_cast<T*>(p.out) + (grow0 + m) * p.rank + r16;
#pragma unroll
        for (int nt = 0; nt < NT; ++nt) {
          const int dt = d0 + wave + 4 * nt;
          if (dt < n16) out[dt * 16] = (T)(o[rt][nt][r] * inv);
        }
      } else {
        float* out = part + (int64_t)m * (p.rank + 2);
#pragma unroll
        for (int nt = 0; nt < NT; ++nt) {
          const int dt = d0 + wave + 4 * nt;
          if (dt < n16) out[dt * 16 + r16] = o[rt][nt][r];
        }
        if (blockIdx.z == 0 && wave == 0 && r16 == 0) {
          out[p.rank] = mrun[rt][r];
          out[p.rank + 1] = l;
        }
      }
    }
  }
}

// RMS norm of the latent, rotation of the shared key and of the query parts; one workgroup per token
template <typename T>
__global__ __launch_bounds__(256) void latent_prep_kernel(const vmi_hy_latent_prep_args p, const vmi_hy_step s) {
  extern __shared__ float cs[];   // [rot_n / 2][2]
  __shared__ float part[4];
  const int t = blockIdx.x, tid = threadIdx.x, half = p.rot_n >> 1, hd = p.dim + p.rot, D = p.rank + p.rot;
  const int seq = s.tok_seq[t];
  const int64_t slot = s.tok_slot[t];
  const double pos = (double)s.tok_pos[t];
  const T* row = static_cast<const T*>(p.proj) + (int64_t)t * p.ldp;
  const T* lat = row + p.heads * hd;
  f32x8 v0 = to_f32<T>(load8(lat + min(tid * 8, p.rank - 8))), w0 = load8(p.norm_w + min(tid * 8, p.rank - 8));
  if (seq < 0) return;
  for (int i = tid; i < half; i += 256) {   // the angle reduced in fp64: exact to fp32 at any position
    const double a = pos * p.freq[i];
    const float r = (float)(a - 6.283185307179586476925 * rint(a * 0.15915494309189533577));
    cs[2 * i] = cosf(r);
    cs[2 * i + 1] = sinf(r);
  }
  float ss = 0.f;
  for (int k = tid * 8; k < p.rank; k += 2048) {
    const f32x8 v = k < 2048 ? v0 : to_f32<T>(load8(lat + k));
#pragma unroll
    for (int e = 0; e < 8; ++e) ss = fmaf(v[e], v[e], ss);
  }
  ss = wave_sum(ss);
  if ((tid & 63) == 0) part[tid >> 6] = ss;
  __syncthreads();
  const float rms = 1.f / sqrtf((part[0] + part[1] + part[2] + part[3]) / (float)p.rank_n + p.eps);
  T* crow = slot >= 0 ? static_cast<T*>(p.cache) + slot * D : nullptr;
  if (crow) {
    for (int k = tid * 8; k < p.rank; k += 2048) {
      f32x8 v = k < 2048 ? v0 : to_f32<T>(load8(lat + k));
      const f32x8 w = k < 2048 ? w0 : load8(p.norm_w + k);
#pragma unroll
      for (int e = 0; e < 8; ++e) v[e] = v[e] * rms * w[e];
      *reinterpret_cast<V8<T>*>(crow + k) = from_f32<T>(v);
    }
  }
  if ((half & 7) == 0) {   // eight pairs at a time
    const int per = half >> 3;
    for (int u = tid; u < (p.heads + 1) * per; u += 256) {
      const int h = u / per, i = (u - h * per) * 8;
      const T* src = h < p.heads ? row + h * hd + p.dim : lat + p.rank;
      T* dst = h < p.heads ? static_cast<T*>(p.q) + ((int64_t)t * p.heads + h) * D + p.rank : (crow ? crow + p.rank : nullptr);
      if (!dst) continue;
      const f32x8 a = to_f32<T>(load8(src + i)), b = to_f32<T>(load8(src + i + half));
      f32x8 x, y;
#pragma unroll
      for (int e = 0; e < 8; ++e) {
        const float c = cs[2 * (i + e)], sn = cs[2 * (i + e) + 1];
        x[e] = a[e] * c - b[e] * sn;
        y[e] = b[e] * c + a[e] * sn;
      }
      *reinterpret_cast<V8<T>*>(dst + i) = from_f32<T>(x);
      *reinterpret_cast<V8<T>*>(dst + i + half) = from_f32<T>(y);
      if (i == 0)
        for (int k = p.rot_n; k < p.rot; k += 8) *reinterpret_cast<V8<T>*>(dst + k) = load8(src + k);   // passes unrotated
    }
    return;
  }
  // heads 0 .. heads - 1: the query's rotated part; "head" `heads`: the shared key
  T* qrow = static_cast<T*>(p.q) + (int64_t)t * p.heads * D;
  for (int u = tid; u < (p.heads + 1) * p.rot; u += 256) {
    const int h = u / p.rot, i = u - h * p.rot;
    const T* src = h < p.heads ? row + h * hd + p.dim : lat + p.rank;
    T* dst = h < p.heads ? qrow + (int64_t)h * D + p.rank : (crow ? crow + p.rank : nullptr);
    if (!dst) continue;
    if (i >= p.rot_n) {
      dst[i] = src[i];   // passes unrotated (padding: zeros)
    } else if (i < half) {
      dst[i] = (T)((float)src[i] * cs[2 * i] - (float)src[i + half] * cs[2 * i + 1]);
    } else {
      const int j = i - half;
      dst[i] = (T)((float)src[i] * cs[2 * j] + (float)src[j] * cs[2 * j + 1]);
    }
  }
}

template <typename T, int KT, int RT, int NT, int U, bool EXACT = false>
static int launch_attention(const vmi_hy_latent_attention_args& p, const vmi_hy_step& s, hipStream_t st) {
  auto* fn = latent_attention_kernel<T, KT, RT, NT, U, EXACT>;
  const int D = p.rank + p.rot;
  const size_t lds = attention_lds<T, KT, RT>(D) - (EXACT && RT == 1 && sizeof(T) == 2 ? (size_t)16 * (D + pad_of<T>()) * sizeof(T) : 0);
  if (int rc = allow_lds(fn, lds, "vmi_hy_latent_attention")) return rc;
  const int zb = ((p.rank >> 4) + 4 * NT - 1) / (4 * NT);
  hipLaunchKernelGGL(fn, dim3(p.n_tiles, p.splits, zb), dim3(256), lds, st, p, s);
  if (p.splits > 1)
    launch_combine<T>(Combine{p.partial, p.out, nullptr, s.tok_seq, (int64_t)p.heads * p.rank, 0, s.T, p.heads, p.rank, p.splits}, st);
  return launched("vmi_hy_latent_attention");
}

template <typename T, int KT, int RT>
static int attention_width(const vmi_hy_latent_attention_args& p, const vmi_hy_step& s, hipStream_t st) {
  const int units = (p.rank + p.rot + 2048 / KT - 1) / (2048 / KT);   // of 8 elements of a cache row, per thread
  if (p.rank <= 128 && units <= 8) return launch_attention<T, KT, RT, 2, 8>(p, s, st);
  if (p.rank <= 256 && units <= 12) return launch_attention<T, KT, RT, 4, 12>(p, s, st);
  if constexpr (sizeof(T) == 2 && KT == 64)
    if (p.rank + p.rot == 576) return launch_attention<T, KT, RT, 8, 18, true>(p, s, st);
  if (units <= 20) return launch_attention<T, KT, RT, 8, 20>(p, s, st);
  if constexpr (RT == 1)
    if (units <= 32) return launch_attention<T, KT, RT, 8, 32>(p, s, st);
  return fail(VMI_HY_E_SHAPE, "vmi_hy_latent_attention", "cache rows this long are not built");
}

// the most row tiles (1, 2, 4; at most `want`) a workgroup can hold beside a tile of 64 keys; fp32 is built for one
static int row_tiles_for(int D, int want, int dtype) {
  if (dtype == VMI_HY_BF16 && D <= 640) {
    if (want >= 4 && attention_lds<b16, 64, 4>(D) <= LDS_PER_CU) return 4;
    if (want >= 2 && attention_lds<b16, 64, 2>(D) <= LDS_PER_CU) return 2;
  }
  return 1;
}

template <typename T>
static int run_attention(const vmi_hy_latent_attention_args& p, const vmi_hy_step& s, hipStream_t st) {
  const int D = p.rank + p.rot;
  if constexpr (sizeof(T) == 2) {
    if (p.row_tiles == 4) return attention_width<T, 64, 4>(p, s, st);
    if (p.row_tiles == 2) return attention_width<T, 64, 2>(p, s, st);
  }
  if (p.row_tiles != 1) return fail(VMI_HY_E_ARG, "vmi_hy_latent_attention", "row_tiles is what vmi_hy_latent_row_tiles returns");
  // tiles of 64 keys where they fit LDS beside the query rows, of 32 otherwise
  return attention_lds<T, 64, 1>(D) <= LDS_PER_CU ? attention_width<T, 64, 1>(p, s, st) : attention_width<T, 32, 1>(p, s, st);
}

}  // namespace vmi_hybrid

using namespace vmi_hybrid;

extern "C" {

int vmi_hy_latent_prep(const vmi_hy_latent_prep_args* a, const vmi_hy_step* s, void* stream) {
  static const char* who = "vmi_hy_latent_prep";
  if (!a || !s || !a->proj || !a->q || !a->cache || !a->norm_w || !a->freq || !s->tok_seq || !s->tok_pos || !s->tok_slot || s->T <= 0 ||
      a->heads <= 0 || a->dim <= 0 || a->rot <= 0 || a->rank <= 0 || a->rot_n <= 0 || a->rot_n > a->rot || (a->rot_n & 1) ||
      a->rank_n <= 0 || a->rank_n > a->rank)
    return fail(VMI_HY_E_ARG, who, "null pointer or a size out of range");
  if ((a->dim & 31) || (a->rot & 31) || (a->rank & 31) || (a->ldp & 7) || a->rot_n > 8192)
    return fail(VMI_HY_E_SHAPE, who, "needs sizes that are multiples of 32");
  DeviceScope dev(a->device);
  if (!dev.ok) return fail(VMI_HY_E_HIP, who, "hipSetDevice failed");
  hipStream_t st = static_cast<hipStream_t>(stream);
  const size_t lds = (size_t)a->rot_n * 4;
  if (a->dtype == VMI_HY_BF16)
    hipLaunchKernelGGL(latent_prep_kernel<b16>, dim3(s->T), dim3(256), lds, st, *a, *s);
  else
    hipLaunchKernelGGL(latent_prep_kernel<float>, dim3(s->T), dim3(256), lds, st, *a, *s);
  return launched(who);
}

int32_t vmi_hy_latent_row_tiles(int32_t row_dim, int32_t want, int32_t dtype) { return row_tiles_for(row_dim, want, dtype); }

int vmi_hy_latent_attention(const vmi_hy_latent_attention_args* a, const vmi_hy_step* s, void* stream) {
  static const char* who = "vmi_hy_latent_attention";
  if (!a || !s || !a->q || !a->cache || !a->out || !a->tiles || !s->tok_seq || !s->q_start || !s->q_len || !s->ctx || !s->table ||
      s->T <= 0 || s->table_ld <= 0 || s->page_size <= 0 || a->heads <= 0 || a->rank <= 0 || a->rot <= 0 || a->n_tiles <= 0 ||
      a->splits <= 0 || a->splits > 128 || (a->splits > 1 && !a->partial))
    return fail(VMI_HY_E_ARG, who, "null pointer or a size out of range");
  if ((a->rank & 31) || (a->rot & 31)) return fail(VMI_HY_E_SHAPE, who, "needs sizes that are multiples of 32");
  DeviceScope dev(a->device);
  if (!dev.ok) return fail(VMI_HY_E_HIP, who, "hipSetDevice failed");
  hipStream_t st = static_cast<hipStream_t>(stream);
  return a->dtype == VMI_HY_BF16 ? run_attention<b16>(*a, *s, st) : run_attention<float>(*a, *s, st);
}

}  // extern "C"
