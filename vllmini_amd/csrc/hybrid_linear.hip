// The linear layers and the elementwise ends of a step (include/vmi_hybrid.h).
//
// y = epilogue(prologue(x) . W^T), written for steps of few rows, where the weights are what has to be read: every wave owns 16
// output columns and streams its weight tiles (one contiguous KiB per k-step of 32) straight into registers one or two chunks ahead; the
// BM rows of x go through LDS in chunks of K, double-buffered, normalised / concatenated / rounded to the element type on their
// way in, so no normalised copy of the residual stream is ever written.  KS > 1: the k-steps of a chunk are dealt over KS waves
// whose partial tiles meet in LDS in a fixed order.  D[row = column n][col = row m]: a lane ends with 4 consecutive columns of
// one row, so every epilogue works on vectors.
#include <string>

#include "hybrid_common.hpp"

namespace vmi_hybrid {

static thread_local std::string g_err;
int fail(int code, const char* who, const char* what) {
  g_err.assign(who);
  g_err.append(": ");
  g_err.append(what);
  return code;
}
int launched(const char* who) {
  const hipError_t e = hipGetLastError();
  return e == hipSuccess ? VMI_HY_OK : fail(VMI_HY_E_HIP, who, hipGetErrorString(e));
}

template <typename T, int BM, int KS>
struct Chunk {
  static constexpr bool DEEP = BM == 16 && sizeof(T) == 2;   // few rows: bytes in flight are what counts
  static constexpr int CS = DEEP && KS < 8 ? 8 : 4;                    // k-steps a wave takes from a chunk
  static constexpr int NB = DEEP ? 3 : 2;                     // chunks of weights in registers, NB - 1 of them ahead
  static constexpr int KC = 32 * CS * KS;                     // columns of x in a chunk
};

// 8 consecutive elements of row m at column k, as they go into LDS
template <typename T, int XK>
struct XUnit;
template <typename T>
struct XUnit<T, VMI_HY_X_ROWS> {
  V8<T> v = zero8<T>();
  __device__ __forceinline__ void load(const vmi_hy_linear_args& p, int64_t row, int64_t goff, int k) {
    v = load8(static_cast<const T*>(p.x) + goff + row * p.ldx + k);
  }
  __device__ __forceinline__ V8<T> finish(const float*, int, float, float) const { return v; }
};
template <typename T>
struct XUnit<T, VMI_HY_X_NORM> {
  f32x8 v = {0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f};
  __device__ __forceinline__ void load(const vmi_hy_linear_args& p, int64_t row, int64_t, int k) {
    v = load8(static_cast<const float*>(p.x) + row * p.ldx + k);
  }
  __device__ __forceinline__ V8<T> finish(const float* nw, int k, float mean, float rstd) const {
    const f32x8 w = load8(nw + k);   // (zero past norm_n: padding columns come out as zeros)
    f32x8 r;
#pragma unroll
    for (int e = 0; e < 8; ++e) r[e] = (v[e] - mean) * rstd * w[e];
    return from_f32<T>(r);
  }
};
template <typename T>
struct XUnit<T, VMI_HY_X_CONCAT> {
  f32x8 v = {0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f};
  __device__ __forceinline__ void load(const vmi_hy_linear_args& p, int64_t row, int64_t, int k) {
    const int half = p.K >> 1;
    const float* src = static_cast<const float*>(k < half ? p.x : p.x2);
    v = load8(src + row * p.ldx + (k < half ? k : k - half));
  }
  __device__ __forceinline__ V8<T> finish(const float*, int, float, float) const { return from_f32<T>(v); }
};

template <typename T, int BM, int NW, int KS, int XK, int EPI>
__global__ __launch_bounds__(NW* KS * 64) void linear_kernel(const vmi_hy_linear_args p) {
  using CK = Chunk<T, BM, KS>;
  constexpr int TH = NW * KS * 64, MT = BM / 16, CS = CK::CS, KC = CK::KC, NB_W = CK::NB;
  constexpr int LD = KC + 16 / (int)sizeof(T), UPR = KC / 8, UPT = BM * UPR / TH;
  static_assert(BM * UPR % TH == 0, "a chunk's units divide over the threads");
  extern __shared__ __attribute__((aligned(16))) unsigned char smem[];
  T* xs = reinterpret_cast<T*>(smem);                                   // [2][BM][LD]
  float* stats = reinterpret_cast<float*>(xs + (size_t)2 * BM * LD);    // [BM][2]
  float* red = stats + 2 * BM;                                          // [KS - 1][NW][MT][64][4]
  // the norm's weight, in LDS: read from memory between the weight tiles it would wait for all of them
  float* nwl = red + (KS - 1) * NW * MT * 256;
  const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6), nw = wave % NW, ks = wave / NW;
  const int kc = lane >> 4, r16 = lane & 15;
  // column blocks are dealt so that all row blocks of one stay on one XCD (workgroups go round-robin over the 8 of them): its
  // weights are read from HBM once
  const int MB = (p.M + BM - 1) / BM, NB = (p.N + 16 * NW - 1) / (16 * NW);
  // (fewer than 8 of them: a plain order, or most XCDs would stay idle)
  const int grp = blockIdx.y;
  const int nb = NB < 8 ? (int)blockIdx.x % NB : (int)(blockIdx.x / (8 * MB)) * 8 + (int)(blockIdx.x & 7);
  const int mb = NB < 8 ? (int)blockIdx.x / NB : (int)(blockIdx.x >> 3) % MB;
  if (nb >= NB) return;
  const int m0 = mb * BM, n0 = (nb * NW + nw) * 16, nks = p.K >> 5;
  const bool nvalid = n0 < p.N;
  const int64_t goff = (int64_t)grp * p.x_gstride;

  const T* wp = static_cast<const T*>(p.w) + (((int64_t)grp * (p.N >> 4) + (nvalid ? n0 >> 4 : 0)) * nks * 64 + lane) * 8;
  const int nchunk = (p.K + KC - 1) / KC;
  V8<T> wb[NB_W][CS];
  auto load_w = [&](V8<T>(&dst)[CS], int c) {
#pragma unroll
    for (int j = 0; j < CS; ++j) {
      // (no lane-wise condition around a load, here or for x: all of a chunk's are in flight together.  A k-step past the last
      //  one reads that one again and meets zeros of x)
      const int k = min(c * (CS * KS) + ks * CS + j, nks - 1);
      dst[j] = load8(wp + (int64_t)k * 512);
    }
  };
#pragma unroll
  for (int b = 0; b < NB_W - 1; ++b) load_w(wb[b], b);

  auto source_row = [&](int m) -> int64_t {
    const int mm = m0 + m < p.M ? m0 + m : p.M - 1;
    if constexpr (XK == VMI_HY_X_NORM) return p.rows ? p.rows[mm] : mm;
    return mm;
  };

  if constexpr (XK == VMI_HY_X_NORM) {   // row statistics, one pass around the row's first element: no cancellation to speak of
    constexpr int NWV = TH / 64;
    const int mrows = min(BM, p.M - m0);
    for (int k = tid * 4; k < p.K; k += TH * 4) *reinterpret_cast<f32x4*>(nwl + k) = *reinterpret_cast<const f32x4*>(p.norm_w + k);
    for (int mbase = wave; mbase < mrows; mbase += 4 * NWV) {
      const float* row[4];
      float sh[4], s[4], q[4];
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int m = mbase + i * NWV < mrows ? mbase + i * NWV : mbase;
        row[i] = static_cast<const float*>(p.x) + source_row(m) * p.ldx;
        sh[i] = p.rms ? 0.f : row[i][0];
        s[i] = q[i] = 0.f;
      }
      for (int k = lane * 4; k < p.K; k += 256) {
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          const f32x4 v = *reinterpret_cast<const f32x4*>(row[i] + k);
#pragma unroll
          for (int e = 0; e < 4; ++e) {
            const float d = k + e < p.norm_n ? v[e] - sh[i] : 0.f;
            s[i] += d;
            q[i] = fmaf(d, d, q[i]);
          }
        }
      }
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const float ms = p.rms ? 0.f : wave_sum(s[i]) / (float)p.norm_n, mq = wave_sum(q[i]) / (float)p.norm_n;
        const int m = mbase + i * NWV;
        if (lane == 0 && m < mrows) {
          stats[2 * m] = sh[i] + ms;
          stats[2 * m + 1] = 1.f / sqrtf(fmaxf(mq - ms * ms, 0.f) + p.eps);
        }
      }
    }
    __syncthreads();
  }

  int64_t srow[UPT];
  int xm[UPT], xk[UPT];
  bool xin[UPT];
  float mean[UPT], rstd[UPT];
#pragma unroll
  for (int i = 0; i < UPT; ++i) {
    const int u = tid + i * TH;
    xm[i] = u / UPR;
    xk[i] = (u % UPR) * 8;
    srow[i] = source_row(xm[i]);
    xin[i] = m0 + xm[i] < p.M;
    mean[i] = rstd[i] = 0.f;
    if (XK == VMI_HY_X_NORM && xin[i]) {
      mean[i] = stats[2 * xm[i]];
      rstd[i] = stats[2 * xm[i] + 1];
    }
  }
  XUnit<T, XK> xu[UPT];
  auto load_x = [&](int c) {
#pragma unroll
    for (int i = 0; i < UPT; ++i)   // (a wave whose rows all lie past M reads none: a scalar condition)
      if ((wave * 64 + i * TH) / UPR < p.M - m0) xu[i].load(p, srow[i], goff, min(c * KC + xk[i], p.K - 8));
  };
  load_x(0);

  f32x4 acc[MT];
#pragma unroll
  for (int mi = 0; mi < MT; ++mi) acc[mi] = f32x4{0.f, 0.f, 0.f, 0.f};
  auto step = [&](int c, V8<T>(&cur)[CS], V8<T>(&nxt)[CS]) {
    T* dst = xs + (size_t)(c & 1) * BM * LD;
#pragma unroll
    for (int u = 0; u < UPT; ++u) {
      const int k = c * KC + xk[u];
      const V8<T> v = xu[u].finish(nwl, min(k, p.K - 8), mean[u], rstd[u]);
      *reinterpret_cast<V8<T>*>(dst + xm[u] * LD + xk[u]) = xin[u] && k < p.K ? v : zero8<T>();
    }
    // x first, and the weights whatever is left (past the end: one tile again, a cache hit): a wait for x then always knows how
    // many younger loads it may leave in flight
    if (c + 1 < nchunk) load_x(c + 1);
    load_w(nxt, c + NB_W - 1);
    __syncthreads();   // (two buffers: the writes of chunk c + 1 go where chunk c - 1 was read, which every wave has left behind)
#pragma unroll
    for (int j = 0; j < CS; ++j)
#pragma unroll
      for (int mi = 0; mi < MT; ++mi) mma(acc[mi], cur[j], load8(dst + (mi * 16 + r16) * LD + (ks * CS + j) * 32 + 8 * kc));
  };
  for (int c = 0; c < nchunk; c += NB_W) {   // chunk c sits in wb[c % NB_W]; the one behind it has been used up
#pragma unroll
    for (int b = 0; b < NB_W; ++b)
      if (c + b < nchunk) step(c + b, wb[b], wb[(b + NB_W - 1) % NB_W]);
  }

  if constexpr (KS > 1) {
    if (ks > 0) {
#pragma unroll
      for (int mi = 0; mi < MT; ++mi)
        *reinterpret_cast<f32x4*>(red + ((((ks - 1) * NW + nw) * MT + mi) * 64 + lane) * 4) = acc[mi];
    }
    __syncthreads();
    if (ks > 0) return;
#pragma unroll
    for (int s = 1; s < KS; ++s)
#pragma unroll
      for (int mi = 0; mi < MT; ++mi)
        acc[mi] += *reinterpret_cast<const f32x4*>(red + ((((s - 1) * NW + nw) * MT + mi) * 64 + lane) * 4);
  }
  if (!nvalid) return;

  const int n = n0 + 4 * kc;
#pragma unroll
  for (int mi = 0; mi < MT; ++mi) {
    const int m = m0 + mi * 16 + r16;
    if (m >= p.M) continue;
    const int64_t yoff = (int64_t)m * p.ldy + (int64_t)grp * p.y_gstride;
    if constexpr (EPI == VMI_HY_E_STORE) {
      f32x4 b = f32x4{0.f, 0.f, 0.f, 0.f};
      if (p.bias) b = *reinterpret_cast<const f32x4*>(p.bias + n);
      V4<T> o;
#pragma unroll
      for (int r = 0; r < 4; ++r) o[r] = (T)(acc[mi][r] + b[r]);
      *reinterpret_cast<V4<T>*>(static_cast<T*>(p.y) + yoff + n) = o;
    } else if constexpr (EPI == VMI_HY_E_RESIDUAL) {
      f32x4* y = reinterpret_cast<f32x4*>(static_cast<float*>(p.y) + yoff + n);
      *y = *y + acc[mi];
    } else if constexpr (EPI == VMI_HY_E_FLOAT) {
      float* y = static_cast<float*>(p.y) + yoff + n;
      if (n + 4 <= p.n_out && (p.ldy & 3) == 0) {
        *reinterpret_cast<f32x4*>(y) = acc[mi] * p.scale;
      } else {
#pragma unroll
        for (int r = 0; r < 4; ++r)
          if (n + r < p.n_out) y[r] = acc[mi][r] * p.scale;
      }
    } else if constexpr (EPI == VMI_HY_E_GLU) {
      typename Elem<T>::v2 o;
      o[0] = (T)glu(acc[mi][0], acc[mi][1], p.scale, p.glu_alpha, p.glu_up);
      o[1] = (T)glu(acc[mi][2], acc[mi][3], p.scale, p.glu_alpha, p.glu_up);
      *reinterpret_cast<typename Elem<T>::v2*>(static_cast<T*>(p.y) + yoff + (n >> 1)) = o;
    } else if constexpr (EPI == VMI_HY_E_STORE_GLU) {
      if (n0 < p.n_split) {
        V4<T> o;
#pragma unroll
        for (int r = 0; r < 4; ++r) o[r] = (T)acc[mi][r];
        *reinterpret_cast<V4<T>*>(static_cast<T*>(p.y) + yoff + n) = o;
      } else {
        typename Elem<T>::v2 o;
        o[0] = (T)glu(acc[mi][0], acc[mi][1], p.scale, p.glu_alpha, p.glu_up);
        o[1] = (T)glu(acc[mi][2], acc[mi][3], p.scale, p.glu_alpha, p.glu_up);
        *reinterpret_cast<typename Elem<T>::v2*>(static_cast<T*>(p.y2) + (int64_t)m * p.ldy2 + ((n - p.n_split) >> 1)) = o;
      }
    } else {   // VMI_HY_E_GATED
      const float g = sigmoid((float)static_cast<const T*>(p.gate)[(int64_t)m * p.ldg + grp]);
      V4<T> o;
#pragma unroll
      for (int r = 0; r < 4; ++r) o[r] = (T)(acc[mi][r] * g);
      *reinterpret_cast<V4<T>*>(static_cast<T*>(p.y) + yoff + n) = o;
    }
  }
}

template <typename T, int BM, int NW, int KS, int XK, int EPI>
static int launch_linear(const vmi_hy_linear_args& p, hipStream_t st) {
  constexpr int KC = Chunk<T, BM, KS>::KC, LD = KC + 16 / (int)sizeof(T);
  const size_t lds = (size_t)2 * BM * LD * sizeof(T) + 2 * BM * 4 + (size_t)(KS - 1) * NW * (BM / 16) * 64 * 16 +
                     (XK == VMI_HY_X_NORM ? (size_t)p.K * 4 : 0);
  auto* fn = linear_kernel<T, BM, NW, KS, XK, EPI>;
  if (int rc = allow_lds(fn, lds, "vmi_hy_linear")) return rc;
  const int MB = (p.M + BM - 1) / BM, NB = (p.N + 16 * NW - 1) / (16 * NW);
  hipLaunchKernelGGL(fn, dim3((NB < 8 ? NB : (NB + 7) / 8 * 8) * MB, p.groups), dim3(NW * KS * 64), lds, st, p);
  return launched("vmi_hy_linear");
}

template <typename T, int XK, int EPI>
static int linear_shape(const vmi_hy_linear_args& p, hipStream_t st) {
  // few rows: 16-row tiles; a layer with few columns splits K over the waves of a workgroup so that all compute units read
  const int64_t slabs = (int64_t)(p.N / 16) * p.groups;
  if (p.M <= 32) {
    const int64_t wgs = slabs * ((p.M + 15) / 16);
    if (wgs >= 2048) return launch_linear<T, 16, 4, 1, XK, EPI>(p, st);
    if (wgs >= 400 || p.K < 256) return launch_linear<T, 16, 2, 2, XK, EPI>(p, st);
    if constexpr (sizeof(T) == 2)
      if (wgs < 192 && p.K >= 1024) return launch_linear<T, 16, 1, 8, XK, EPI>(p, st);
    return launch_linear<T, 16, 1, 4, XK, EPI>(p, st);
  }
  if (p.M <= 96 || slabs / 4 * ((p.M + 63) / 64) < 256) return launch_linear<T, 32, 4, 1, XK, EPI>(p, st);
  return launch_linear<T, 64, 4, 1, XK, EPI>(p, st);
}

template <typename T>
static int linear_kind(const vmi_hy_linear_args& p, hipStream_t st) {
  switch (p.x_kind * 8 + p.epilogue) {
    case VMI_HY_X_ROWS * 8 + VMI_HY_E_STORE: return linear_shape<T, VMI_HY_X_ROWS, VMI_HY_E_STORE>(p, st);
    case VMI_HY_X_ROWS * 8 + VMI_HY_E_RESIDUAL: return linear_shape<T, VMI_HY_X_ROWS, VMI_HY_E_RESIDUAL>(p, st);
    case VMI_HY_X_ROWS * 8 + VMI_HY_E_GATED: return linear_shape<T, VMI_HY_X_ROWS, VMI_HY_E_GATED>(p, st);
    case VMI_HY_X_NORM * 8 + VMI_HY_E_STORE: return linear_shape<T, VMI_HY_X_NORM, VMI_HY_E_STORE>(p, st);
    case VMI_HY_X_NORM * 8 + VMI_HY_E_FLOAT: return linear_shape<T, VMI_HY_X_NORM, VMI_HY_E_FLOAT>(p, st);
    case VMI_HY_X_NORM * 8 + VMI_HY_E_GLU: return linear_shape<T, VMI_HY_X_NORM, VMI_HY_E_GLU>(p, st);
    case VMI_HY_X_NORM * 8 + VMI_HY_E_STORE_GLU: return linear_shape<T, VMI_HY_X_NORM, VMI_HY_E_STORE_GLU>(p, st);
    case VMI_HY_X_CONCAT * 8 + VMI_HY_E_FLOAT: return linear_shape<T, VMI_HY_X_CONCAT, VMI_HY_E_FLOAT>(p, st);
    default: return fail(VMI_HY_E_ARG, "vmi_hy_linear", "this combination of input and epilogue is not built");
  }
}

// ---- elementwise ends ---------------------------------------------------------------------------------------------------------
__global__ __launch_bounds__(256) void embed_kernel(const int64_t* __restrict__ ids, const b16* __restrict__ table,
                                                    float* __restrict__ x, int width, int ld, int vocab, float scale) {
  const int t = blockIdx.x;
  int64_t id = ids[t];
  if (id < 0 || id >= vocab) id = 0;   // (ids are checked on the host; sampled ones are in range by construction)
  for (int k = threadIdx.x * 4; k < ld; k += 1024) {
    f32x4 o;
#pragma unroll
    for (int e = 0; e < 4; ++e) o[e] = k + e < width ? (float)table[id * (int64_t)ld + k + e] * scale : 0.f;
    *reinterpret_cast<f32x4*>(x + (int64_t)t * ld + k) = o;
  }
}

// one workgroup per row; a row of up to 4 * 4096 columns stays in registers between the three passes
template <typename T>
__global__ __launch_bounds__(256) void add_norm_kernel(float* x, const T* add, int64_t ld_add, const float* norm_w, T* out, int n,
                                                       int ld, float eps, int rms) {
  __shared__ float part[2][4];
  const int t = blockIdx.x, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  float* row = x + (int64_t)t * ld;
  constexpr int MAXV = 8;
  f32x4 v[MAXV];
  float s = 0.f;
  auto fetch = [&](int k) {
    f32x4 a = *reinterpret_cast<const f32x4*>(row + k);
    if (add) {
      const V4<T> d = *reinterpret_cast<const V4<T>*>(add + (int64_t)t * ld_add + k);
#pragma unroll
      for (int e = 0; e < 4; ++e) a[e] += (float)d[e];
      *reinterpret_cast<f32x4*>(row + k) = a;
    }
    return a;
  };
#pragma unroll
  for (int i = 0; i < MAXV; ++i) {
    const int k = (tid + i * 256) * 4;
    v[i] = f32x4{0.f, 0.f, 0.f, 0.f};
    if (k < ld) v[i] = fetch(k);
    s += v[i][0] + v[i][1] + v[i][2] + v[i][3];   // (padding columns are zeros)
  }
  for (int k = (tid + MAXV * 256) * 4; k < ld; k += 1024) {
    const f32x4 a = fetch(k);
    s += a[0] + a[1] + a[2] + a[3];
  }
  if (!out) return;
  float mean = 0.f;
  if (!rms) {
    s = wave_sum(s);
    if (lane == 0) part[0][wave] = s;
    __syncthreads();
    mean = (part[0][0] + part[0][1] + part[0][2] + part[0][3]) / (float)n;
  }
  float q = 0.f;
  auto dev2 = [&](const f32x4& a, int k) {
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const float d = k + e < n ? a[e] - mean : 0.f;
      q = fmaf(d, d, q);
    }
  };
#pragma unroll
  for (int i = 0; i < MAXV; ++i) dev2(v[i], (tid + i * 256) * 4);
  for (int k = (tid + MAXV * 256) * 4; k < ld; k += 1024) dev2(*reinterpret_cast<const f32x4*>(row + k), k);
  q = wave_sum(q);
  if (lane == 0) part[1][wave] = q;
  __syncthreads();
  const float rstd = 1.f / sqrtf((part[1][0] + part[1][1] + part[1][2] + part[1][3]) / (float)n + eps);
  auto put = [&](const f32x4& a, int k) {
    const f32x4 w = *reinterpret_cast<const f32x4*>(norm_w + k);
    V4<T> o;
#pragma unroll
    for (int e = 0; e < 4; ++e) o[e] = (T)((a[e] - mean) * rstd * w[e]);
    *reinterpret_cast<V4<T>*>(out + (int64_t)t * ld + k) = o;
  };
#pragma unroll
  for (int i = 0; i < MAXV; ++i) {
    const int k = (tid + i * 256) * 4;
    if (k < ld) put(v[i], k);
  }
  for (int k = (tid + MAXV * 256) * 4; k < ld; k += 1024) put(*reinterpret_cast<const f32x4*>(row + k), k);
}

// x += scale (rms norm of a + rms norm of b) + add; one workgroup per row
template <typename T>
__global__ __launch_bounds__(256) void merge_kernel(float* x, const T* a, int64_t ld_a, const T* b, int64_t ld_b, const T* add,
                                                    int64_t ld_add, const float* wa, const float* wb, int n, int ld, float eps,
                                                    float scale) {
  __shared__ float part[2][4];
  const int t = blockIdx.x, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  a += (int64_t)t * ld_a;
  b += (int64_t)t * ld_b;
  float sa = 0.f, sb = 0.f;
  for (int k = tid * 4; k < ld; k += 1024) {   // (padding columns are zeros)
    const V4<T> va = *reinterpret_cast<const V4<T>*>(a + k), vb = *reinterpret_cast<const V4<T>*>(b + k);
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      sa = fmaf((float)va[e], (float)va[e], sa);
      sb = fmaf((float)vb[e], (float)vb[e], sb);
    }
  }
  sa = wave_sum(sa);
  sb = wave_sum(sb);
  if (lane == 0) part[0][wave] = sa, part[1][wave] = sb;
  __syncthreads();
  const float ra = scale / sqrtf((part[0][0] + part[0][1] + part[0][2] + part[0][3]) / (float)n + eps);
  const float rb = scale / sqrtf((part[1][0] + part[1][1] + part[1][2] + part[1][3]) / (float)n + eps);
  float* row = x + (int64_t)t * ld;
  for (int k = tid * 4; k < ld; k += 1024) {
    const V4<T> va = *reinterpret_cast<const V4<T>*>(a + k), vb = *reinterpret_cast<const V4<T>*>(b + k);
    const f32x4 w0 = *reinterpret_cast<const f32x4*>(wa + k), w1 = *reinterpret_cast<const f32x4*>(wb + k);
    f32x4 v = *reinterpret_cast<const f32x4*>(row + k);
    if (add) {
      const V4<T> d = *reinterpret_cast<const V4<T>*>(add + (int64_t)t * ld_add + k);
#pragma unroll
      for (int e = 0; e < 4; ++e) v[e] += (float)d[e];
    }
#pragma unroll
    for (int e = 0; e < 4; ++e) v[e] += (float)va[e] * ra * w0[e] + (float)vb[e] * rb * w1[e];
    *reinterpret_cast<f32x4*>(row + k) = v;
  }
}

// out [T, 2 n] = (x | x2) in the element type
template <typename T>
__global__ __launch_bounds__(256) void concat_kernel(const float* __restrict__ x, const float* __restrict__ x2, T* __restrict__ out, int n) {
  const int t = blockIdx.y, j = (blockIdx.x * 256 + threadIdx.x) * 8;
  if (j >= 2 * n) return;
  *reinterpret_cast<V8<T>*>(out + (int64_t)t * 2 * n + j) = from_f32<T>(load8((j < n ? x + j : x2 + j - n) + (int64_t)t * n));
}

template <typename T>
__global__ __launch_bounds__(256) void glu_kernel(const T* __restrict__ in, int64_t ld_in, T* __restrict__ out, int64_t ld_out, int n,
                                                  float limit, float alpha, float up) {
  const int t = blockIdx.y, j = (blockIdx.x * 256 + threadIdx.x) * 4;
  if (j >= n) return;
  const V8<T> v = load8(in + (int64_t)t * ld_in + 2 * j);
  V4<T> o;
#pragma unroll
  for (int e = 0; e < 4; ++e) o[e] = (T)glu((float)v[2 * e], (float)v[2 * e + 1], limit, alpha, up);
  *reinterpret_cast<V4<T>*>(out + (int64_t)t * ld_out + j) = o;
}

__global__ __launch_bounds__(1024) void argmax_kernel(const float* __restrict__ logits, int64_t ld, int V, int64_t* __restrict__ out) {
  __shared__ float sb[16];
  __shared__ int si[16];
  const float* row = logits + (int64_t)blockIdx.x * ld;
  float best = -INFINITY;
  int at = 0x7fffffff;
  auto take = [&](float v, int i) {
    if (v > best || (v == best && i < at)) {
      best = v;
      at = i;
    }
  };
  for (int i = threadIdx.x; i < V; i += 1024) take(row[i], i);
#pragma unroll
  for (int o = 32; o > 0; o >>= 1) {
    const float ob = __shfl_xor(best, o, 64);
    const int oi = __shfl_xor(at, o, 64);
    take(ob, oi);
  }
  if ((threadIdx.x & 63) == 0) {
    sb[threadIdx.x >> 6] = best;
    si[threadIdx.x >> 6] = at;
  }
  __syncthreads();
  if (threadIdx.x == 0) {
    for (int w = 1; w < 16; ++w) take(sb[w], si[w]);
    out[blockIdx.x] = at == 0x7fffffff ? 0 : at;
  }
}

}  // namespace vmi_hybrid

using namespace vmi_hybrid;

extern "C" {

int vmi_hy_linear(const vmi_hy_linear_args* a, void* stream) {
  static const char* who = "vmi_hy_linear";
  if (!a || !a->x || !a->w || !a->y || a->M <= 0 || a->N <= 0 || a->K <= 0 || a->groups <= 0 || a->dtype < 0 || a->dtype > 1 ||
      (a->x_kind == VMI_HY_X_NORM && (!a->norm_w || a->norm_n <= 0 || a->norm_n > a->K)) || (a->x_kind == VMI_HY_X_CONCAT && !a->x2) ||
      (a->epilogue == VMI_HY_E_GATED && !a->gate) || (a->epilogue == VMI_HY_E_STORE_GLU && !a->y2))
    return fail(VMI_HY_E_ARG, who, "null pointer, non-positive size or unknown element type");
  if ((a->K & 31) || (a->N & 15) || (a->x_kind == VMI_HY_X_CONCAT && (a->K & 63)) || (a->ldx & 7) || (a->x_gstride & 7) ||
      (a->epilogue != VMI_HY_E_FLOAT && ((a->ldy & 3) || (a->y_gstride & 3))) || ((uintptr_t)a->x & 15) || ((uintptr_t)a->w & 15) ||
      ((uintptr_t)a->y & 15) || (a->epilogue == VMI_HY_E_FLOAT && (a->n_out <= 0 || a->n_out > a->N || a->groups != 1)) ||
      (a->epilogue == VMI_HY_E_STORE_GLU && (a->n_split < 0 || a->n_split > a->N || (a->n_split & 15) || (a->ldy2 & 1) ||
                                             ((uintptr_t)a->y2 & 7) || a->groups != 1)))
    return fail(VMI_HY_E_SHAPE, who, "needs K % 32 == 0, N % 16 == 0 and 16-byte aligned rows");
  DeviceScope dev(a->device);
  if (!dev.ok) return fail(VMI_HY_E_HIP, who, "hipSetDevice failed");
  hipStream_t st = static_cast<hipStream_t>(stream);
  return a->dtype == VMI_HY_BF16 ? linear_kind<b16>(*a, st) : linear_kind<float>(*a, st);
}

int vmi_hy_embed(const int64_t* ids, const void* table, float* x, int32_t T, int32_t width, int32_t ld, int32_t vocab, float scale,
                 int32_t device, void* stream) {
  static const char* who = "vmi_hy_embed";
  if (!ids || !table || !x || T <= 0 || width <= 0 || ld < width || (ld & 3) || vocab <= 0) return fail(VMI_HY_E_ARG, who, "bad argument");
  DeviceScope dev(device);
  if (!dev.ok) return fail(VMI_HY_E_HIP, who, "hipSetDevice failed");
  hipLaunchKernelGGL(embed_kernel, dim3(T), dim3(256), 0, static_cast<hipStream_t>(stream), ids, static_cast<const b16*>(table), x,
                     width, ld, vocab, scale);
  return launched(who);
}

int vmi_hy_add_norm(float* x, const void* add, int64_t ld_add, const float* norm_w, void* out, int32_t T, int32_t n, int32_t ld,
                    float eps, int32_t rms, int32_t dtype, int32_t device, void* stream) {
  static const char* who = "vmi_hy_add_norm";
  if (!x || T <= 0 || n <= 0 || ld < n || (ld & 3) || (add && (ld_add & 3)) || (out && !norm_w)) return fail(VMI_HY_E_ARG, who, "bad argument");
  DeviceScope dev(device);
  if (!dev.ok) return fail(VMI_HY_E_HIP, who, "hipSetDevice failed");
  hipStream_t st = static_cast<hipStream_t>(stream);
  if (dtype == VMI_HY_BF16)
    hipLaunchKernelGGL(add_norm_kernel<b16>, dim3(T), dim3(256), 0, st, x, static_cast<const b16*>(add), ld_add, norm_w,
                       static_cast<b16*>(out), n, ld, eps, rms);
  else
    hipLaunchKernelGGL(add_norm_kernel<float>, dim3(T), dim3(256), 0, st, x, static_cast<const float*>(add), ld_add, norm_w,
                       static_cast<float*>(out), n, ld, eps, rms);
  return launched(who);
}

int vmi_hy_glu(const void* in, int64_t ld_in, void* out, int64_t ld_out, int32_t T, int32_t n, float limit, float alpha,
               float up, int32_t dtype, int32_t device, void* stream) {
  static const char* who = "vmi_hy_glu";
  if (!in || !out || T <= 0 || T > 65535 || n <= 0 || (n & 3) || (ld_in & 7) || (ld_out & 3)) return fail(VMI_HY_E_ARG, who, "bad argument");
  DeviceScope dev(device);
  if (!dev.ok) return fail(VMI_HY_E_HIP, who, "hipSetDevice failed");
  hipStream_t st = static_cast<hipStream_t>(stream);
  const dim3 grid((n / 4 + 255) / 256, T);
  if (dtype == VMI_HY_BF16)
    hipLaunchKernelGGL(glu_kernel<b16>, grid, dim3(256), 0, st, static_cast<const b16*>(in), ld_in, static_cast<b16*>(out), ld_out, n,
                       limit, alpha, up);
  else
    hipLaunchKernelGGL(glu_kernel<float>, grid, dim3(256), 0, st, static_cast<const float*>(in), ld_in, static_cast<float*>(out), ld_out, n,
                       limit, alpha, up);
  return launched(who);
}

int vmi_hy_merge(float* x, const void* a, int64_t ld_a, const void* b, int64_t ld_b, const void* add, int64_t ld_add, const float* wa,
                 const float* wb, int32_t T, int32_t n, int32_t ld, float eps, float scale, int32_t dtype, int32_t device,
                 void* stream) {
  static const char* who = "vmi_hy_merge";
  if (!x || !a || !b || !wa || !wb || T <= 0 || n <= 0 || ld < n || (ld & 3) || (ld_a & 3) || (ld_b & 3) || (add && (ld_add & 3)))
    return fail(VMI_HY_E_ARG, who, "bad argument");
  DeviceScope dev(device);
  if (!dev.ok) return fail(VMI_HY_E_HIP, who, "hipSetDevice failed");
  hipStream_t st = static_cast<hipStream_t>(stream);
  if (dtype == VMI_HY_BF16)
    hipLaunchKernelGGL(merge_kernel<b16>, dim3(T), dim3(256), 0, st, x, static_cast<const b16*>(a), ld_a, static_cast<const b16*>(b), ld_b,
                       static_cast<const b16*>(add), ld_add, wa, wb, n, ld, eps, scale);
  else
    hipLaunchKernelGGL(merge_kernel<float>, dim3(T), dim3(256), 0, st, x, static_cast<const float*>(a), ld_a, static_cast<const float*>(b),
                       ld_b, static_cast<const float*>(add), ld_add, wa, wb, n, ld, eps, scale);
  return launched(who);
}

int vmi_hy_concat(const float* x, const float* x2, void* out, int32_t T, int32_t n, int32_t dtype, int32_t device, void* stream) {
  static const char* who = "vmi_hy_concat";
  if (!x || !x2 || !out || T <= 0 || T > 65535 || n <= 0 || (n & 7)) return fail(VMI_HY_E_ARG, who, "bad argument");
  DeviceScope dev(device);
  if (!dev.ok) return fail(VMI_HY_E_HIP, who, "hipSetDevice failed");
  hipStream_t st = static_cast<hipStream_t>(stream);
  const dim3 grid((2 * n / 8 + 255) / 256, T);
  if (dtype == VMI_HY_BF16)
    hipLaunchKernelGGL(concat_kernel<b16>, grid, dim3(256), 0, st, x, x2, static_cast<b16*>(out), n);
  else
    hipLaunchKernelGGL(concat_kernel<float>, grid, dim3(256), 0, st, x, x2, static_cast<float*>(out), n);
  return launched(who);
}

int vmi_hy_argmax(const float* logits, int64_t ld, int32_t rows, int32_t V, int64_t* out, int32_t device, void* stream) {
  static const char* who = "vmi_hy_argmax";
  if (!logits || !out || rows <= 0 || V <= 0 || ld < V) return fail(VMI_HY_E_ARG, who, "bad argument");
  DeviceScope dev(device);
  if (!dev.ok) return fail(VMI_HY_E_HIP, who, "hipSetDevice failed");
  hipLaunchKernelGGL(argmax_kernel, dim3(rows), dim3(1024), 0, static_cast<hipStream_t>(stream), logits, ld, V, out);
  return launched(who);
}

const char* vmi_hybrid_last_error(void) { return g_err.c_str(); }
int32_t vmi_hybrid_abi_version(void) { return VMI_HYBRID_ABI_VERSION; }
const char* vmi_hybrid_target_arch(void) { return "gfx950"; }

}  // extern "C"
