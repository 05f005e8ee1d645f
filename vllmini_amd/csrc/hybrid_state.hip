// Linear attention with a matrix state per head (include/vmi_hybrid.h): retention (fixed decay per head, rotated q and k) and the
// gated delta rule (decay per head and key channel, short convolutions, unit q and k).  All of it is fp32 from the projections on.
//
// Portions: cut into chunks of 16 rows.  With G_i the decay accumulated from the chunk's start through row i (log), the rows obey
//     u_i + beta_i sum_{j<i} A_ij u_j = beta_i (v_i - S^T k_i e^{G_i}),    A_ij = sum_c k_ic k_jc e^{G_ic - G_jc}
//     o_i = S^T (q_i e^{G_i}) + sum_{j<=i} B_ij u_j,                       B_ij = sum_c q_ic k_jc e^{G_ic - G_jc}
//     S  <- e^{G_15} S + sum_j (k_j e^{G_15 - G_j}) u_j^T
// (retention: u = v, no A).  state_prep_kernel makes, for every (chunk, head) independently, the triangular system's solutions
// W = (I + beta A)^-1 beta (k e^G) and U0 = (I + beta A)^-1 beta v, q e^G, k e^{G_15 - G} and B; exponents are always of differences
// i >= j, so nothing can overflow (where a chunk decays little, products of e^{G_i} and e^{-G_j} on the matrix cores instead).
// state_scan_kernel then walks a state's chunks: u = U0 - W S, o = q e^G S + B u, S update, on v_mfma_f32_16x16x4_f32.  A workgroup
// owns 16 value columns of one head's state for the whole walk, each wave some of its rows, in the matrix core's result layout
// (lane (kc, r16): rows 4 kc + r of column r16), which is at the same time the operand layout of the next product.  What the waves
// exchange per chunk is their part of W S and, a chunk later, of o (16 x 16 each, one barrier); the operands of the next chunks are in
// flight meanwhile, and rows past a portion's end are zeros in all of them.
//
// Steps of single tokens: state_step_kernel reads each state once, keeps it in registers between the correction and the read-out,
// and writes it back; convolution, gates, norm and output gate ride along.
#include "hybrid_common.hpp"

namespace vmi_hybrid {

constexpr int CH = 16;        // rows of a chunk
constexpr int MAX_TAPS = 16;

__device__ __forceinline__ float softplus(float z) { return fmaxf(z, 0.f) + log1pf(expf(-fabsf(z))); }

struct Portion {
  int qs, len, ctx, slot, flip;
};
__device__ __forceinline__ Portion portion(const vmi_hy_step& s, int e) {
  return Portion{s.q_start[e], s.q_len[e], s.ctx[e], s.state_slot[e], s.flip[e]};
}

// 8 channels from channel c of the token in packed row t, through the convolution and silu.  TAPS = 0: any number of taps
template <typename T, int TAPS>
__device__ __forceinline__ f32x8 conv_silu8(const vmi_hy_state_args& p, const Portion& r, int C, int t, int c) {
  f32x8 acc = {0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f};
  const T* in = static_cast<const T*>(p.proj) + c;
  const int taps = TAPS ? TAPS : p.taps, pos = r.ctx + t - r.qs;
  const T* tail = static_cast<const T*>(p.tail) + ((int64_t)r.slot * 2 + r.flip) * (taps - 1) * C + c;   // positions ctx - (taps - 1) ..
  auto tap = [&](int j) {
    const int back = taps - 1 - j;
    const T* src = t - back >= r.qs ? in + (int64_t)(t - back) * p.ldp
                   : pos >= back    ? tail + (int64_t)(pos - back - (r.ctx - (taps - 1))) * C
                                    : in + (int64_t)t * p.ldp;
    const V8<T> v = load8(src);
    const f32x8 w = load8(p.conv_w + (int64_t)j * C + c);
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
#pragma unroll
  for (int e = 0; e < 8; ++e) acc[e] = silu(acc[e]);
  return acc;
}

// the last taps - 1 inputs of an entry, channels [c0, c0 + n), into the half of the tail this step does not read
template <typename T>
__device__ __forceinline__ void write_tail(const vmi_hy_state_args& p, const Portion& r, int C, int c0, int n, int tid, int threads) {
  const int nt = p.taps - 1, per = n >> 3;
  const T* from = static_cast<const T*>(p.tail) + ((int64_t)r.slot * 2 + r.flip) * nt * C;
  T* to = static_cast<T*>(p.tail) + ((int64_t)r.slot * 2 + (r.flip ^ 1)) * nt * C;
  for (int u = tid; u < nt * per; u += threads) {
    const int e = u / per, c = c0 + (u - e * per) * 8, pos = r.ctx + r.len - nt + e;   // the position this row stands for
    V8<T> v = zero8<T>();
    if (pos >= r.ctx) v = load8(static_cast<const T*>(p.proj) + (int64_t)(r.qs + pos - r.ctx) * p.ldp + c);
    else if (pos >= 0) v = load8(from + (int64_t)(pos - (r.ctx - nt)) * C + c);
    *reinterpret_cast<V8<T>*>(to + (int64_t)e * C + c) = v;
  }
}

// cos, sin of position * frequency, the angle reduced in fp64: exact to fp32 at any position.  One row per token
__global__ __launch_bounds__(64) void rotations_kernel(const double* __restrict__ freq, int half, float* __restrict__ out,
                                                       const int* __restrict__ tok_pos) {
  const int t = blockIdx.x;
  const double pos = (double)tok_pos[t];
  for (int i = threadIdx.x; i < half; i += 64) {
    const double a = pos * freq[i];
    const float r = (float)(a - 6.283185307179586476925 * rint(a * 0.15915494309189533577));
    *reinterpret_cast<f32x2*>(out + ((int64_t)t * half + i) * 2) = f32x2{cosf(r), sinf(r)};
  }
}

// q and k of one head in packed row t, rotated, k / sqrt(dim_n), into LDS rows: the share of lane l of L
template <typename T>
__device__ __forceinline__ void rotated_row(const vmi_hy_state_args& p, int t, int hk, float* ql, float* kl, int l, int L) {
  const int half = p.rot_n >> 1;
  const float ks = 1.f / sqrtf((float)p.dim_n);
  const T* qr = static_cast<const T*>(p.proj) + (int64_t)t * p.ldp + (int64_t)hk * p.dim;
  const T* kr = qr + (int64_t)p.kv_heads * p.dim;
  const float* cs = p.turns + (int64_t)t * half * 2;
  if ((half & 3) == 0) {   // four pairs at a time
    for (int i = 4 * l; i < half; i += 4 * L) {
      const V4<T> qa = *reinterpret_cast<const V4<T>*>(qr + i), qb = *reinterpret_cast<const V4<T>*>(qr + i + half);
      const V4<T> ka = *reinterpret_cast<const V4<T>*>(kr + i), kb = *reinterpret_cast<const V4<T>*>(kr + i + half);
      const f32x8 c = load8(cs + 2 * i);
      f32x4 q0, q1, k0, k1;
#pragma unroll
      for (int x = 0; x < 4; ++x) {
        const float co = c[2 * x], si = c[2 * x + 1];
        q0[x] = (float)qa[x] * co - (float)qb[x] * si;
        q1[x] = (float)qb[x] * co + (float)qa[x] * si;
        k0[x] = ((float)ka[x] * co - (float)kb[x] * si) * ks;
        k1[x] = ((float)kb[x] * co + (float)ka[x] * si) * ks;
      }
      *reinterpret_cast<f32x4*>(ql + i) = q0;
      *reinterpret_cast<f32x4*>(ql + i + half) = q1;
      *reinterpret_cast<f32x4*>(kl + i) = k0;
      *reinterpret_cast<f32x4*>(kl + i + half) = k1;
    }
  } else {
    for (int i = l; i < half; i += L) {
      const float qa = (float)qr[i], qb = (float)qr[i + half], ka = (float)kr[i], kb = (float)kr[i + half];
      const float co = cs[2 * i], si = cs[2 * i + 1];
      ql[i] = qa * co - qb * si;
      ql[i + half] = qb * co + qa * si;
      kl[i] = (ka * co - kb * si) * ks;
      kl[i + half] = (kb * co + ka * si) * ks;
    }
  }
  for (int i = p.rot_n + l; i < p.dim; i += L) {   // passes unrotated (padding: zeros)
    ql[i] = (float)qr[i];
    kl[i] = (float)kr[i] * ks;
  }
}

__device__ __forceinline__ void mma4(f32x4& acc, const f32x4& a, const f32x4& b) {
#pragma unroll
  for (int r = 0; r < 4; ++r) acc = __builtin_amdgcn_mfma_f32_16x16x4f32(a[r], b[r], acc, 0, 0, 0);
}

// this wave's part (every fourth 16 channels) of the 16 x 16 products of LDS rows a and b
__device__ __forceinline__ f32x4 row_products(const float* a, const float* b, int ld, int dim, int wave, int lane) {
  const int at = (lane & 15) * ld + 4 * (lane >> 4);
  f32x4 acc = f32x4{0.f, 0.f, 0.f, 0.f};
  for (int c = 16 * wave; c < dim; c += 64)
    mma4(acc, *reinterpret_cast<const f32x4*>(a + at + c), *reinterpret_cast<const f32x4*>(b + at + c));
  return acc;
}
// ... and its place: part[wave][16][20], row i = 4 kc + r, column j
__device__ __forceinline__ void put_products(float* part, const f32x4& v, int wave, int lane) {
#pragma unroll
  for (int r = 0; r < 4; ++r) part[(wave * CH + 4 * (lane >> 4) + r) * 20 + (lane & 15)] = v[r];
}
__device__ __forceinline__ float sum_products(const float* part, int i, int j) {
  const float* v = part + i * 20 + j;
  return (v[0] + v[CH * 20]) + (v[2 * CH * 20] + v[3 * CH * 20]);
}

// what one (chunk, head) hands to the walk, in floats
struct Scratch {
  int q, w, k, u, b, d, o, size;
  __host__ __device__ Scratch(int kind, int dim, int vdim) {
    q = 0;                                                // [16][dim]   q e^G
    w = q + CH * dim;                                     // [16][dim]   W (delta only)
    k = w + (kind == VMI_HY_DELTA ? CH * dim : 0);        // [dim][16]   k e^{G_15 - G}
    u = k + CH * dim;                                     // [vdim][16]  U0
    b = u + CH * vdim;                                    // [16][16]    B
    d = b + CH * CH;                                      // [dim]       e^{G_15}
    o = d + dim;                                          // [16][vdim]  what the walk leaves: o
    size = o + CH * vdim;
  }
};

inline size_t prep_lds(int kind, int dim, int vdim) {
  const bool delta = kind == VMI_HY_DELTA;
  return ((size_t)CH * (dim + 4) * (delta ? 3 : 2) + (size_t)CH * (vdim + 4) + (size_t)(delta ? 9 : 4) * CH * 20 + 2 * CH + (delta ? dim : 0)) *
         sizeof(float);
}

constexpr float LITTLE_DECAY = 24.f;   // a chunk whose channels decay by at most e^-24 takes the matrix cores for A and B

template <typename T, int KIND, int TAPS>
__global__ __launch_bounds__(256) void state_prep_kernel(const vmi_hy_state_args p, const vmi_hy_step s) {
  extern __shared__ __attribute__((aligned(16))) float lds[];
  const int dim = p.dim, vdim = p.vdim, LD = dim + 4, LDV = vdim + 4;
  float* ql = lds;                                             // [16][LD]
  float* kl = ql + CH * LD;                                    // [16][LD]
  float* gl = kl + CH * LD;                                    // [16][LD] (delta)
  float* vl = gl + (KIND == VMI_HY_DELTA ? CH * LD : 0);       // [16][LDV]
  float* pb = vl + CH * LDV;                                   // [4][16][20] parts of B
  float* pa = pb + 4 * CH * 20;                                // [4][16][20] parts of A (delta)
  float* Al = pa + (KIND == VMI_HY_DELTA ? 4 * CH * 20 : 0);   // [16][20] beta_i A_ij (delta)
  float* be = Al + (KIND == VMI_HY_DELTA ? CH * 20 : 0);       // [16]: beta | (retention) powers of the decay
  float* most = be + CH;                                       // [4]
  float* dl = most + CH;                                       // [dim] e^{G_15} (delta)
  const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6), m16 = tid >> 4, l16 = tid & 15;
  const int h = blockIdx.y, hk = h / (p.heads / p.kv_heads);
  const int e = s.chunks[2 * blockIdx.x], first = s.chunks[2 * blockIdx.x + 1];
  const Portion r = portion(s, e);
  const int t0 = r.qs + first, n = min(CH, r.len - first), C = 2 * p.kv_heads * dim + p.heads * vdim;
  const int cq = hk * dim, ck = (p.kv_heads + hk) * dim, cv = 2 * p.kv_heads * dim + h * vdim;
  const Scratch sc(KIND, dim, vdim);
  float* out = p.scratch + ((int64_t)blockIdx.x * p.heads + h) * sc.size;
  const f32x4 zero = f32x4{0.f, 0.f, 0.f, 0.f};

  if constexpr (KIND == VMI_HY_DELTA) {
    // row m16, 16 lanes: channels through the convolution
    auto conv = [&](float* dst, int ch, int width) {
      for (int c = 8 * l16; c < width; c += 128) {
        f32x8 v = {0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f};
        if (m16 < n) v = conv_silu8<T, TAPS>(p, r, C, t0 + m16, ch + c);
        *reinterpret_cast<f32x4*>(dst + c) = f32x4{v[0], v[1], v[2], v[3]};
        *reinterpret_cast<f32x4*>(dst + c + 4) = f32x4{v[4], v[5], v[6], v[7]};
      }
    };
    conv(ql + m16 * LD, cq, dim);
    conv(kl + m16 * LD, ck, dim);
    conv(vl + m16 * LDV, cv, vdim);
    if (tid < CH) be[tid] = tid < n ? sigmoid((float)static_cast<const T*>(p.beta)[(int64_t)(t0 + tid) * p.ldp + h]) : 0.f;
    {   // decays: the steps row by row, then their sums down the rows
      const float rate = p.rate[h];
      const T* z = static_cast<const T*>(p.z) + (int64_t)(t0 + min(m16, n - 1)) * p.ldz + (int64_t)h * dim;
      const float* bias = p.dt_bias + (int64_t)h * dim;
      for (int c = 4 * l16; c < dim; c += 64) {
        const V4<T> zv = *reinterpret_cast<const V4<T>*>(z + c);
        const f32x4 bv = *reinterpret_cast<const f32x4*>(bias + c);
        f32x4 g;
#pragma unroll
        for (int x = 0; x < 4; ++x) g[x] = m16 < n ? -rate * softplus((float)zv[x] + bv[x]) : 0.f;
        *reinterpret_cast<f32x4*>(gl + m16 * LD + c) = g;
      }
    }
    {   // unit lengths of the rows of this lane group's own making
      float* q = ql + m16 * LD;
      float* k = kl + m16 * LD;
      float a = 0.f, b = 0.f;
      for (int c = 8 * l16; c < dim; c += 128)
#pragma unroll
        for (int x = 0; x < 8; ++x) a = fmaf(q[c + x], q[c + x], a), b = fmaf(k[c + x], k[c + x], b);
#pragma unroll
      for (int o = 8; o > 0; o >>= 1) a += __shfl_xor(a, o, 64), b += __shfl_xor(b, o, 64);
      a = 1.f / sqrtf((a + 1e-6f) * (float)p.dim_n);
      b = 1.f / sqrtf(b + 1e-6f);
      for (int c = 8 * l16; c < dim; c += 128)
#pragma unroll
        for (int x = 0; x < 8; ++x) q[c + x] *= a, k[c + x] *= b;
    }
    __syncthreads();
    float deepest = 0.f;
    for (int c = tid; c < dim; c += 256) {
      float G = 0.f;
#pragma unroll
      for (int m = 0; m < CH; ++m) gl[m * LD + c] = G += gl[m * LD + c];
      dl[c] = exp_hw(G);
      deepest = fminf(deepest, G);
    }
#pragma unroll
    for (int o = 32; o > 0; o >>= 1) deepest = fminf(deepest, __shfl_xor(deepest, o, 64));
    if (lane == 0) most[wave] = deepest;
    __syncthreads();
    const bool little = fminf(fminf(most[0], most[1]), fminf(most[2], most[3])) >= -LITTLE_DECAY;
    if (!little) {   // exponents of differences, pair by pair
      float a = 0.f, b = 0.f;
      if (l16 <= m16) {
        for (int c = 0; c < dim; c += 4) {
          const f32x4 qi = *reinterpret_cast<const f32x4*>(ql + m16 * LD + c), ki = *reinterpret_cast<const f32x4*>(kl + m16 * LD + c);
          const f32x4 kj = *reinterpret_cast<const f32x4*>(kl + l16 * LD + c), gi = *reinterpret_cast<const f32x4*>(gl + m16 * LD + c);
          const f32x4 gj = *reinterpret_cast<const f32x4*>(gl + l16 * LD + c);
#pragma unroll
          for (int x = 0; x < 4; ++x) {
            const float w = kj[x] * exp_hw(gi[x] - gj[x]);
            a = fmaf(ki[x], w, a);
            b = fmaf(qi[x], w, b);
          }
        }
      }
      Al[m16 * 20 + l16] = l16 < m16 ? a * be[m16] : 0.f;
      out[sc.b + tid] = l16 <= m16 ? b : 0.f;
      __syncthreads();
    }
    // q e^G; where it decays little also k e^G (in G's place) and k e^-G (in k's)
    for (int c = 4 * l16; c < dim; c += 64) {
      const int at = m16 * LD + c;
      const f32x4 g = *reinterpret_cast<const f32x4*>(gl + at), k = *reinterpret_cast<const f32x4*>(kl + at);
      f32x4 q = *reinterpret_cast<const f32x4*>(ql + at), kg, kn;
#pragma unroll
      for (int x = 0; x < 4; ++x) {
        const float eg = exp_hw(g[x]);
        q[x] *= eg;
        kg[x] = k[x] * eg;
        kn[x] = little ? k[x] * exp_hw(-g[x]) : k[x];
      }
      *reinterpret_cast<f32x4*>(ql + at) = q;
      *reinterpret_cast<f32x4*>(out + sc.q + m16 * dim + c) = q;
      *reinterpret_cast<f32x4*>(kl + at) = kn;
      if (little) *reinterpret_cast<f32x4*>(gl + at) = kg;
    }
    __syncthreads();
    if (little) {
      put_products(pa, row_products(gl, kl, LD, dim, wave, lane), wave, lane);
      put_products(pb, row_products(ql, kl, LD, dim, wave, lane), wave, lane);
      __syncthreads();
      Al[m16 * 20 + l16] = l16 < m16 ? sum_products(pa, m16, l16) * be[m16] : 0.f;
      out[sc.b + tid] = l16 <= m16 ? sum_products(pb, m16, l16) : 0.f;
    }
    // k e^{G_15 - G}, transposed: 4 rows of a channel a thread
    for (int c = tid >> 2; c < dim; c += 64) {
      const int y = 4 * (tid & 3);
      f32x4 k;
#pragma unroll
      for (int x = 0; x < 4; ++x) {
        const float g = little ? dl[c] : exp_hw(gl[(CH - 1) * LD + c] - gl[(y + x) * LD + c]);
        k[x] = kl[(y + x) * LD + c] * g;
      }
      *reinterpret_cast<f32x4*>(out + sc.k + c * CH + y) = k;
    }
    if (!little) {
      __syncthreads();
      for (int c = 4 * l16; c < dim; c += 64) {
        const int at = m16 * LD + c;
        const f32x4 g = *reinterpret_cast<const f32x4*>(gl + at), k = *reinterpret_cast<const f32x4*>(kl + at);
        f32x4 kg;
#pragma unroll
        for (int x = 0; x < 4; ++x) kg[x] = k[x] * exp_hw(g[x]);
        *reinterpret_cast<f32x4*>(gl + at) = kg;
      }
    }
    __syncthreads();
    // forward substitution, a column a thread: of W (dim of them), of U0 (vdim)
    for (int col = tid; col < dim + vdim; col += 256) {
      const bool isw = col < dim;
      const int c = isw ? col : col - dim;
      const float* rhs = isw ? gl + c : vl + c;
      const int ld = isw ? LD : LDV;
      float x[CH];
#pragma unroll
      for (int i = 0; i < CH; ++i) {
        float v = rhs[i * ld] * be[i];
#pragma unroll
        for (int j = 0; j < i; ++j) v = fmaf(-Al[i * 20 + j], x[j], v);
        x[i] = v;
      }
      if (isw) {
        out[sc.d + c] = dl[c];
#pragma unroll
        for (int i = 0; i < CH; ++i) out[sc.w + i * dim + c] = x[i];
      } else {
#pragma unroll
        for (int i = 0; i < CH; i += 4) *reinterpret_cast<f32x4*>(out + sc.u + c * CH + i) = f32x4{x[i], x[i + 1], x[i + 2], x[i + 3]};
      }
    }
    if (first + CH >= r.len && p.taps > 1) {   // the chunk that ends the portion
      write_tail<T>(p, r, C, cv, vdim, tid, 256);
      if (h == hk * (p.heads / p.kv_heads)) {
        write_tail<T>(p, r, C, cq, dim, tid, 256);
        write_tail<T>(p, r, C, ck, dim, tid, 256);
      }
    }
  } else {
    const float ld = p.log2_decay[h];
    if (tid <= CH) be[tid] = exp2f(ld * (float)tid);   // d^0 .. d^16 (runs one past be, into most)
    if (m16 < n) {
      rotated_row<T>(p, t0 + m16, hk, ql + m16 * LD, kl + m16 * LD, l16, 16);
    } else {
      for (int c = 4 * l16; c < dim; c += 64)
        *reinterpret_cast<f32x4*>(ql + m16 * LD + c) = *reinterpret_cast<f32x4*>(kl + m16 * LD + c) = zero;
    }
    for (int c = 4 * l16; c < vdim; c += 64) {
      const V4<T> v = *reinterpret_cast<const V4<T>*>(static_cast<const T*>(p.proj) + (int64_t)(t0 + min(m16, n - 1)) * p.ldp + cv + c);
      f32x4 f;
#pragma unroll
      for (int x = 0; x < 4; ++x) f[x] = m16 < n ? (float)v[x] : 0.f;
      *reinterpret_cast<f32x4*>(vl + m16 * LDV + c) = f;
    }
    __syncthreads();
    put_products(pb, row_products(ql, kl, LD, dim, wave, lane), wave, lane);
    const float dq = be[m16 + 1];
    for (int c = 4 * l16; c < dim; c += 64)
      *reinterpret_cast<f32x4*>(out + sc.q + m16 * dim + c) = *reinterpret_cast<const f32x4*>(ql + m16 * LD + c) * dq;
    const int y = 4 * (tid & 3);   // four rows of a channel a thread
    f32x4 dk;
#pragma unroll
    for (int x = 0; x < 4; ++x) dk[x] = be[max(n - 1 - y - x, 0)];
    for (int c = tid >> 2; c < dim; c += 64) {
      f32x4 k;
#pragma unroll
      for (int x = 0; x < 4; ++x) k[x] = kl[(y + x) * LD + c] * dk[x];
      *reinterpret_cast<f32x4*>(out + sc.k + c * CH + y) = k;
    }
    for (int c = tid >> 2; c < vdim; c += 64) {
      f32x4 v;
#pragma unroll
      for (int x = 0; x < 4; ++x) v[x] = vl[(y + x) * LDV + c];
      *reinterpret_cast<f32x4*>(out + sc.u + c * CH + y) = v;
    }
    for (int c = tid; c < dim; c += 256) out[sc.d + c] = be[n];
    __syncthreads();
    out[sc.b + tid] = l16 <= m16 ? sum_products(pb, m16, l16) * be[max(m16 - l16, 0)] : 0.f;
  }
}

// NT: 16-row tiles of the state, dealt over RS waves.  One workgroup: CT tiles of 16 value columns of one (entry, head)
template <int KIND, int NT, int RS, int CT>
__global__ __launch_bounds__(64 * RS, CT > 1 && NT <= 8 ? 2 : 1) void state_scan_kernel(const vmi_hy_state_args p, const vmi_hy_step s) {
  constexpr int NW = NT / RS, DEPTH = NW <= 2 && CT == 1 ? 3 : 2;   // tiles of a wave, chunks of operands in registers
  constexpr bool DELTA = KIND == VMI_HY_DELTA;
  constexpr int EW = 4 / RS;                             // elements of a lane's four that a wave finishes of o
  __shared__ f32x4 reda[DELTA ? 2 : 1][CT][DELTA ? RS : 1][64];
  __shared__ float redo[2][CT][RS][4][64];
  const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), kc = lane >> 4, r16 = lane & 15;
  // (heads vary fastest: the column blocks of one head, which read the same operands, then share an XCD's L2)
  const int h = blockIdx.x % p.heads, col0 = (int)(blockIdx.x / p.heads) * 16 * CT, e = blockIdx.y;
  const Portion r = portion(s, e);
  if (r.len <= 0) return;
  constexpr int dim = NT * 16;
  const int ct0 = wave * NW;
  const Scratch sc(KIND, dim, p.vdim);
  const int nch = (r.len + CH - 1) / CH;
  const int64_t step = (int64_t)p.heads * sc.size;
  float* const base = p.scratch + ((int64_t)s.chunk_start[e] * p.heads + h) * sc.size;
  float* st = p.state + (((int64_t)r.slot * p.heads + h) * dim + 16 * ct0 + 4 * kc) * p.vdim + col0 + r16;
  f32x4 S[NW][CT];
#pragma unroll
  for (int t = 0; t < NW; ++t)
#pragma unroll
    for (int c = 0; c < CT; ++c)
#pragma unroll
      for (int x = 0; x < 4; ++x) S[t][c][x] = r.ctx > 0 ? st[(int64_t)(16 * t + x) * p.vdim + 16 * c] : 0.f;

  struct Operands {
    f32x4 w[DELTA ? NW : 1], q[NW], k[NW], d[NW], u[CT];
    float b[EW];
  };
  const int row = r16 * dim + 16 * ct0 + 4 * kc, col = r16 * CH + 4 * kc;
  // (no branch stands in a chunk: every path issues the same loads and stores, so the waits count them exactly)
  auto load = [&](Operands& o, int c) {
    const float* at = base + min(c, nch - 1) * step;   // (past the end: the last one again)
#pragma unroll
    for (int t = 0; t < NW; ++t) {
      if constexpr (DELTA) o.w[t] = *reinterpret_cast<const f32x4*>(at + sc.w + row + 16 * t);
      o.q[t] = *reinterpret_cast<const f32x4*>(at + sc.q + row + 16 * t);
    }
#pragma unroll
    for (int j = 0; j < CT; ++j) o.u[j] = *reinterpret_cast<const f32x4*>(at + sc.u + (col0 + 16 * j) * CH + col);
#pragma unroll
    for (int i = 0; i < EW; ++i) o.b[i] = at[sc.b + col + wave + RS * i];
#pragma unroll
    for (int t = 0; t < NW; ++t) {
      o.d[t] = *reinterpret_cast<const f32x4*>(at + sc.d + 16 * (ct0 + t) + 4 * kc);
      o.k[t] = *reinterpret_cast<const f32x4*>(at + sc.k + 16 * (ct0 + t) * CH + col);
    }
  };
  f32x4 part[CT];                           // this wave's part of the last chunk's o
#pragma unroll
  for (int j = 0; j < CT; ++j) part[j] = f32x4{0.f, 0.f, 0.f, 0.f};
  auto publish = [&](int c) {               // (two places: a wave still reading those of c has passed the barrier of c, not of c + 1)
#pragma unroll
    for (int j = 0; j < CT; ++j)
#pragma unroll
      for (int x = 0; x < 4; ++x) redo[c & 1][j][wave][x][lane] = part[j][x];
  };
  auto finish = [&](int c) {                // the elements wave, wave + RS, .. of every lane's four of chunk c - 1
    float* out = base + max(c - 1, 0) * step + sc.o + 4 * kc * p.vdim + col0 + r16;
#pragma unroll
    for (int j = 0; j < CT; ++j)
#pragma unroll
      for (int i = 0; i < EW; ++i) {
        const int x = wave + RS * i;
        float y = redo[c & 1][j][0][x][lane];
#pragma unroll
        for (int w = 1; w < RS; ++w) y += redo[c & 1][j][w][x][lane];
        out[x * p.vdim + 16 * j] = y;       // (c = 0: zeros, which the next chunk overwrites)
      }
  };
  auto chunk = [&](Operands& o, int c) {
    f32x4 a[CT], b[CT], u[CT];
    publish(c);
#pragma unroll
    for (int j = 0; j < CT; ++j) a[j] = b[j] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int t = 0; t < NW; ++t)
#pragma unroll
      for (int j = 0; j < CT; ++j) {
        if constexpr (DELTA) mma4(a[j], o.w[t], S[t][j]);
        mma4(b[j], o.q[t], S[t][j]);
      }
    if constexpr (DELTA) {
#pragma unroll
      for (int j = 0; j < CT; ++j) reda[c & 1][j][wave][lane] = a[j];
    }
    __syncthreads();
#pragma unroll
    for (int j = 0; j < CT; ++j) {
      u[j] = o.u[j];
      if constexpr (DELTA) {
#pragma unroll
        for (int w = 0; w < RS; ++w) u[j] -= reda[c & 1][j][w][lane];
      }
    }
#pragma unroll
    for (int t = 0; t < NW; ++t)
#pragma unroll
      for (int j = 0; j < CT; ++j) {
#pragma unroll
        for (int x = 0; x < 4; ++x) S[t][j][x] *= o.d[t][x];
        mma4(S[t][j], o.k[t], u[j]);
      }
#pragma unroll
    for (int j = 0; j < CT; ++j) {
#pragma unroll
      for (int i = 0; i < EW; ++i) {        // B u, a share of its inner rows a wave
        float ux = u[j][RS * i];
#pragma unroll
        for (int w = 1; w < RS; ++w) ux = wave == w ? u[j][w + RS * i] : ux;
        b[j] = __builtin_amdgcn_mfma_f32_16x16x4f32(o.b[i], ux, b[j], 0, 0, 0);
      }
      part[j] = b[j];
    }
    finish(c);
    load(o, c + DEPTH);
  };
  Operands ops[DEPTH];
#pragma unroll
  for (int i = 0; i < DEPTH; ++i) load(ops[i], i);
  int c = 0;
  for (; c + DEPTH <= nch; c += DEPTH) {
#pragma unroll
    for (int i = 0; i < DEPTH; ++i) chunk(ops[i], c + i);
  }
#pragma unroll
  for (int i = 0; i + 1 < DEPTH; ++i)
    if (c + i < nch) chunk(ops[i], c + i);
  publish(nch);
  __syncthreads();
  finish(nch);
#pragma unroll
  for (int t = 0; t < NW; ++t)
#pragma unroll
    for (int j = 0; j < CT; ++j)
#pragma unroll
      for (int x = 0; x < 4; ++x) st[(int64_t)(16 * t + x) * p.vdim + 16 * j] = S[t][j][x];
}

// every head's o over its root mean square, times a weight and the activated gate; 16 lanes per (token, head).  o: rows of p.o, or
// (portions) where the walk left them
template <typename T>
__global__ __launch_bounds__(256) void head_norm_gate_kernel(const vmi_hy_state_args p, const vmi_hy_step s) {
  const int64_t row = (int64_t)blockIdx.x * 16 + (threadIdx.x >> 4);
  if (row >= (int64_t)s.T * p.heads) return;
  const int64_t t = row / p.heads;
  const int h = (int)(row - t * p.heads), l = threadIdx.x & 15, vdim = p.vdim;
  const float* o = p.o + row * vdim;
  if (!p.single) {
    const int e = s.tok_seq[t];
    if (e < 0) return;
    const int m = (int)t - s.q_start[e];
    const Scratch sc(p.kind, p.dim, vdim);
    o = p.scratch + ((int64_t)(s.chunk_start[e] + m / CH) * p.heads + h) * sc.size + sc.o + (m % CH) * vdim;
  }
  const T* gate = static_cast<const T*>(p.gate) + t * p.ldg + (int64_t)h * vdim;
  T* out = static_cast<T*>(p.out) + t * p.ldo + (int64_t)h * vdim;
  float ss = 0.f;
  for (int k = l * 4; k < vdim; k += 64) {
    const f32x4 v = *reinterpret_cast<const f32x4*>(o + k);
#pragma unroll
    for (int e = 0; e < 4; ++e) ss = fmaf(v[e], v[e], ss);
  }
#pragma unroll
  for (int m = 8; m > 0; m >>= 1) ss += __shfl_xor(ss, m, 64);
  const float r = 1.f / sqrtf(ss / (float)p.vdim_n + p.eps);
  for (int k = l * 4; k < vdim; k += 64) {
    const f32x4 v = *reinterpret_cast<const f32x4*>(o + k);
    const V4<T> g = *reinterpret_cast<const V4<T>*>(gate + k);
    f32x4 w = f32x4{1.f, 1.f, 1.f, 1.f};
    if (p.norm_w) w = *reinterpret_cast<const f32x4*>(p.norm_w + k);
    V4<T> y;
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const float z = (float)g[e];
      y[e] = (T)(v[e] * r * w[e] * (p.act == VMI_HY_ACT_SILU ? silu(z) : sigmoid(z)));
    }
    *reinterpret_cast<V4<T>*>(out + k) = y;
  }
}

// the columns of a state that one workgroup of the single-token step takes, and the rows a thread then holds
inline int step_slice(int dim, int vdim) {
  const int most = dim <= 128 ? 128 : dim <= 256 ? 64 : 32;
  return vdim <= most ? vdim : most;
}
inline int step_rows(int dim, int slice) {
  const int groups = 256 / (slice / 4);
  return (dim + groups - 1) / groups;
}

// one token of one (entry, head), a slice of the value columns.  RPT: state rows a thread holds (at most)
template <typename T, int KIND, int RPT>
__global__ __launch_bounds__(256) void state_step_kernel(const vmi_hy_state_args p, const vmi_hy_step s, const int slice) {
  extern __shared__ __attribute__((aligned(16))) float lds[];
  const int dim = p.dim, tid = threadIdx.x, h = blockIdx.x, e = blockIdx.y, c0 = (int)blockIdx.z * slice;
  const int width = min(slice, p.vdim - c0), quads = slice >> 2, groups = 256 / quads;
  float* ql = lds;               // [dim]
  float* kl = ql + dim;          // [dim]
  float* gl = kl + dim;          // [dim]
  float* vl = gl + dim;          // [slice]
  float* ul = vl + slice;        // [slice]
  float* red = ul + slice;       // [groups][slice]
  float* sums = red + 1024;      // [8]
  const Portion r = portion(s, e);
  if (r.len <= 0) return;
  const int t = r.qs, hk = h / (p.heads / p.kv_heads), C = 2 * p.kv_heads * dim + p.heads * p.vdim;
  const int cq = hk * dim, ck = (p.kv_heads + hk) * dim, cv = 2 * p.kv_heads * dim + h * p.vdim + c0;
  const int quad = tid % quads, grp = tid / quads;
  const bool mine = grp < groups && quad * 4 < width;
  float* st = p.state + (((int64_t)r.slot * p.heads + h) * dim) * p.vdim + c0 + quad * 4;
  f32x4 S[RPT];
  const bool have = r.ctx > 0;
#pragma unroll
  for (int i = 0; i < RPT; ++i) {
    const int row = grp + i * groups;
    S[i] = f32x4{0.f, 0.f, 0.f, 0.f};
    if (have && mine && row < dim) S[i] = *reinterpret_cast<const f32x4*>(st + (int64_t)row * p.vdim);
  }
  float beta = 1.f;
  if constexpr (KIND == VMI_HY_DELTA) {
    const int ud = dim >> 3, uv = width >> 3;
    for (int u = tid; u < 2 * ud + uv; u += 256) {
      float* dst;
      int ch;
      if (u < ud) dst = ql + u * 8, ch = cq + u * 8;
      else if (u < 2 * ud) dst = kl + (u - ud) * 8, ch = ck + (u - ud) * 8;
      else dst = vl + (u - 2 * ud) * 8, ch = cv + (u - 2 * ud) * 8;
      const f32x8 v = p.taps == 4 ? conv_silu8<T, 4>(p, r, C, t, ch) : conv_silu8<T, 0>(p, r, C, t, ch);
      *reinterpret_cast<f32x4*>(dst) = f32x4{v[0], v[1], v[2], v[3]};
      *reinterpret_cast<f32x4*>(dst + 4) = f32x4{v[4], v[5], v[6], v[7]};
    }
    const float rate = p.rate[h];
    for (int c = tid; c < dim; c += 256)
      gl[c] = exp_hw(-rate * softplus((float)static_cast<const T*>(p.z)[(int64_t)t * p.ldz + (int64_t)h * dim + c] + p.dt_bias[(int64_t)h * dim + c]));
    beta = sigmoid((float)static_cast<const T*>(p.beta)[(int64_t)t * p.ldp + h]);
    if (p.taps > 1) {
      write_tail<T>(p, r, C, cv, width, tid, 256);
      if (blockIdx.z == 0 && h == hk * (p.heads / p.kv_heads)) {
        write_tail<T>(p, r, C, cq, dim, tid, 256);
        write_tail<T>(p, r, C, ck, dim, tid, 256);
      }
    }
    __syncthreads();
    if (tid < 128) {   // wave 0: q, wave 1: k
      float* x = tid < 64 ? ql : kl;
      float a = 0.f;
      for (int c = tid & 63; c < dim; c += 64) a = fmaf(x[c], x[c], a);
      a = wave_sum(a) + 1e-6f;
      a = 1.f / sqrtf(tid < 64 ? a * (float)p.dim_n : a);
      for (int c = tid & 63; c < dim; c += 64) x[c] *= a;
    }
  } else {
    if (tid < 64) rotated_row<T>(p, t, hk, ql, kl, tid, 64);
    for (int c = tid; c < width; c += 256) vl[c] = (float)static_cast<const T*>(p.proj)[(int64_t)t * p.ldp + cv + c];
    beta = p.decay[h];   // (the one decay of the head)
  }
  __syncthreads();
  auto gather = [&](const f32x4& part) {   // sums over the row groups, into red[0]'s place of every column; returns column tid's
    if (mine) *reinterpret_cast<f32x4*>(red + grp * slice + quad * 4) = part;
    __syncthreads();
    float v = 0.f;
    if (tid < width)
      for (int g = 0; g < groups; ++g) v += red[g * slice + tid];
    return v;
  };
  f32x4 part = f32x4{0.f, 0.f, 0.f, 0.f}, u;
  if constexpr (KIND == VMI_HY_DELTA) {
#pragma unroll
    for (int i = 0; i < RPT; ++i) {
      const int row = grp + i * groups;
      if (mine && row < dim) {
        S[i] = S[i] * gl[row];
        const float k = kl[row];
#pragma unroll
        for (int x = 0; x < 4; ++x) part[x] = fmaf(S[i][x], k, part[x]);
      }
    }
    const float held = gather(part);
    if (tid < width) ul[tid] = beta * (vl[tid] - held);
    __syncthreads();
    if (mine) u = *reinterpret_cast<const f32x4*>(ul + quad * 4);
  } else {
    if (mine) u = *reinterpret_cast<const f32x4*>(vl + quad * 4);
  }
  part = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
  for (int i = 0; i < RPT; ++i) {
    const int row = grp + i * groups;
    if (mine && row < dim) {
      const float k = kl[row], q = ql[row];
      if constexpr (KIND == VMI_HY_RETENTION) S[i] = S[i] * beta;
#pragma unroll
      for (int x = 0; x < 4; ++x) {
        S[i][x] = fmaf(k, u[x], S[i][x]);
        part[x] = fmaf(S[i][x], q, part[x]);
      }
      *reinterpret_cast<f32x4*>(st + (int64_t)row * p.vdim) = S[i];
    }
  }
  const float o = gather(part);
  if (slice < p.vdim) {
    if (tid < width) p.o[((int64_t)t * p.heads + h) * p.vdim + c0 + tid] = o;
    return;
  }
  const float ss = wave_sum(tid < width ? o * o : 0.f);   // (this workgroup holds the whole head, at most 128 columns of it)
  if ((tid & 63) == 0) sums[tid >> 6] = ss;
  __syncthreads();
  if (tid < width) {
    const float z = (float)static_cast<const T*>(p.gate)[(int64_t)t * p.ldg + (int64_t)h * p.vdim + tid];
    const float y = o / sqrtf((sums[0] + sums[1] + sums[2] + sums[3]) / (float)p.vdim_n + p.eps) * (p.norm_w ? p.norm_w[tid] : 1.f);
    static_cast<T*>(p.out)[(int64_t)t * p.ldo + (int64_t)h * p.vdim + tid] = (T)(y * (p.act == VMI_HY_ACT_SILU ? silu(z) : sigmoid(z)));
  }
}

template <typename T>
static void launch_norm_gate(const vmi_hy_state_args& p, const vmi_hy_step& s, hipStream_t st) {
  hipLaunchKernelGGL(head_norm_gate_kernel<T>, dim3(((int64_t)s.T * p.heads + 15) / 16), dim3(256), 0, st, p, s);
}

template <typename T, int KIND>
static int run_step(const vmi_hy_state_args& p, const vmi_hy_step& s, hipStream_t st) {
  const int slice = step_slice(p.dim, p.vdim), rows = step_rows(p.dim, slice);
  const dim3 grid(p.heads, s.B, (p.vdim + slice - 1) / slice);
  const size_t lds = (size_t)(3 * p.dim + 2 * slice + 1024 + 8) * sizeof(float);
  if (rows <= 4) hipLaunchKernelGGL(HIP_KERNEL_NAME(state_step_kernel<T, KIND, 4>), grid, dim3(256), lds, st, p, s, slice);
  else if (rows <= 8) hipLaunchKernelGGL(HIP_KERNEL_NAME(state_step_kernel<T, KIND, 8>), grid, dim3(256), lds, st, p, s, slice);
  else if (rows <= 16) hipLaunchKernelGGL(HIP_KERNEL_NAME(state_step_kernel<T, KIND, 16>), grid, dim3(256), lds, st, p, s, slice);
  else if (rows <= 32) hipLaunchKernelGGL(HIP_KERNEL_NAME(state_step_kernel<T, KIND, 32>), grid, dim3(256), lds, st, p, s, slice);
  else return fail(VMI_HY_E_SHAPE, "vmi_hy_state", "heads this large are not built");
  if (slice < p.vdim) launch_norm_gate<T>(p, s, st);
  return launched("vmi_hy_state");
}

template <int KIND, int NT>
static void launch_scan(const vmi_hy_state_args& p, const vmi_hy_step& s, hipStream_t st) {
  constexpr int RS = NT % 4 == 0 ? 4 : 2;
  const int tiles = p.vdim / 16;   // (even: vdim is a multiple of 32)
  // states enough for the chip: a workgroup takes two column tiles, which halves what is read per column
  if (NT <= 16 && (int64_t)p.heads * tiles * s.B >= 1024)
    hipLaunchKernelGGL(HIP_KERNEL_NAME(state_scan_kernel<KIND, NT, RS, NT <= 16 ? 2 : 1>), dim3(p.heads * (tiles / 2), s.B), dim3(64 * RS), 0,
                       st, p, s);
  else
    hipLaunchKernelGGL(HIP_KERNEL_NAME(state_scan_kernel<KIND, NT, RS, 1>), dim3(p.heads * tiles, s.B), dim3(64 * RS), 0, st, p, s);
}

template <typename T, int KIND>
static int run_chunks(const vmi_hy_state_args& p, const vmi_hy_step& s, hipStream_t st) {
  auto* fn = KIND == VMI_HY_DELTA && p.taps == 4 ? state_prep_kernel<T, KIND, 4> : state_prep_kernel<T, KIND, 0>;
  const size_t lds = prep_lds(KIND, p.dim, p.vdim);
  if (int rc = allow_lds(fn, lds, "vmi_hy_state")) return rc;
  hipLaunchKernelGGL(fn, dim3(s.n_chunks, p.heads), dim3(256), lds, st, p, s);
  switch (p.dim) {
    case 32: launch_scan<KIND, 2>(p, s, st); break;
    case 64: launch_scan<KIND, 4>(p, s, st); break;
    case 96: launch_scan<KIND, 6>(p, s, st); break;
    case 128: launch_scan<KIND, 8>(p, s, st); break;
    case 192: launch_scan<KIND, 12>(p, s, st); break;
    case 256: launch_scan<KIND, 16>(p, s, st); break;
    case 512: launch_scan<KIND, 32>(p, s, st); break;
    default: return fail(VMI_HY_E_SHAPE, "vmi_hy_state", "key dimensions of 32, 64, 96, 128, 192, 256 and 512 are built");
  }
  launch_norm_gate<T>(p, s, st);
  return launched("vmi_hy_state");
}

template <typename T>
static int run_state(const vmi_hy_state_args& p, const vmi_hy_step& s, hipStream_t st) {
  if (p.kind == VMI_HY_DELTA) return p.single ? run_step<T, VMI_HY_DELTA>(p, s, st) : run_chunks<T, VMI_HY_DELTA>(p, s, st);
  return p.single ? run_step<T, VMI_HY_RETENTION>(p, s, st) : run_chunks<T, VMI_HY_RETENTION>(p, s, st);
}

}  // namespace vmi_hybrid

using namespace vmi_hybrid;

extern "C" {

int64_t vmi_hy_state_scratch(int32_t kind, int32_t dim, int32_t vdim) { return Scratch(kind, dim, vdim).size; }

int32_t vmi_hy_state_fuses(int32_t dim, int32_t vdim) { return step_slice(dim, vdim) == vdim; }

int vmi_hy_rotations(const double* freq, int32_t half, float* out, const vmi_hy_step* s, int32_t device, void* stream) {
  static const char* who = "vmi_hy_rotations";
  if (!freq || !out || !s || !s->tok_pos || s->T <= 0 || half <= 0) return fail(VMI_HY_E_ARG, who, "null pointer or non-positive size");
  DeviceScope dev(device);
  if (!dev.ok) return fail(VMI_HY_E_HIP, who, "hipSetDevice failed");
  hipLaunchKernelGGL(rotations_kernel, dim3(s->T), dim3(64), 0, static_cast<hipStream_t>(stream), freq, half, out, s->tok_pos);
  return launched(who);
}

int vmi_hy_state(const vmi_hy_state_args* a, const vmi_hy_step* s, void* stream) {
  static const char* who = "vmi_hy_state";
  if (!a || !s || !a->proj || !a->state || !a->out || !a->gate || !s->q_start || !s->q_len || !s->ctx || !s->state_slot || !s->flip ||
      s->T <= 0 || s->B <= 0 || a->heads <= 0 || a->kv_heads <= 0 || a->dim <= 0 || a->vdim <= 0 || a->dim_n <= 0 || a->dim_n > a->dim ||
      a->vdim_n <= 0 || a->vdim_n > a->vdim || a->heads % a->kv_heads || a->kind < 0 || a->kind > 1 || a->dtype < 0 || a->dtype > 1)
    return fail(VMI_HY_E_ARG, who, "null pointer or a size out of range");
  if (a->kind == VMI_HY_DELTA && (!a->beta || !a->z || !a->conv_w || !a->rate || !a->dt_bias || a->taps < 1 || a->taps > MAX_TAPS ||
                                  (a->taps > 1 && !a->tail)))
    return fail(VMI_HY_E_ARG, who, "the delta rule needs its gates and a convolution of 1 to 16 taps");
  if (a->kind == VMI_HY_RETENTION && ((a->rot_n > 0 && !a->turns) || !a->decay || !a->log2_decay || a->rot_n < 0 || a->rot_n > a->dim || (a->rot_n & 1)))
    return fail(VMI_HY_E_ARG, who, "retention needs decays and an even number of rotated dimensions");
  if (a->single ? !a->o && !vmi_hy_state_fuses(a->dim, a->vdim)
                : !a->scratch || !s->tok_seq || !s->chunks || !s->chunk_start || s->n_chunks <= 0)
    return fail(VMI_HY_E_ARG, who, "portions need chunks and scratch, single tokens of heads this large a place for o");
  if ((a->dim & 31) || (a->vdim & 31) || (a->ldp & 7) || ((uintptr_t)a->proj & 15) || (a->ldg & 3) || (a->ldo & 3) || a->dim > 512 || s->B > 65535 || a->heads > 65535)
    return fail(VMI_HY_E_SHAPE, who, "needs sizes that are multiples of 32, key dimensions up to 512 and aligned rows");
  DeviceScope dev(a->device);
  if (!dev.ok) return fail(VMI_HY_E_HIP, who, "hipSetDevice failed");
  hipStream_t st = static_cast<hipStream_t>(stream);
  return a->dtype == VMI_HY_BF16 ? run_state<b16>(*a, *s, st) : run_state<float>(*a, *s, st);
}

}  // extern "C"
