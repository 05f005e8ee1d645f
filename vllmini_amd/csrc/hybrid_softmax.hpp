// Pieces of the softmax attention kernels (hybrid_latent.hip, hybrid_attention.hip): reading an LDS tile by columns, reductions over
// the 16 lanes of a row, and the sum over key splits.
#pragma once
#include "hybrid_common.hpp"

namespace vmi_hybrid {

typedef short s16x4 __attribute__((ext_vector_type(4)));

// 8 consecutive rows (keys) of one column of an LDS tile, as a matrix operand's fragment: lane = (kc, column r16)
__device__ __forceinline__ b16x8 column8(const b16* tile, int ld, int row0, int col0, int r16) {
  const b16* a = tile + (row0 + (r16 >> 2)) * ld + col0 + 4 * (r16 & 3);
  const s16x4 lo = __builtin_amdgcn_ds_read_tr16_b64_v4i16((__attribute__((address_space(3))) s16x4*)a);
  const s16x4 hi = __builtin_amdgcn_ds_read_tr16_b64_v4i16((__attribute__((address_space(3))) s16x4*)(a + 4 * ld));
  // (whole vectors are cast: a bit_cast of one vector element takes element 0 on this compiler)
  return __builtin_shufflevector(__builtin_bit_cast(b16x4, lo), __builtin_bit_cast(b16x4, hi), 0, 1, 2, 3, 4, 5, 6, 7);
}
__device__ __forceinline__ f32x8 column8(const float* tile, int ld, int row0, int col0, int r16) {
  f32x8 r;
#pragma unroll
  for (int e = 0; e < 8; ++e) r[e] = tile[(row0 + e) * ld + col0 + r16];
  return r;
}

// maximum / sum over the 16 lanes that share kc, on the cross-lane paths of the vector unit (no LDS round trip)
template <int CTRL>
__device__ __forceinline__ float dpp(float v) {
  return __builtin_bit_cast(float, __builtin_amdgcn_mov_dpp(__builtin_bit_cast(int, v), CTRL, 0xf, 0xf, true));
}
__device__ __forceinline__ float max16(float v) {
  v = fmaxf(v, dpp<0xB1>(v));    // quad_perm [1,0,3,2]
  v = fmaxf(v, dpp<0x4E>(v));    // quad_perm [2,3,0,1]
  v = fmaxf(v, dpp<0x141>(v));   // row_half_mirror
  return fmaxf(v, dpp<0x140>(v));   // row_mirror
}
__device__ __forceinline__ float sum16(float v) {
  v += dpp<0xB1>(v);
  v += dpp<0x4E>(v);
  v += dpp<0x141>(v);
  return v + dpp<0x140>(v);
}

__device__ __forceinline__ float exp2_hw(float x) { return __builtin_amdgcn_exp2f(x); }

template <typename T>
constexpr int pad_of() {
  return 16 / (int)sizeof(T);
}

struct Combine {
  const float* partial;    // [splits][T * heads][width + 2]: unnormalised sums, their maximum (log2 units), their weight
  void* out;               // [T][ldo], head h at column h * width
  const void* gate;        // [T][ldg] one column per head, or NULL
  const int32_t* tok_seq;
  int64_t ldo, ldg;
  int T, heads, width, splits;
};

// out[row] = sum over splits of 2^(m_s - m) part_s / sum of 2^(m_s - m) l_s (times sigmoid(gate)); one workgroup per (token, head)
template <typename T>
__global__ __launch_bounds__(256) void combine_kernel(const Combine p) {
  const int64_t row = blockIdx.x, n = (int64_t)p.T * p.heads, t = row / p.heads;
  const int h = (int)(row - t * p.heads);
  if (p.tok_seq[t] < 0) return;
  const int ld = p.width + 2;
  __shared__ float wt[128];   // weight of every part (at most 128 of them)
  const float* first = p.partial + row * ld;
  if (threadIdx.x < 64) {
    float m[2], l[2], top = -1e30f, sum = 0.f;
#pragma unroll
    for (int j = 0; j < 2; ++j) {
      const int i = threadIdx.x + 64 * j;
      m[j] = i < p.splits ? first[i * n * ld + p.width] : -1e30f;
      l[j] = i < p.splits ? first[i * n * ld + p.width + 1] : 0.f;
      top = fmaxf(top, m[j]);
    }
#pragma unroll
    for (int o = 32; o > 0; o >>= 1) top = fmaxf(top, __shfl_xor(top, o, 64));
#pragma unroll
    for (int j = 0; j < 2; ++j) {
      m[j] = l[j] > 0.f ? exp2_hw(m[j] - top) : 0.f;   // (a part without keys holds no values)
      sum += m[j] * l[j];
    }
    sum = wave_sum(sum);
    const float g = p.gate ? sigmoid((float)static_cast<const T*>(p.gate)[t * p.ldg + h]) : 1.f;
#pragma unroll
    for (int j = 0; j < 2; ++j) wt[threadIdx.x + 64 * j] = m[j] / sum * g;
  }
  __syncthreads();
  for (int k = threadIdx.x; k < p.width; k += blockDim.x) {
    float a = 0.f;
#pragma unroll 8
    for (int i = 0; i < p.splits; ++i) {
      const float w = wt[i], v = first[i * n * ld + k];
      a = fmaf(w, w != 0.f ? v : 0.f, a);   // (a part without keys holds whatever was there)
    }
    static_cast<T*>(p.out)[t * p.ldo + (int64_t)h * p.width + k] = (T)a;
  }
}

template <typename T>
inline void launch_combine(const Combine& p, hipStream_t st) {
  hipLaunchKernelGGL(combine_kernel<T>, dim3((int64_t)p.T * p.heads), dim3(p.width > 128 ? 256 : 128), 0, st, p);
}

}  // namespace vmi_hybrid
