// Shared pieces of libvmi_hybrid.so (include/vmi_hybrid.h): element types, matrix-core fragments, host-side helpers.
//
// Both element types use ONE fragment shape: a lane holds 8 consecutive k of one row (k = 8 * (lane / 16) + e, row = lane % 16).
// In bfloat16 that is one v_mfma_f32_16x16x32_bf16; in float32 element e of the four lane groups is one
// v_mfma_f32_16x16x4_f32, eight of them per fragment — the order of the k inside a fragment does not matter as long as both
// operands agree.  D: lane holds rows 4 * (lane / 16) + r (r = 0 .. 3) of column lane % 16.
#pragma once
#include <hip/hip_runtime.h>
#include <stdint.h>

#include "vmi_hybrid.h"

namespace vmi_hybrid {

typedef __bf16 b16;
typedef b16 b16x2 __attribute__((ext_vector_type(2)));
typedef b16 b16x4 __attribute__((ext_vector_type(4)));
typedef b16 b16x8 __attribute__((ext_vector_type(8)));
typedef float f32x2 __attribute__((ext_vector_type(2)));
typedef float f32x4 __attribute__((ext_vector_type(4)));
typedef float f32x8 __attribute__((ext_vector_type(8)));

template <typename T>
struct Elem;
template <>
struct Elem<b16> {
  using v8 = b16x8;
  using v4 = b16x4;
  using v2 = b16x2;
};
template <>
struct Elem<float> {
  using v8 = f32x8;
  using v4 = f32x4;
  using v2 = f32x2;
};
template <typename T>
using V8 = typename Elem<T>::v8;
template <typename T>
using V4 = typename Elem<T>::v4;

__device__ __forceinline__ void mma(f32x4& acc, const b16x8& a, const b16x8& b) {
  acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, b, acc, 0, 0, 0);
}
__device__ __forceinline__ void mma(f32x4& acc, const f32x8& a, const f32x8& b) {
#pragma unroll
  for (int e = 0; e < 8; ++e) acc = __builtin_amdgcn_mfma_f32_16x16x4f32(a[e], b[e], acc, 0, 0, 0);
}

template <typename T>
__device__ __forceinline__ V8<T> zero8() {
  V8<T> z;
#pragma unroll
  for (int e = 0; e < 8; ++e) z[e] = (T)0.f;
  return z;
}
template <typename T>
__device__ __forceinline__ V8<T> load8(const T* p) {
  return *reinterpret_cast<const V8<T>*>(p);
}
template <typename T>
__device__ __forceinline__ f32x8 to_f32(const V8<T>& v) {
  f32x8 r;
#pragma unroll
  for (int e = 0; e < 8; ++e) r[e] = (float)v[e];
  return r;
}
template <typename T>
__device__ __forceinline__ V8<T> from_f32(const f32x8& v) {
  V8<T> r;
#pragma unroll
  for (int e = 0; e < 8; ++e) r[e] = (T)v[e];
  return r;
}

// exponential, reciprocal and root on the vector unit's own instructions (about 1 ulp each, all of it fp32)
__device__ __forceinline__ float exp_hw(float z) { return __builtin_amdgcn_exp2f(z * 1.4426950408889634f); }
__device__ __forceinline__ float sigmoid(float z) { return __builtin_amdgcn_rcpf(1.f + exp_hw(-z)); }
// 0.5 (1 + tanh w) is sigmoid(2 w)
__device__ __forceinline__ float gelu_tanh(float z) {
  return z * sigmoid(1.5957691216057308f * (z + 0.044715f * z * z * z));
}
// 1 - exp(-x), x >= 0, given e = exp(-x): a series where the difference would cancel
__device__ __forceinline__ float one_minus_exp(float x, float e) {
  const float s = x * fmaf(-x, fmaf(-x, fmaf(-x, fmaf(-x, fmaf(-x, 1.f / 720.f, 1.f / 120.f), 1.f / 24.f), 1.f / 6.f), 0.5f), 1.f);
  return x < 0.25f ? s : 1.f - e;
}
// the gated unit: gate g (already a product), up-projection u.  limit infinite, alpha 1, up 0: silu(g) u
__device__ __forceinline__ float glu(float g, float u, float limit, float alpha, float up) {
  g = fminf(g, limit);
  u = fminf(fmaxf(u, -limit), limit);
  return g * sigmoid(alpha * g) * (u + up);
}
__device__ __forceinline__ float silu(float z) { return z * sigmoid(z); }

__device__ __forceinline__ float wave_sum(float v) {
#pragma unroll
  for (int o = 32; o > 0; o >>= 1) v += __shfl_xor(v, o, 64);
  return v;
}

// ---- host ------------------------------------------------------------------------------------------------------------------
int fail(int code, const char* who, const char* what);
int launched(const char* who);   // after a launch: hipGetLastError -> code

// selects the device for the scope of an entry and puts the caller's back
struct DeviceScope {
  int prev = -1;
  bool ok = true, changed = false;
  explicit DeviceScope(int device) {
    ok = hipGetDevice(&prev) == hipSuccess;
    if (ok && prev != device) {
      ok = hipSetDevice(device) == hipSuccess;
      changed = ok;
    }
  }
  ~DeviceScope() {
    if (changed) (void)hipSetDevice(prev);
  }
};

constexpr int LDS_PER_CU = 160 * 1024;

template <typename F>
inline int allow_lds(F* fn, size_t bytes, const char* who) {
  if (bytes > LDS_PER_CU) return fail(VMI_HY_E_SHAPE, who, "a tile of these sizes does not fit a compute unit's LDS");
  if (bytes > 64 * 1024 &&
      hipFuncSetAttribute(reinterpret_cast<const void*>(fn), hipFuncAttributeMaxDynamicSharedMemorySize, (int)bytes) != hipSuccess)
    return fail(VMI_HY_E_HIP, who, "hipFuncSetAttribute failed");
  return VMI_HY_OK;
}

}  // namespace vmi_hybrid
