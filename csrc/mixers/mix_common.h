// Element types of the mixer kernels: every kernel is built for bf16 and for fp32 activations /
// weights (a model served in float32 runs the same kernels with T = float), and accumulates,
// normalises and keeps the residual stream in fp32 in both.
#pragma once
#include "kernels/common.h"

namespace pkm {

using pk::bf16_t;

template <typename T>
__device__ __forceinline__ float ld(const T* p);
template <>
__device__ __forceinline__ float ld<float>(const float* p) { return *p; }
template <>
__device__ __forceinline__ float ld<bf16_t>(const bf16_t* p) { return pk::bf2f(*p); }

template <typename T>
__device__ __forceinline__ void st(T* p, float v);
template <>
__device__ __forceinline__ void st<float>(float* p, float v) { *p = v; }
template <>
__device__ __forceinline__ void st<bf16_t>(bf16_t* p, float v) { *p = pk::f2bf(v); }

__device__ __forceinline__ float sigmoidf(float z) { return 1.f / (1.f + expf(-z)); }

// 8 consecutive elements at a 16-byte address
__device__ __forceinline__ void load8(const float* p, float* f) {
  const float4 a = *reinterpret_cast<const float4*>(p), b = *reinterpret_cast<const float4*>(p + 4);
  f[0] = a.x, f[1] = a.y, f[2] = a.z, f[3] = a.w, f[4] = b.x, f[5] = b.y, f[6] = b.z, f[7] = b.w;
}
__device__ __forceinline__ void load8(const bf16_t* p, float* f) { pk::unpack8(*reinterpret_cast<const pk::u32x4*>(p), f); }
__device__ __forceinline__ void store8(float* p, const float* f) {
  *reinterpret_cast<float4*>(p) = float4{f[0], f[1], f[2], f[3]};
  *reinterpret_cast<float4*>(p + 4) = float4{f[4], f[5], f[6], f[7]};
}
__device__ __forceinline__ void store8(bf16_t* p, const float* f) { *reinterpret_cast<pk::u32x4*>(p) = pk::pack8(f); }

inline bool aligned16(const void* p) { return reinterpret_cast<uintptr_t>(p) % 16 == 0; }

// dtype codes of the extern "C" launchers
constexpr int kBF16 = 0, kF32 = 1;

}  // namespace pkm

// launcher body for both element types: DISPATCH(dt, T, launch<T>(...))
#define PKM_DISPATCH(dt, T, ...)            \
  if ((dt) == pkm::kBF16) {                 \
    using T = pkm::bf16_t;                  \
    __VA_ARGS__;                            \
  } else if ((dt) == pkm::kF32) {           \
    using T = float;                        \
    __VA_ARGS__;                            \
  } else {                                  \
    return -2;                              \
  }
