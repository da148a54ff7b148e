// Element conversion and vector access for kernels that run in bf16 and f32.
#pragma once

#include "common.h"

namespace amd_ops {

__device__ __forceinline__ float to_f32(float x) { return x; }
__device__ __forceinline__ float to_f32(bf16 x) { return bf2f(x); }
template <typename T>
__device__ __forceinline__ T from_f32(float x);
template <>
__device__ __forceinline__ float from_f32<float>(float x) { return x; }
template <>
__device__ __forceinline__ bf16 from_f32<bf16>(float x) { return f2bf(x); }

template <typename T, int V>
struct alignas(sizeof(T) * V > 16 ? 16 : sizeof(T) * V) ElemPack {
  T v[V];
};
template <typename T, int V>
__device__ __forceinline__ void load_vec(const T* p, float (&o)[V]) {
  const ElemPack<T, V> t = *reinterpret_cast<const ElemPack<T, V>*>(p);
#pragma unroll
  for (int j = 0; j < V; ++j) o[j] = to_f32(t.v[j]);
}
template <typename T, int V>
__device__ __forceinline__ void store_vec(T* p, const float (&x)[V]) {
  ElemPack<T, V> t;
#pragma unroll
  for (int j = 0; j < V; ++j) t.v[j] = from_f32<T>(x[j]);
  *reinterpret_cast<ElemPack<T, V>*>(p) = t;
}

__device__ __forceinline__ float sigmoid_f(float x) { return 1.0f / (1.0f + expf(-x)); }
__device__ __forceinline__ float silu_f(float x) { return x * sigmoid_f(x); }
// log(1 + e^x) without overflow
__device__ __forceinline__ float softplus_f(float x) {
  return fmaxf(x, 0.f) + log1pf(expf(-fabsf(x)));
}

}  // namespace amd_ops

// Runs the statement with `scalar` = bf16 / float by DT.
#define AMD_DISPATCH_T(DT, ...)         \
  do {                                  \
    if ((DT) == at::kBFloat16) {        \
      using scalar = ::bf16;            \
      __VA_ARGS__                       \
    } else {                            \
      using scalar = float;             \
      __VA_ARGS__                       \
    }                                   \
  } while (0)
// ... and `V` = 16 bytes of it if VEC, else 1.
#define AMD_DISPATCH_T_V(DT, VEC, ...)                                                   \
  AMD_DISPATCH_T(DT, {                                                                   \
    if (VEC) { constexpr int V = 16 / sizeof(scalar); __VA_ARGS__ }                      \
    else { constexpr int V = 1; __VA_ARGS__ }                                            \
  })
