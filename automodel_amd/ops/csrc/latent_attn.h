// Shared by the latent-attention kernels: element conversion, vector access
// and the cache row layout
//   row = [ latent : rank, zero to RP | rotated key : rot, zero to PP ]
// with RP and PP multiples of 32, so that 16x16x32 MFMA steps never straddle
// the two parts and every row starts 64-byte aligned.
#pragma once

#include "common.h"

namespace amd_ops {

__host__ __device__ constexpr int pad32(int n) { return (n + 31) / 32 * 32; }

__device__ __forceinline__ float lat_f(float x) { return x; }
__device__ __forceinline__ float lat_f(bf16 x) { return bf2f(x); }
template <typename T>
__device__ __forceinline__ T lat_t(float x);
template <>
__device__ __forceinline__ float lat_t<float>(float x) { return x; }
template <>
__device__ __forceinline__ bf16 lat_t<bf16>(float x) { return f2bf(x); }

template <typename T, int V>
struct alignas(sizeof(T) * V > 16 ? 16 : sizeof(T) * V) LatPack {
  T v[V];
};

// Where each packed token sits in the cache; out-of-range rows are never
// written, so a bad slot cannot reach another sequence's memory.
__device__ __forceinline__ long cache_row(int slot, int pos, int n_slots, int max_len) {
  if (slot < 0 || slot >= n_slots || pos < 0 || pos >= max_len) return -1;
  return (long)slot * max_len + pos;
}

// One token's latent + shared rotated key: c = rms(down[:rank]) * w, and the
// last `rot` values turned by the position's angles ('rotate half' pairs).
// All threads of the block call it. `cache` / `c_out` / `kr_out` may be null.
template <typename T>
__device__ __forceinline__ void latent_token(
    const T* __restrict__ down, const T* __restrict__ w, float eps,
    const float* __restrict__ cosr, const float* __restrict__ sinr, int rank, int rot,
    T* __restrict__ cache, T* __restrict__ c_out, T* __restrict__ kr_out, float* red) {
  float ss = 0.f;
  for (int i = threadIdx.x; i < rank; i += blockDim.x) {
    const float a = lat_f(down[i]);
    ss = fmaf(a, a, ss);
  }
  const float inv = 1.0f / sqrtf(block_reduce_sum(ss, red) / (float)rank + eps);
  for (int i = threadIdx.x; i < rank; i += blockDim.x) {
    const T c = lat_t<T>(lat_f(down[i]) * inv * lat_f(w[i]));
    if (cache) cache[i] = c;
    if (c_out) c_out[i] = c;
  }
  const int half = rot / 2;
  for (int i = threadIdx.x; i < half; i += blockDim.x) {
    const float u = lat_f(down[rank + i]), v = lat_f(down[rank + half + i]);
    const float c = cosr[i], s = sinr[i];
    const T a = lat_t<T>(u * c - v * s), b = lat_t<T>(v * c + u * s);
    if (cache) {
      cache[pad32(rank) + i] = a;
      cache[pad32(rank) + half + i] = b;
    }
    if (kr_out) {
      kr_out[i] = a;
      kr_out[half + i] = b;
    }
  }
}

}  // namespace amd_ops
