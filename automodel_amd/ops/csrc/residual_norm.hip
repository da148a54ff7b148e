// RMS norms around a 32-bit residual stream (inference).
//
// Models that keep the residual sum in f32 pay for it in elementwise traffic
// unless norm, scaled residual add and the next norm share one pass: here a
// row is read once, kept in LDS as f32 between the two reductions, and the
// updated residual and the next sublayer's input leave together.
//   embed_rms_norm      x = rms(table[id]) * w                    (f32 out)
//   residual_rms_norm   h = rms(x) * w                            (f32 -> T)
//   residual_add_norm   x += mult * rms(y) * w_post; h = rms(x) * w_next
//   concat_cast         [a ; b] rows, f32 -> T                     (loop input)
//   relu2_              elementwise max(x, 0)^2 in place
// T is bf16 or f32 (the 32-bit model). One workgroup per row; 4-wide accesses
// when the width allows, scalar otherwise, so any width works.

#include <torch/library.h>
#include <ATen/ATen.h>
#include <c10/hip/HIPStream.h>

#include "common.h"
#include "ops_api.h"

namespace amd_ops {

namespace {

__device__ __forceinline__ float to_f(float x) { return x; }
__device__ __forceinline__ float to_f(bf16 x) { return bf2f(x); }
__device__ __forceinline__ void from_f(float x, float& o) { o = x; }
__device__ __forceinline__ void from_f(float x, bf16& o) { o = f2bf(x); }

template <typename T, int V>
struct alignas(sizeof(T) * V) Pack {
  T v[V];
};

template <typename T, int V>
__device__ __forceinline__ void load_f(const T* p, float (&o)[V]) {
  const Pack<T, V> t = *reinterpret_cast<const Pack<T, V>*>(p);
#pragma unroll
  for (int j = 0; j < V; ++j) o[j] = to_f(t.v[j]);
}
template <typename T, int V>
__device__ __forceinline__ void store_f(T* p, const float (&x)[V]) {
  Pack<T, V> t;
#pragma unroll
  for (int j = 0; j < V; ++j) from_f(x[j], t.v[j]);
  *reinterpret_cast<Pack<T, V>*>(p) = t;
}

// 1/sqrt in full precision (v_rsq_f32 alone is an approximation)
__device__ __forceinline__ float inv_rms(float sumsq, int n, float eps) {
  return 1.0f / sqrtf(sumsq / (float)n + eps);
}

// One row; every thread touches only its own columns of the LDS row, so the
// reductions are the only barriers.
template <typename T, int V>
__global__ void embed_rms_norm_kernel(const long* __restrict__ ids, const T* __restrict__ table,
                                      const T* __restrict__ w, float* __restrict__ x,
                                      int W, long vocab, float eps) {
  __shared__ float red[16];
  const long row = blockIdx.x;
  long id = ids[row];
  id = id < 0 ? 0 : (id >= vocab ? vocab - 1 : id);
  const T* src = table + id * W;
  float ss = 0.f;
  for (int i = threadIdx.x * V; i < W; i += blockDim.x * V) {
    float a[V];
    load_f<T, V>(src + i, a);
#pragma unroll
    for (int j = 0; j < V; ++j) ss = fmaf(a[j], a[j], ss);
  }
  const float inv = inv_rms(block_reduce_sum(ss, red), W, eps);
  for (int i = threadIdx.x * V; i < W; i += blockDim.x * V) {
    float a[V], g[V];
    load_f<T, V>(src + i, a);
    load_f<T, V>(w + i, g);
#pragma unroll
    for (int j = 0; j < V; ++j) a[j] = a[j] * inv * g[j];
    store_f<float, V>(x + row * W + i, a);
  }
}

template <typename T, int V>
__global__ void residual_rms_norm_kernel(const float* __restrict__ x, const T* __restrict__ w,
                                         T* __restrict__ h, int W, float eps) {
  __shared__ float red[16];
  extern __shared__ __attribute__((aligned(16))) float xs[];
  const long row = blockIdx.x;
  float ss = 0.f;
  for (int i = threadIdx.x * V; i < W; i += blockDim.x * V) {
    float a[V];
    load_f<float, V>(x + row * W + i, a);
    store_f<float, V>(xs + i, a);
#pragma unroll
    for (int j = 0; j < V; ++j) ss = fmaf(a[j], a[j], ss);
  }
  const float inv = inv_rms(block_reduce_sum(ss, red), W, eps);
  for (int i = threadIdx.x * V; i < W; i += blockDim.x * V) {
    float a[V], g[V];
    load_f<float, V>(xs + i, a);
    load_f<T, V>(w + i, g);
#pragma unroll
    for (int j = 0; j < V; ++j) a[j] = a[j] * inv * g[j];
    store_f<T, V>(h + row * W + i, a);
  }
}

template <typename T, int V>
__global__ void residual_add_norm_kernel(float* __restrict__ x, const T* __restrict__ y,
                                         const T* __restrict__ w_post, float mult, float eps_post,
                                         const T* __restrict__ w_next, float eps_next,
                                         T* __restrict__ h, int W) {
  __shared__ float red[16];
  extern __shared__ __attribute__((aligned(16))) float xs[];
  const long row = blockIdx.x;
  float ss = 0.f;
  for (int i = threadIdx.x * V; i < W; i += blockDim.x * V) {
    float a[V];
    load_f<T, V>(y + row * W + i, a);
    store_f<float, V>(xs + i, a);
#pragma unroll
    for (int j = 0; j < V; ++j) ss = fmaf(a[j], a[j], ss);
  }
  const float inv = inv_rms(block_reduce_sum(ss, red), W, eps_post);
  ss = 0.f;
  for (int i = threadIdx.x * V; i < W; i += blockDim.x * V) {
    float a[V], g[V], r[V];
    load_f<float, V>(xs + i, a);
    load_f<T, V>(w_post + i, g);
    load_f<float, V>(x + row * W + i, r);
#pragma unroll
    for (int j = 0; j < V; ++j) {
      r[j] = fmaf(mult, a[j] * inv * g[j], r[j]);
      ss = fmaf(r[j], r[j], ss);
    }
    store_f<float, V>(x + row * W + i, r);
    store_f<float, V>(xs + i, r);
  }
  if (w_next == nullptr) return;                      // uniform over the grid
  const float inv2 = inv_rms(block_reduce_sum(ss, red), W, eps_next);
  for (int i = threadIdx.x * V; i < W; i += blockDim.x * V) {
    float a[V], g[V];
    load_f<float, V>(xs + i, a);
    load_f<T, V>(w_next + i, g);
#pragma unroll
    for (int j = 0; j < V; ++j) a[j] = a[j] * inv2 * g[j];
    store_f<T, V>(h + row * W + i, a);
  }
}

template <typename T, int V>
__global__ void concat_cast_kernel(const float* __restrict__ a, const float* __restrict__ b,
                                   T* __restrict__ out, int W) {
  const long row = blockIdx.x;
  for (int i = threadIdx.x * V; i < 2 * W; i += blockDim.x * V) {
    float t[V];
    load_f<float, V>(i < W ? a + row * W + i : b + row * W + (i - W), t);
    store_f<T, V>(out + row * 2 * W + i, t);
  }
}

template <typename T, int V>
__global__ void relu2_kernel(T* __restrict__ x, long n) {
  const long step = (long)gridDim.x * blockDim.x * V;
  for (long i = ((long)blockIdx.x * blockDim.x + threadIdx.x) * V; i < n; i += step) {
    float a[V];
    load_f<T, V>(x + i, a);
#pragma unroll
    for (int j = 0; j < V; ++j) {
      const float r = fmaxf(a[j], 0.f);
      a[j] = r * r;
    }
    store_f<T, V>(x + i, a);
  }
}

int row_threads(int W, int V, long rows) {
  const int need = (W + V - 1) / V;
  const int cap = rows <= 64 ? 1024 : 256;            // few rows: latency, not throughput
  return std::min(cap, ((need + WAVE_SIZE - 1) / WAVE_SIZE) * WAVE_SIZE);
}

void check_rows(const at::Tensor& x, const char* who) {
  TORCH_CHECK(x.is_cuda() && x.dim() == 2 && x.is_contiguous() && x.scalar_type() == at::kFloat,
              who, ": residual must be a contiguous f32 [T, W] GPU tensor");
  TORCH_CHECK(x.size(1) >= 1 && x.size(1) <= 16384, who, ": width out of range");
}
void check_vec(const at::Tensor& w, int64_t n, const char* who) {
  TORCH_CHECK(w.is_cuda() && w.is_contiguous() && w.numel() == n &&
                  (w.scalar_type() == at::kBFloat16 || w.scalar_type() == at::kFloat),
              who, ": weight must be a contiguous bf16/f32 [W] GPU tensor");
}

}  // namespace

// Runs the statement with `scalar` = bf16/float by DT and `V` = 4/1 by divisibility.
#define DISPATCH_T_V(DT, NELEM, ...)                               \
  do {                                                             \
    const bool vec_ = ((NELEM) % 4) == 0;                          \
    if ((DT) == at::kBFloat16) {                                   \
      using scalar = bf16;                                         \
      if (vec_) { constexpr int V = 4; __VA_ARGS__ } else { constexpr int V = 1; __VA_ARGS__ } \
    } else {                                                       \
      using scalar = float;                                        \
      if (vec_) { constexpr int V = 4; __VA_ARGS__ } else { constexpr int V = 1; __VA_ARGS__ } \
    }                                                              \
  } while (0)

#define PTR(t) reinterpret_cast<scalar*>((t).data_ptr())

at::Tensor embed_rms_norm(const at::Tensor& ids, const at::Tensor& table, const at::Tensor& w,
                          double eps) {
  TORCH_CHECK(ids.is_cuda() && ids.is_contiguous() && ids.scalar_type() == at::kLong,
              "embed_rms_norm: ids must be contiguous int64");
  TORCH_CHECK(table.is_cuda() && table.dim() == 2 && table.is_contiguous(),
              "embed_rms_norm: table [V, W]");
  const int W = (int)table.size(1);
  check_vec(w, W, "embed_rms_norm");
  TORCH_CHECK(w.scalar_type() == table.scalar_type(), "embed_rms_norm: dtype mismatch");
  const long T = ids.numel();
  auto x = at::empty({T, W}, table.options().dtype(at::kFloat));
  if (T == 0) return x;
  auto stream = c10::hip::getCurrentHIPStream();
  DISPATCH_T_V(w.scalar_type(), W, {
    embed_rms_norm_kernel<scalar, V><<<dim3(T), dim3(row_threads(W, V, T)), 0, stream>>>(
        ids.data_ptr<long>(), PTR(table), PTR(w), x.data_ptr<float>(), W, table.size(0),
        (float)eps);
  });
  HIP_CHECK_KERNEL();
  return x;
}

at::Tensor residual_rms_norm(const at::Tensor& x, const at::Tensor& w, double eps) {
  check_rows(x, "residual_rms_norm");
  const int W = (int)x.size(1);
  const long T = x.size(0);
  check_vec(w, W, "residual_rms_norm");
  auto h = at::empty({T, W}, w.options());
  if (T == 0) return h;
  auto stream = c10::hip::getCurrentHIPStream();
  DISPATCH_T_V(w.scalar_type(), W, {
    residual_rms_norm_kernel<scalar, V>
        <<<dim3(T), dim3(row_threads(W, V, T)), W * sizeof(float), stream>>>(
            x.data_ptr<float>(), PTR(w), PTR(h), W, (float)eps);
  });
  HIP_CHECK_KERNEL();
  return h;
}

// x is updated in place; returns h (empty when w_next is not given).
at::Tensor residual_add_norm(at::Tensor x, const at::Tensor& y, const at::Tensor& w_post,
                             double mult, double eps_post,
                             const std::optional<at::Tensor>& w_next, double eps_next) {
  check_rows(x, "residual_add_norm");
  const int W = (int)x.size(1);
  const long T = x.size(0);
  check_vec(w_post, W, "residual_add_norm");
  TORCH_CHECK(y.is_cuda() && y.is_contiguous() && y.numel() == T * W &&
                  y.scalar_type() == w_post.scalar_type(),
              "residual_add_norm: y must be contiguous [T, W] in the weight dtype");
  const bool next = w_next.has_value();
  if (next) {
    check_vec(*w_next, W, "residual_add_norm");
    TORCH_CHECK(w_next->scalar_type() == w_post.scalar_type(), "residual_add_norm: dtype");
  }
  auto h = at::empty({next ? T : 0, W}, y.options());
  if (T == 0) return h;
  auto stream = c10::hip::getCurrentHIPStream();
  DISPATCH_T_V(w_post.scalar_type(), W, {
    residual_add_norm_kernel<scalar, V>
        <<<dim3(T), dim3(row_threads(W, V, T)), W * sizeof(float), stream>>>(
            x.data_ptr<float>(), PTR(y), PTR(w_post), (float)mult, (float)eps_post,
            next ? PTR(*w_next) : nullptr, (float)eps_next, next ? PTR(h) : nullptr, W);
  });
  HIP_CHECK_KERNEL();
  return h;
}

at::Tensor concat_cast(const at::Tensor& a, const at::Tensor& b, bool to_bf16) {
  check_rows(a, "concat_cast");
  check_rows(b, "concat_cast");
  TORCH_CHECK(a.sizes() == b.sizes(), "concat_cast: shapes differ");
  const int W = (int)a.size(1);
  const long T = a.size(0);
  const auto dt = to_bf16 ? at::kBFloat16 : at::kFloat;
  auto out = at::empty({T, 2 * W}, a.options().dtype(dt));
  if (T == 0) return out;
  auto stream = c10::hip::getCurrentHIPStream();
  DISPATCH_T_V(dt, W, {
    concat_cast_kernel<scalar, V><<<dim3(T), dim3(row_threads(2 * W, V, T)), 0, stream>>>(
        a.data_ptr<float>(), b.data_ptr<float>(), PTR(out), W);
  });
  HIP_CHECK_KERNEL();
  return out;
}

at::Tensor relu2_(at::Tensor x) {
  TORCH_CHECK(x.is_cuda() && x.is_contiguous() &&
                  (x.scalar_type() == at::kBFloat16 || x.scalar_type() == at::kFloat),
              "relu2_: contiguous bf16/f32 GPU tensor");
  const long n = x.numel();
  if (n == 0) return x;
  auto stream = c10::hip::getCurrentHIPStream();
  if (x.scalar_type() == at::kBFloat16 && n % 8 == 0) {
    const int blocks = (int)std::min<long>((n / 8 + 255) / 256, 4096);
    relu2_kernel<bf16, 8><<<dim3(blocks), dim3(256), 0, stream>>>(
        reinterpret_cast<bf16*>(x.data_ptr()), n);
  } else {
    DISPATCH_T_V(x.scalar_type(), n, {
      const int blocks = (int)std::min<long>((n / V + 255) / 256, 4096);
      relu2_kernel<scalar, V><<<dim3(blocks), dim3(256), 0, stream>>>(PTR(x), n);
    });
  }
  HIP_CHECK_KERNEL();
  return x;
}

#undef PTR
#undef DISPATCH_T_V

}  // namespace amd_ops
