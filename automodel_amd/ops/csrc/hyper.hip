// Hyper-connections: a residual of S parallel f32 streams [T, S, W] around the
// sublayers (inference).
//
//   hyper_embed   every stream = scale * table[id]; h = rms(sum_s in[s] x_s) * w
//   hyper_step    x_t <- sum_s mix[s, t] x_s + out[t] * y, then the next
//                 sublayer's input h = rms(sum_t in[t] x_t) * w
//
// One pass over the streams per sublayer: a workgroup owns a token, a thread
// owns columns of all its streams, so the old values are in registers when the
// new ones are formed. y may be given as two branches whose normed mean it is:
// y = (rms(a) * wa + rms(b) * wb) / 2. Without `in` all streams count once
// (the model's output). T is bf16 or f32.

#include <torch/library.h>
#include <ATen/ATen.h>
#include <c10/hip/HIPStream.h>

#include "elem.h"
#include "ops_api.h"

namespace amd_ops {

namespace {

__device__ __forceinline__ float inv_root(float sumsq, int n, float eps) {
  return 1.0f / sqrtf(sumsq / (float)n + eps);
}

// two sums over the block at once
__device__ __forceinline__ float2 block_sum2(float a, float b, float2* scratch) {
  const int lane = threadIdx.x & (WAVE_SIZE - 1), wid = threadIdx.x / WAVE_SIZE;
  a = wave_reduce_sum(a);
  b = wave_reduce_sum(b);
  if (lane == 0) scratch[wid] = float2{a, b};
  __syncthreads();
  float2 t{0.f, 0.f};
  for (int i = 0; i < (int)blockDim.x / WAVE_SIZE; ++i) {
    t.x += scratch[i].x;
    t.y += scratch[i].y;
  }
  __syncthreads();
  return t;
}

template <typename T, int V>
__global__ void hyper_embed_kernel(const long* __restrict__ ids, const T* __restrict__ table,
                                   float scale, const T* __restrict__ w_in,
                                   const T* __restrict__ w_norm, float* __restrict__ x,
                                   T* __restrict__ h, int S, int W, long vocab, float eps) {
  __shared__ float2 red[16];
  const long t = blockIdx.x;
  const long id = min(max(ids[t], 0L), vocab - 1);
  const T* src = table + id * W;
  float c = 0.f;                                   // sum of the input weights
  for (int s = 0; s < S; ++s) c += to_f32(w_in[s]);
  float ss = 0.f;
  for (int i = threadIdx.x * V; i < W; i += blockDim.x * V) {
    float a[V];
    load_vec<T, V>(src + i, a);
#pragma unroll
    for (int j = 0; j < V; ++j) {
      a[j] *= scale;
      ss = fmaf(c * a[j], c * a[j], ss);
    }
    for (int s = 0; s < S; ++s) store_vec<float, V>(x + (t * S + s) * W + i, a);
  }
  const float inv = inv_root(block_sum2(ss, 0.f, red).x, W, eps);
  for (int i = threadIdx.x * V; i < W; i += blockDim.x * V) {
    float a[V], g[V];
    load_vec<T, V>(src + i, a);
    load_vec<T, V>(w_norm + i, g);
#pragma unroll
    for (int j = 0; j < V; ++j) a[j] = c * (a[j] * scale) * inv * g[j];
    store_vec<T, V>(h + t * W + i, a);
  }
}

// SM: streams held in registers, S <= SM.
template <typename T, int V, int SM>
__global__ void hyper_step_kernel(float* __restrict__ x, const T* __restrict__ ya,
                                  const T* __restrict__ yb, const T* __restrict__ wa,
                                  const T* __restrict__ wb, const T* __restrict__ w_mix,
                                  const T* __restrict__ w_out, const T* __restrict__ w_in,
                                  const T* __restrict__ w_norm, T* __restrict__ h, int S, int W,
                                  float eps, bool keep) {
  __shared__ float2 red[16];
  extern __shared__ __attribute__((aligned(16))) float us[];
  const long t = blockIdx.x;
  float ia = 1.f, ib = 0.f;
  if (yb != nullptr) {                             // uniform over the grid
    float sa = 0.f, sb = 0.f;
    for (int i = threadIdx.x * V; i < W; i += blockDim.x * V) {
      float a[V], b[V];
      load_vec<T, V>(ya + t * W + i, a);
      load_vec<T, V>(yb + t * W + i, b);
#pragma unroll
      for (int j = 0; j < V; ++j) {
        sa = fmaf(a[j], a[j], sa);
        sb = fmaf(b[j], b[j], sb);
      }
    }
    const float2 r = block_sum2(sa, sb, red);
    ia = 0.5f * inv_root(r.x, W, eps);
    ib = 0.5f * inv_root(r.y, W, eps);
  }
  float ss = 0.f;
  for (int i = threadIdx.x * V; i < W; i += blockDim.x * V) {
    float y[V], u[V], xs[SM][V];
    load_vec<T, V>(ya + t * W + i, y);
    if (yb != nullptr) {
      float b[V], ga[V], gb[V];
      load_vec<T, V>(yb + t * W + i, b);
      load_vec<T, V>(wa + i, ga);
      load_vec<T, V>(wb + i, gb);
#pragma unroll
      for (int j = 0; j < V; ++j) y[j] = y[j] * ia * ga[j] + b[j] * ib * gb[j];
    }
#pragma unroll
    for (int s = 0; s < SM; ++s)
      if (s < S) load_vec<float, V>(x + (t * S + s) * W + i, xs[s]);
#pragma unroll
    for (int j = 0; j < V; ++j) u[j] = 0.f;
#pragma unroll
    for (int q = 0; q < SM; ++q) {
      if (q >= S) break;
      const float o = to_f32(w_out[q]), c = w_in ? to_f32(w_in[q]) : 1.f;
      float n[V];
#pragma unroll
      for (int j = 0; j < V; ++j) n[j] = o * y[j];
#pragma unroll
      for (int s = 0; s < SM; ++s) {
        if (s >= S) break;
        const float m = to_f32(w_mix[s * S + q]);
#pragma unroll
        for (int j = 0; j < V; ++j) n[j] = fmaf(m, xs[s][j], n[j]);
      }
      if (keep) store_vec<float, V>(x + (t * S + q) * W + i, n);
#pragma unroll
      for (int j = 0; j < V; ++j) u[j] = fmaf(c, n[j], u[j]);
    }
#pragma unroll
    for (int j = 0; j < V; ++j) ss = fmaf(u[j], u[j], ss);
    store_vec<float, V>(us + i, u);
  }
  const float inv = inv_root(block_sum2(ss, 0.f, red).x, W, eps);
  for (int i = threadIdx.x * V; i < W; i += blockDim.x * V) {
    float u[V], g[V];
    load_vec<float, V>(us + i, u);
    load_vec<T, V>(w_norm + i, g);
#pragma unroll
    for (int j = 0; j < V; ++j) u[j] = u[j] * inv * g[j];
    store_vec<T, V>(h + t * W + i, u);
  }
}

// min(g, L) * sigmoid(alpha * min(g, L)) * (clamp(u, -L, L) + 1) on rows [g | u]
template <typename T, int V>
__global__ void clamped_glu_kernel(const T* __restrict__ gu, T* __restrict__ out, long rows,
                                   int F, float limit, float alpha) {
  const int c = (blockIdx.y * blockDim.x + threadIdx.x) * V;
  if (c >= F) return;
  for (long r = blockIdx.x; r < rows; r += gridDim.x) {
    float g[V], u[V];
    load_vec<T, V>(gu + r * 2 * F + c, g);
    load_vec<T, V>(gu + r * 2 * F + F + c, u);
#pragma unroll
    for (int j = 0; j < V; ++j) {
      const float a = fminf(g[j], limit);
      const float b = fminf(fmaxf(u[j], -limit), limit);
      g[j] = a * sigmoid_f(alpha * a) * (b + 1.f);
    }
    store_vec<T, V>(out + r * F + c, g);
  }
}

void check_t(const at::Tensor& t, at::ScalarType dt, int64_t n, const char* what) {
  TORCH_CHECK(t.is_cuda() && t.is_contiguous() && t.scalar_type() == dt && t.numel() == n, what,
              ": contiguous GPU tensor of ", n, " ", dt, " elements expected");
}

int row_threads(int W, int V, long rows) {
  const int cap = rows <= 64 ? 1024 : 256;         // few rows: latency, not throughput
  return std::min(cap, (ceil_div_i(W, V) + WAVE_SIZE - 1) / WAVE_SIZE * WAVE_SIZE);
}

constexpr int64_t MAX_STREAMS = 16, MAX_WIDTH = 16384;

}  // namespace

#define PTR(t) reinterpret_cast<scalar*>((t).data_ptr())
#define OPT(t) ((t).has_value() ? reinterpret_cast<scalar*>((t)->data_ptr()) : nullptr)

std::tuple<at::Tensor, at::Tensor> hyper_embed(const at::Tensor& ids, const at::Tensor& table,
                                               double scale, const at::Tensor& w_in,
                                               const at::Tensor& w_norm, double eps) {
  TORCH_CHECK(ids.is_cuda() && ids.is_contiguous() && ids.scalar_type() == at::kLong,
              "hyper_embed: ids must be contiguous int64");
  TORCH_CHECK(table.dim() == 2, "hyper_embed: table [V, W]");
  const auto dt = table.scalar_type();
  TORCH_CHECK(dt == at::kBFloat16 || dt == at::kFloat, "hyper_embed: bf16 or f32");
  const int64_t W = table.size(1), S = w_in.numel(), T = ids.numel();
  TORCH_CHECK(S >= 1 && S <= MAX_STREAMS && W >= 1 && W <= MAX_WIDTH, "hyper_embed: sizes");
  check_t(table, dt, table.numel(), "hyper_embed table");
  check_t(w_in, dt, S, "hyper_embed in");
  check_t(w_norm, dt, W, "hyper_embed norm");
  auto x = at::empty({T, S, W}, table.options().dtype(at::kFloat));
  auto h = at::empty({T, W}, table.options());
  if (T == 0) return {x, h};
  auto stream = c10::hip::getCurrentHIPStream();
  AMD_DISPATCH_T_V(dt, W % 8 == 0, {
    hyper_embed_kernel<scalar, V><<<dim3(T), dim3(row_threads(W, V, T)), 0, stream>>>(
        ids.data_ptr<long>(), PTR(table), (float)scale, PTR(w_in), PTR(w_norm),
        x.data_ptr<float>(), PTR(h), (int)S, (int)W, table.size(0), (float)eps);
  });
  HIP_CHECK_KERNEL();
  return {x, h};
}

at::Tensor hyper_step(at::Tensor x, const at::Tensor& y, const std::optional<at::Tensor>& y2,
                      const std::optional<at::Tensor>& w_y, const std::optional<at::Tensor>& w_y2,
                      const at::Tensor& w_mix, const at::Tensor& w_out,
                      const std::optional<at::Tensor>& w_in, const at::Tensor& w_norm, double eps,
                      bool keep) {
  TORCH_CHECK(x.dim() == 3, "hyper_step: x [T, S, W]");
  const int64_t T = x.size(0), S = x.size(1), W = x.size(2);
  const auto dt = w_norm.scalar_type();
  TORCH_CHECK(dt == at::kBFloat16 || dt == at::kFloat, "hyper_step: bf16 or f32");
  TORCH_CHECK(S >= 1 && S <= MAX_STREAMS && W >= 1 && W <= MAX_WIDTH, "hyper_step: sizes");
  check_t(x, at::kFloat, T * S * W, "hyper_step x");
  check_t(y, dt, T * W, "hyper_step y");
  check_t(w_norm, dt, W, "hyper_step norm");
  check_t(w_mix, dt, S * S, "hyper_step mix");
  check_t(w_out, dt, S, "hyper_step out");
  if (w_in) check_t(*w_in, dt, S, "hyper_step in");
  if (y2) {
    TORCH_CHECK(w_y && w_y2, "hyper_step: two branches need their norm weights");
    check_t(*y2, dt, T * W, "hyper_step y2");
    check_t(*w_y, dt, W, "hyper_step branch norm");
    check_t(*w_y2, dt, W, "hyper_step branch norm");
  }
  auto h = at::empty({T, W}, y.options());
  if (T == 0) return h;
  auto stream = c10::hip::getCurrentHIPStream();
  // 4 columns per thread: S streams of them stay in registers
#define LAUNCH(V, SM)                                                                        \
  hyper_step_kernel<scalar, V, SM>                                                           \
      <<<dim3(T), dim3(row_threads(W, V, T)), W * sizeof(float), stream>>>(                  \
          x.data_ptr<float>(), PTR(y), OPT(y2), OPT(w_y), OPT(w_y2), PTR(w_mix), PTR(w_out), \
          OPT(w_in), PTR(w_norm), PTR(h), (int)S, (int)W, (float)eps, keep)
#define BY_STREAMS(V)              \
  if (S == 1) LAUNCH(V, 1);        \
  else if (S == 2) LAUNCH(V, 2);   \
  else if (S <= 4) LAUNCH(V, 4);   \
  else if (S <= 8) LAUNCH(V, 8);   \
  else LAUNCH(V, 16);
  AMD_DISPATCH_T(dt, {
    if (W % 4 == 0) { BY_STREAMS(4) } else { BY_STREAMS(1) }
  });
#undef BY_STREAMS
#undef LAUNCH
  HIP_CHECK_KERNEL();
  return h;
}

at::Tensor clamped_glu(const at::Tensor& gu, double limit, double alpha) {
  TORCH_CHECK(gu.is_cuda() && gu.is_contiguous() && gu.dim() == 2 && gu.size(1) % 2 == 0 &&
                  (gu.scalar_type() == at::kBFloat16 || gu.scalar_type() == at::kFloat),
              "clamped_glu: contiguous [T, 2F] bf16/f32 GPU tensor");
  const int64_t T = gu.size(0), F = gu.size(1) / 2;
  auto out = at::empty({T, F}, gu.options());
  if (T * F == 0) return out;
  auto stream = c10::hip::getCurrentHIPStream();
  AMD_DISPATCH_T_V(gu.scalar_type(), F % 8 == 0, {
    const int threads = std::min(256, ceil_div_i(F, V * WAVE_SIZE) * WAVE_SIZE);
    const dim3 grid(std::min<int64_t>(T, 2048), ceil_div_i(F, V * threads));
    clamped_glu_kernel<scalar, V><<<grid, dim3(threads), 0, stream>>>(
        PTR(gu), PTR(out), T, (int)F, (float)limit, (float)alpha);
  });
  HIP_CHECK_KERNEL();
  return out;
}

#undef PTR
#undef OPT

}  // namespace amd_ops
