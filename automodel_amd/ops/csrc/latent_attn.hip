// Latent attention, prompt side: everything around the projections and the
// flash kernel for packed sequences, plus a plain row-parallel attention that
// takes any head size and runs in f32 as well as bf16.
//
//   latent_prep      qkv rows -> rotated q (padded heads), normed latent,
//                    rotated shared key, and the cache rows, in one pass
//   latent_assemble  up-projected [k | v] + shared rotated key -> the padded
//                    per-head K and V the flash kernel reads
//   attn_rows        softmax(q k^T) v for one (token, head) per workgroup over
//                    an arbitrary strided key range, f32 arithmetic throughout

#include <torch/library.h>
#include <ATen/ATen.h>
#include <c10/hip/HIPStream.h>

#include "common.h"
#include "latent_attn.h"
#include "ops_api.h"

namespace amd_ops {

// grid Tp rows; rows [T, Tp) are padding and come out as zeros.
template <typename T, int V>
__global__ __launch_bounds__(256) void latent_prep_kernel(
    const T* __restrict__ qkv, const T* __restrict__ w, float eps,
    const float* __restrict__ cosb, const float* __restrict__ sinb, int n_pos, int cs_stride,
    const int* __restrict__ pos, const int* __restrict__ slot, T* __restrict__ cache,
    int n_slots, int max_len, int C, T* __restrict__ q_out, int QD, T* __restrict__ c_out,
    T* __restrict__ kr_out, int n_tok, int H, int dn, int dr, int rank) {
  __shared__ float red[8];
  const long t = blockIdx.x;
  const int hd = dn + dr, half = dr / 2;
  T* qo = q_out + t * (long)H * QD;
  T* co = c_out + t * (long)rank;
  T* ko = kr_out + t * (long)dr;
  if (t >= n_tok) {
    for (int i = threadIdx.x; i < H * QD; i += blockDim.x) qo[i] = lat_t<T>(0.f);
    for (int i = threadIdx.x; i < rank; i += blockDim.x) co[i] = lat_t<T>(0.f);
    for (int i = threadIdx.x; i < dr; i += blockDim.x) ko[i] = lat_t<T>(0.f);
    return;
  }
  const int p = min(max(pos[t], 0), n_pos - 1);
  const float* cosr = cosb + (long)p * cs_stride;
  const float* sinr = sinb + (long)p * cs_stride;
  const T* row = qkv + t * ((long)H * hd + rank + dr);

  // q: unrotated part copied, rotated part turned, head padding zeroed
  const int vn = dn / V, vp = (QD - hd) / V;
  for (int i = threadIdx.x; i < H * vn; i += blockDim.x) {
    const int h = i / vn, d = (i % vn) * V;
    *reinterpret_cast<LatPack<T, V>*>(qo + h * QD + d) =
        *reinterpret_cast<const LatPack<T, V>*>(row + h * hd + d);
  }
  const int vh = half / V;
  for (int i = threadIdx.x; i < H * vh; i += blockDim.x) {
    using P = LatPack<T, V>;
    const int h = i / vh, d = (i % vh) * V;
    const P u = *reinterpret_cast<const P*>(row + h * hd + dn + d);
    const P v = *reinterpret_cast<const P*>(row + h * hd + dn + half + d);
    const LatPack<float, V> c = *reinterpret_cast<const LatPack<float, V>*>(cosr + d);
    const LatPack<float, V> s = *reinterpret_cast<const LatPack<float, V>*>(sinr + d);
    P a, b;
#pragma unroll
    for (int j = 0; j < V; ++j) {
      a.v[j] = lat_t<T>(lat_f(u.v[j]) * c.v[j] - lat_f(v.v[j]) * s.v[j]);
      b.v[j] = lat_t<T>(lat_f(v.v[j]) * c.v[j] + lat_f(u.v[j]) * s.v[j]);
    }
    *reinterpret_cast<P*>(qo + h * QD + dn + d) = a;
    *reinterpret_cast<P*>(qo + h * QD + dn + half + d) = b;
  }
  for (int i = threadIdx.x; i < H * vp; i += blockDim.x) {
    const int h = i / vp, d = hd + (i % vp) * V;
#pragma unroll
    for (int j = 0; j < V; ++j) qo[h * QD + d + j] = lat_t<T>(0.f);
  }
  const long cr = cache ? cache_row(slot[t], pos[t], n_slots, max_len) : -1;
  latent_token<T>(row + (long)H * hd, w, eps, cosr, sinr, rank, dr,
                  cr >= 0 ? cache + cr * C : nullptr, co, ko, red);
}

template <typename T, int V>
__global__ __launch_bounds__(256) void latent_assemble_kernel(
    const T* __restrict__ kv, const T* __restrict__ kr, T* __restrict__ k_out,
    T* __restrict__ v_out, int n_tok, int H, int dn, int dr, int dv, int QD, int VD) {
  using P = LatPack<T, V>;
  const long t = blockIdx.x;
  const bool live = t < n_tok;
  const T* row = kv + t * (long)H * (dn + dv);
  const T* krow = kr + t * (long)dr;
  P zero;
#pragma unroll
  for (int j = 0; j < V; ++j) zero.v[j] = lat_t<T>(0.f);
  const int qv = QD / V, vv = VD / V;
  for (int i = threadIdx.x; i < H * qv; i += blockDim.x) {
    const int h = i / qv, d = (i % qv) * V;
    P x = zero;
    if (live && d < dn) x = *reinterpret_cast<const P*>(row + h * dn + d);
    else if (live && d < dn + dr) x = *reinterpret_cast<const P*>(krow + (d - dn));
    *reinterpret_cast<P*>(k_out + (t * H + h) * (long)QD + d) = x;
  }
  for (int i = threadIdx.x; i < H * vv; i += blockDim.x) {
    const int h = i / vv, d = (i % vv) * V;
    P x = zero;
    if (live && d < dv) x = *reinterpret_cast<const P*>(row + (long)H * dn + h * dv + d);
    *reinterpret_cast<P*>(v_out + (t * H + h) * (long)VD + d) = x;
  }
}

// Row-parallel attention. Key j of token t, head h: k + (base[t] + j) * k_rs +
// h * k_hs, j < count[t]; values alike. Online softmax over 256-key chunks:
// thread = key for the scores, thread = column for the value sum.
constexpr int AR_COLS = 8;            // value columns per thread (dv <= 2048)
template <typename T, typename TO>
__global__ __launch_bounds__(256) void attn_rows_kernel(
    const T* __restrict__ q, long q_rs, long q_hs, const T* __restrict__ k, long k_rs, long k_hs,
    const T* __restrict__ v, long v_rs, long v_hs, const long* __restrict__ base,
    const int* __restrict__ count, long n_rows, const T* __restrict__ sink, int per_k, int per_v,
    TO* __restrict__ out, int dq, int dv, float scale) {
  extern __shared__ float sm[];
  float* qs = sm;                     // dq
  float* ps = sm + dq;                // 256
  float* red = ps + 256;              // 4
  const int h = blockIdx.x;
  const long t = blockIdx.y;
  const int tid = threadIdx.x, lane = tid & 63, wid = tid >> 6;
  const long b0 = base[t];
  const int n = b0 < 0 ? 0 : (int)max(0L, min((long)count[t], n_rows - b0));
  for (int i = tid; i < dq; i += 256) qs[i] = lat_f(q[t * q_rs + h * q_hs + i]);
  float acc[AR_COLS];
#pragma unroll
  for (int c = 0; c < AR_COLS; ++c) acc[c] = 0.f;
  float m = -INFINITY, l = 0.f;
  __syncthreads();
  for (int j0 = 0; j0 < n; j0 += 256) {
    const int j = j0 + tid;
    float s = -INFINITY;
    if (j < n) {
      const T* kr = k + (b0 + j) * k_rs + h / per_k * k_hs;
      float d = 0.f;
      for (int i = 0; i < dq; ++i) d = fmaf(qs[i], lat_f(kr[i]), d);
      s = d * scale;
    }
    const float wm = wave_reduce_max(s);
    if (lane == 0) red[wid] = wm;
    __syncthreads();
    const float mn = fmaxf(m, fmaxf(fmaxf(red[0], red[1]), fmaxf(red[2], red[3])));
    const float alpha = expf(m - mn);             // m = -inf at first: 0
    const float p = expf(s - mn);
    ps[tid] = p;
    const float ws = wave_reduce_sum(p);
    __syncthreads();                              // red read, ps written
    if (lane == 0) red[wid] = ws;
    __syncthreads();
    l = l * alpha + (red[0] + red[1] + red[2] + red[3]);
    m = mn;
    const int jn = min(256, n - j0);
#pragma unroll
    for (int c = 0; c < AR_COLS; ++c) {
      const int col = tid + c * 256;
      if (col >= dv) continue;
      const T* vr = v + (b0 + j0) * v_rs + h / per_v * v_hs + col;
      float a = acc[c] * alpha;
      for (int jj = 0; jj < jn; ++jj) a = fmaf(ps[jj], lat_f(vr[jj * v_rs]), a);
      acc[c] = a;
    }
    __syncthreads();                              // before ps and red change
  }
  float own = 1.f;
  if (sink) {                                     // one more logit, without a key
    const float s = lat_f(sink[h]), mn = fmaxf(m, s);
    own = expf(m - mn);
    l = l * own + expf(s - mn);
  }
  const float inv = l > 0.f ? own / l : 0.f;
#pragma unroll
  for (int c = 0; c < AR_COLS; ++c) {
    const int col = tid + c * 256;
    if (col < dv)
      out[(t * gridDim.x + h) * (long)dv + col] = lat_t<TO>(acc[c] * inv);
  }
}

namespace {
bool is_t(const at::Tensor& x) {
  return x.scalar_type() == at::kBFloat16 || x.scalar_type() == at::kFloat;
}
void check_t(const at::Tensor& x, at::ScalarType dt, const char* what) {
  TORCH_CHECK(x.is_cuda() && x.is_contiguous() && x.scalar_type() == dt, what,
              ": contiguous GPU tensor of the activation dtype expected");
}
void check_i32(const at::Tensor& x, int64_t n, const char* what) {
  TORCH_CHECK(x.is_cuda() && x.is_contiguous() && x.scalar_type() == at::kInt && x.numel() == n,
              what, ": contiguous int32 GPU tensor, one value per token, expected");
}
}  // namespace

void latent_check_rope(const at::Tensor& cos, const at::Tensor& sin, int64_t rot) {
  TORCH_CHECK(cos.is_cuda() && sin.is_cuda() && cos.dim() == 2 && sin.sizes() == cos.sizes() &&
                  cos.scalar_type() == at::kFloat && sin.scalar_type() == at::kFloat &&
                  cos.is_contiguous() && sin.is_contiguous() && cos.size(0) >= 1 &&
                  cos.size(1) >= rot / 2 && rot % 2 == 0,
              "latent attention: cos/sin must be contiguous f32 [positions, >= rot/2]");
}

void latent_check_cache(const at::Tensor& cache, at::ScalarType dt, int64_t rank, int64_t rot) {
  TORCH_CHECK(cache.is_cuda() && cache.is_contiguous() && cache.dim() == 3 &&
                  cache.scalar_type() == dt && cache.size(2) == pad32(rank) + pad32(rot),
              "latent attention: cache must be [slots, max_len, pad32(rank) + pad32(rot)]");
}

std::tuple<at::Tensor, at::Tensor, at::Tensor> latent_prep(
    const at::Tensor& qkv, const at::Tensor& w, double eps, const at::Tensor& cos,
    const at::Tensor& sin, const at::Tensor& pos, const std::optional<at::Tensor>& slot,
    const std::optional<at::Tensor>& cache, int64_t heads, int64_t dn, int64_t dr,
    int64_t head_pad, int64_t rows_pad) {
  TORCH_CHECK(is_t(qkv) && qkv.dim() == 2, "latent_prep: qkv [T, N] bf16/f32");
  const auto dt = qkv.scalar_type();
  check_t(qkv, dt, "latent_prep qkv");
  check_t(w, dt, "latent_prep norm weight");
  const int64_t T = qkv.size(0), rank = w.numel();
  TORCH_CHECK(qkv.size(1) == heads * (dn + dr) + rank + dr && rank >= 1 && dn >= 0,
              "latent_prep: qkv width does not match the head sizes");
  TORCH_CHECK(head_pad >= dn + dr && rows_pad >= T, "latent_prep: padding too small");
  latent_check_rope(cos, sin, dr);
  check_i32(pos, T, "latent_prep pos");
  int n_slots = 0, max_len = 0, C = 0;
  if (cache.has_value()) {
    latent_check_cache(*cache, dt, rank, dr);
    TORCH_CHECK(slot.has_value(), "latent_prep: a cache needs slots");
    check_i32(*slot, T, "latent_prep slot");
    n_slots = cache->size(0), max_len = cache->size(1), C = cache->size(2);
  }
  auto q = at::empty({rows_pad, heads, head_pad}, qkv.options());
  auto c = at::empty({rows_pad, rank}, qkv.options());
  auto kr = at::empty({rows_pad, dr}, qkv.options());
  if (rows_pad == 0) return {q, c, kr};
  auto stream = c10::hip::getCurrentHIPStream();
  // every offset and row start a multiple of the vector, tables included
  auto all = [&](int64_t m) {
    return dn % m == 0 && dr % (2 * m) == 0 && head_pad % m == 0 && rank % m == 0 &&
           cos.size(1) % m == 0;
  };
#define LAUNCH(TT, VV)                                                                         \
  latent_prep_kernel<TT, VV><<<dim3(rows_pad), dim3(256), 0, stream>>>(                        \
      reinterpret_cast<const TT*>(qkv.data_ptr()), reinterpret_cast<const TT*>(w.data_ptr()),  \
      (float)eps, cos.data_ptr<float>(), sin.data_ptr<float>(), (int)cos.size(0),              \
      (int)cos.size(1), pos.data_ptr<int>(), cache ? slot->data_ptr<int>() : nullptr,          \
      cache ? reinterpret_cast<TT*>(cache->data_ptr()) : nullptr, n_slots, max_len, C,         \
      reinterpret_cast<TT*>(q.data_ptr()), (int)head_pad, reinterpret_cast<TT*>(c.data_ptr()), \
      reinterpret_cast<TT*>(kr.data_ptr()), (int)T, (int)heads, (int)dn, (int)dr, (int)rank)
  if (dt == at::kBFloat16) {
    if (all(8)) LAUNCH(bf16, 8); else if (all(4)) LAUNCH(bf16, 4); else LAUNCH(bf16, 1);
  } else {
    if (all(4)) LAUNCH(float, 4); else LAUNCH(float, 1);
  }
#undef LAUNCH
  HIP_CHECK_KERNEL();
  return {q, c, kr};
}

std::tuple<at::Tensor, at::Tensor> latent_assemble(const at::Tensor& kv, const at::Tensor& kr,
                                                   int64_t heads, int64_t dn, int64_t dv,
                                                   int64_t k_pad, int64_t v_pad, int64_t n_tok) {
  TORCH_CHECK(is_t(kv) && kv.dim() == 2 && kr.dim() == 2, "latent_assemble: kv [T,N], kr [Tp,rot]");
  const auto dt = kv.scalar_type();
  check_t(kv, dt, "latent_assemble kv");
  check_t(kr, dt, "latent_assemble kr");
  const int64_t Tp = kr.size(0), dr = kr.size(1);
  TORCH_CHECK(kv.size(1) == heads * (dn + dv) && n_tok <= kv.size(0) && n_tok <= Tp,
              "latent_assemble: kv shape");
  TORCH_CHECK(k_pad >= dn + dr && v_pad >= dv, "latent_assemble: padding too small");
  auto k = at::empty({Tp, heads, k_pad}, kv.options());
  auto v = at::empty({Tp, heads, v_pad}, kv.options());
  if (Tp == 0) return {k, v};
  auto stream = c10::hip::getCurrentHIPStream();
  auto all = [&](int64_t m) {
    return dn % m == 0 && dr % m == 0 && dv % m == 0 && k_pad % m == 0 && v_pad % m == 0;
  };
#define LAUNCH(TT, VV)                                                                        \
  latent_assemble_kernel<TT, VV><<<dim3(Tp), dim3(256), 0, stream>>>(                         \
      reinterpret_cast<const TT*>(kv.data_ptr()), reinterpret_cast<const TT*>(kr.data_ptr()), \
      reinterpret_cast<TT*>(k.data_ptr()), reinterpret_cast<TT*>(v.data_ptr()), (int)n_tok,   \
      (int)heads, (int)dn, (int)dr, (int)dv, (int)k_pad, (int)v_pad)
  if (dt == at::kBFloat16) {
    if (all(8)) LAUNCH(bf16, 8); else if (all(2)) LAUNCH(bf16, 2); else LAUNCH(bf16, 1);
  } else {
    if (all(4)) LAUNCH(float, 4); else LAUNCH(float, 1);
  }
#undef LAUNCH
  HIP_CHECK_KERNEL();
  return {k, v};
}

// q [T, H, dq]; k/v [rows, Hk, d], query heads in equal groups per key head (v
// may be a column slice of k). base [T] int64, count [T] int32; sink [H], a
// logit without a key. -> [T, H, dv]
at::Tensor attn_rows(const at::Tensor& q, const at::Tensor& k, const at::Tensor& v,
                     const at::Tensor& base, const at::Tensor& count, double scale,
                     bool out_f32, const std::optional<at::Tensor>& sink) {
  TORCH_CHECK(is_t(q) && q.is_cuda() && q.dim() == 3 && k.dim() == 3 && v.dim() == 3,
              "attn_rows: q [T,H,dq], k/v [rows,Hk,d]");
  const auto dt = q.scalar_type();
  TORCH_CHECK(k.is_cuda() && v.is_cuda() && k.scalar_type() == dt && v.scalar_type() == dt,
              "attn_rows: dtypes differ");
  TORCH_CHECK(q.stride(2) == 1 && k.stride(2) == 1 && v.stride(2) == 1,
              "attn_rows: head dims must be contiguous");
  const int64_t T = q.size(0), H = q.size(1), dq = q.size(2), dv = v.size(2);
  TORCH_CHECK(k.size(1) >= 1 && v.size(1) >= 1 && H % k.size(1) == 0 && H % v.size(1) == 0 &&
                  k.size(2) >= dq && k.size(0) == v.size(0),
              "attn_rows: k/v shapes");
  TORCH_CHECK(dq <= 8192 && dv <= 256 * AR_COLS && T <= 65535 * 16L, "attn_rows: sizes");
  TORCH_CHECK(base.is_cuda() && base.is_contiguous() && base.scalar_type() == at::kLong &&
                  base.numel() == T, "attn_rows: base int64 [T]");
  check_i32(count, T, "attn_rows count");
  if (sink)
    TORCH_CHECK(sink->is_cuda() && sink->is_contiguous() && sink->numel() == H &&
                    sink->scalar_type() == dt, "attn_rows: sink [H]");
  auto out = at::empty({T, H, dv}, q.options().dtype(out_f32 ? at::kFloat : dt));
  if (T == 0) return out;
  auto stream = c10::hip::getCurrentHIPStream();
  const size_t smem = (dq + 256 + 8) * sizeof(float);
  const int per_k = (int)(H / k.size(1)), per_v = (int)(H / v.size(1));
  constexpr int64_t STEP = 32768;                       // grid.y limit is 65535
#define LAUNCH(TT, TO)                                                                         \
  attn_rows_kernel<TT, TO><<<dim3(H, n), dim3(256), smem, stream>>>(                           \
      reinterpret_cast<const TT*>(q.data_ptr()) + t0 * q.stride(0), q.stride(0), q.stride(1),  \
      reinterpret_cast<const TT*>(k.data_ptr()), k.stride(0), k.stride(1),                     \
      reinterpret_cast<const TT*>(v.data_ptr()), v.stride(0), v.stride(1),                     \
      base.data_ptr<long>() + t0, count.data_ptr<int>() + t0, (long)k.size(0),                 \
      sink ? reinterpret_cast<const TT*>(sink->data_ptr()) : nullptr, per_k, per_v,             \
      reinterpret_cast<TO*>(out.data_ptr()) + t0 * H * dv, (int)dq, (int)dv, (float)scale)
  for (int64_t t0 = 0; t0 < T; t0 += STEP) {
    const int64_t n = std::min(STEP, T - t0);
    if (dt == at::kFloat) LAUNCH(float, float);
    else if (out_f32) LAUNCH(bf16, float);
    else LAUNCH(bf16, bf16);
  }
#undef LAUNCH
  HIP_CHECK_KERNEL();
  return out;
}

}  // namespace amd_ops
