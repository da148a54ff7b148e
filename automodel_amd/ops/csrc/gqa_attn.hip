// Grouped-head attention over packed sequences and a slot cache, optionally in
// chunks of the sequence (a token sees its own chunk only) and with a sink (one
// learned logit per head in the softmax's denominator).
//
//   gqa_prep          partial rotation of q and k, head padding, cache rows
//   gqa_store_v       prompt values into the blocked cache
//   gqa_decode_attn   split-KV attention of one token per sequence; the heads
//                     of a group are columns of 16x16x32 MFMAs
//   gqa_decode_merge  merges the splits and the sink
//
// Caches hold one chunk (position modulo chunk), since no earlier key is ever
// read. Two layouts:
//   plain    K [slots, rows, G, d], V [slots, rows, G, dv]
//   blocked  K [slots, G, rows, pad32(d)], V [slots, G, rows/32, pad16(dv), 32]
// In the blocked one both operands of both products are 16-byte loads straight
// from memory, without LDS: a wave's score tiles leave lane (g, head) with keys
// 4g..4g+3 of two 16-key tiles, and V keeps the 32 keys of a block in that
// order, so the probabilities are the next product's operand as they are.
// Prompts run through the flash kernel (bf16) or attn_rows.

#include <torch/library.h>
#include <ATen/ATen.h>
#include <c10/hip/HIPStream.h>

#include "elem.h"
#include "ops_api.h"

namespace amd_ops {

typedef __bf16 gqa_bf16x8 __attribute__((ext_vector_type(8)));
typedef float gqa_f32x4 __attribute__((ext_vector_type(4)));

namespace {

// place of key `row` within its block of 32: lane group (row % 16) / 4 owns 8
__host__ __device__ constexpr int v_place(int row) {
  return 8 * ((row & 15) >> 2) + 4 * ((row >> 4) & 1) + (row & 3);
}

struct GqaCache {
  void* k;
  void* v;
  int n_slots, rows, kd, vd;    // rows per slot; padded head sizes (blocked)
  bool blocked;
};

template <typename T, int V>
__device__ __forceinline__ void rotate_head(const T* __restrict__ src, const float* __restrict__ c,
                                            const float* __restrict__ s, int half, int d, int pad,
                                            int i, T* __restrict__ o1, T* __restrict__ o2) {
  // unit i of a head: first the rotated pairs, then the rest, then zero padding
  const int nr = half / V, np = (d - 2 * half) / V;
  if (i < nr) {
    const int e = i * V;
    float u[V], v[V], cc[V], ss[V], a[V], b[V];
    load_vec<T, V>(src + e, u);
    load_vec<T, V>(src + half + e, v);
    load_vec<float, V>(c + e, cc);
    load_vec<float, V>(s + e, ss);
#pragma unroll
    for (int j = 0; j < V; ++j) {
      a[j] = u[j] * cc[j] - v[j] * ss[j];
      b[j] = v[j] * cc[j] + u[j] * ss[j];
    }
    if (o1) {
      store_vec<T, V>(o1 + e, a);
      store_vec<T, V>(o1 + half + e, b);
    }
    if (o2) {
      store_vec<T, V>(o2 + e, a);
      store_vec<T, V>(o2 + half + e, b);
    }
  } else if (i < nr + np) {
    const int e = 2 * half + (i - nr) * V;
    float u[V];
    load_vec<T, V>(src + e, u);
    if (o1) store_vec<T, V>(o1 + e, u);
    if (o2) store_vec<T, V>(o2 + e, u);
  } else if (o1) {
    const int e = d + (i - nr - np) * V;
    float z[V];
#pragma unroll
    for (int j = 0; j < V; ++j) z[j] = 0.f;
    if (e < pad) store_vec<T, V>(o1 + e, z);
  }
}

// One token per workgroup; rows [n_tok, gridDim.x) are padding (zeros).
template <typename T, int V>
__global__ __launch_bounds__(256) void gqa_prep_kernel(
    const T* __restrict__ proj, long ld, const float* __restrict__ cosb,
    const float* __restrict__ sinb, int n_pos, const int* __restrict__ pos,
    const int* __restrict__ slot, const int* __restrict__ seq_end, GqaCache cache, int chunk,
    T* __restrict__ q_out, T* __restrict__ k_out, T* __restrict__ v_out, int n_tok, int H, int G,
    int d, int dv, int half, int qd, int vd) {
  const long t = blockIdx.x;
  if (t >= n_tok) {
    for (int i = threadIdx.x; i < H * qd; i += blockDim.x) q_out[t * H * qd + i] = from_f32<T>(0.f);
    if (k_out)
      for (int i = threadIdx.x; i < G * qd; i += blockDim.x)
        k_out[t * G * qd + i] = from_f32<T>(0.f);
    if (v_out)
      for (int i = threadIdx.x; i < G * vd; i += blockDim.x)
        v_out[t * G * vd + i] = from_f32<T>(0.f);
    return;
  }
  const T* row = proj + t * ld;
  const int p = min(max(pos[t], 0), n_pos - 1);
  const float* c = cosb + (long)p * half;
  const float* s = sinb + (long)p * half;
  const int units = qd / V - half / V;              // rotated pairs count once
  for (int i = threadIdx.x; i < H * units; i += blockDim.x) {
    const int h = i / units;
    rotate_head<T, V>(row + h * d, c, s, half, d, qd, i % units, q_out + (t * H + h) * qd,
                      (T*)nullptr);
  }
  // the cache keeps the tokens of a sequence's last chunk
  int at = -1;
  if (cache.k) {
    const int sl = slot[t], last = seq_end ? pos[t] + seq_end[t] - 1 - (int)t : pos[t];
    const int r = pos[t] % chunk;
    if (sl >= 0 && sl < cache.n_slots && pos[t] >= 0 && r < cache.rows &&
        last / chunk == pos[t] / chunk)
      at = r;
  }
  const long sl = at >= 0 ? slot[t] : 0;
  T* kc = reinterpret_cast<T*>(cache.k);
  T* vc = reinterpret_cast<T*>(cache.v);
  for (int i = threadIdx.x; i < G * units; i += blockDim.x) {
    const int g = i / units;
    T* to = nullptr;
    if (at >= 0)
      to = cache.blocked ? kc + ((sl * G + g) * cache.rows + at) * cache.kd
                         : kc + ((sl * cache.rows + at) * G + g) * d;
    rotate_head<T, V>(row + (H + g) * d, c, s, half, d, qd, i % units,
                      k_out ? k_out + (t * G + g) * qd : nullptr, to);
  }
  const T* vrow = row + (long)(H + G) * d;
  const int vu = vd / V;
  for (int i = threadIdx.x; i < G * vu; i += blockDim.x) {
    const int g = i / vu, e = (i % vu) * V;
    float x[V];
    if (e < dv) {
      load_vec<T, V>(vrow + g * dv + e, x);
    } else {
#pragma unroll
      for (int j = 0; j < V; ++j) x[j] = 0.f;
    }
    if (v_out) store_vec<T, V>(v_out + (t * G + g) * vd + e, x);
    if (at >= 0 && e < dv) {
      if (!cache.blocked) {
        store_vec<T, V>(vc + ((sl * cache.rows + at) * G + g) * dv + e, x);
      } else if (!seq_end) {                         // prompts: gqa_store_v
        T* to = vc + ((sl * G + g) * (cache.rows / 32) + at / 32) * (long)cache.vd * 32 +
                v_place(at & 31);
#pragma unroll
        for (int j = 0; j < V; ++j) to[(e + j) * 32] = from_f32<T>(x[j]);
      }
    }
  }
}

// Blocks of 32 keys of every sequence's last chunk, from v [rows, G, vs].
__global__ __launch_bounds__(256) void gqa_store_v_kernel(
    const bf16* __restrict__ v, int vs, const int* __restrict__ cu, const int* __restrict__ slot,
    GqaCache cache, int chunk, int G, int dv) {
  const int t0 = cu[blockIdx.z], len = cu[blockIdx.z + 1] - t0, g = blockIdx.y, b = blockIdx.x;
  const int c0 = (len - 1) / chunk * chunk;          // the last chunk's first position
  const int p0 = c0 + 32 * b, n = min(len - p0, 32);
  if (n <= 0 || 32 * b >= cache.rows) return;
  const int sl = slot[t0];
  if (sl < 0 || sl >= cache.n_slots) return;
  bf16* to = reinterpret_cast<bf16*>(cache.v) +
             (((long)sl * G + g) * (cache.rows / 32) + b) * (long)cache.vd * 32;
  for (int i = threadIdx.x; i < 4 * dv; i += blockDim.x) {
    const int c = i % dv, lg = i / dv;
    gqa_bf16x8 o;
#pragma unroll
    for (int j = 0; j < 8; ++j) {
      const int key = 16 * (j >> 2) + 4 * lg + (j & 3);
      const bf16 x = key < n ? v[((long)(t0 + p0 + key) * G + g) * vs + c] : f2bf(0.f);
      o[j] = __builtin_bit_cast(__bf16, x);
    }
    *reinterpret_cast<gqa_bf16x8*>(to + c * 32 + lg * 8) = o;
  }
}

// grid (splits / 4, G * head blocks, rows); a wave is a split.
template <int D>
__global__ __launch_bounds__(256) void gqa_decode_attn_kernel(
    const bf16* __restrict__ q, GqaCache cache, const int* __restrict__ slot,
    const int* __restrict__ pos, int chunk, int H, int G, float scale, int splits,
    float* __restrict__ part_o, float* __restrict__ part_ml) {
  constexpr int KT = D / 32, VT = D / 16;
  const int lane = threadIdx.x & 63, lo = lane & 15, lg = lane >> 4;
  const int split = blockIdx.x * 4 + (threadIdx.x >> 6);
  if (split >= splits) return;
  const int per = H / G, hbs = (per + 15) / 16;
  const int g = blockIdx.y / hbs, hb = blockIdx.y % hbs;
  const int r = blockIdx.z;
  const int kd = cache.kd, vd = cache.vd, kt = kd / 32, vt = vd / 16;
  const int sl = slot[r];
  const bool ok = sl >= 0 && sl < cache.n_slots && pos[r] >= 0;
  const int n = ok ? min(pos[r] % chunk + 1, cache.rows) : 0;
  const int nb = (n + 31) / 32, each = (nb + splits - 1) / splits;
  const int b0 = split * each, b1 = min(b0 + each, nb);
  const bool own = hb * 16 + lo < per;
  const int h = g * per + min(hb * 16 + lo, per - 1);

  gqa_bf16x8 qf[KT];
#pragma unroll
  for (int c = 0; c < KT; ++c) {
    qf[c] = gqa_bf16x8{};
    if (c < kt && own)
      qf[c] = *reinterpret_cast<const gqa_bf16x8*>(q + ((long)r * H + h) * kd + c * 32 + lg * 8);
  }
  gqa_f32x4 o[VT];
#pragma unroll
  for (int c = 0; c < VT; ++c) o[c] = gqa_f32x4{0.f, 0.f, 0.f, 0.f};
  float m = -INFINITY, l = 0.f;
  const bf16* kb = reinterpret_cast<const bf16*>(cache.k) +
                   (((long)max(sl, 0) * G + g) * cache.rows + lo) * kd + lg * 8;
  const bf16* vb = reinterpret_cast<const bf16*>(cache.v) + lo * 32 + lg * 8 +
                   ((long)max(sl, 0) * G + g) * (cache.rows / 32) * (long)vd * 32;
  for (int b = b0; b < b1; ++b) {
    gqa_bf16x8 kf[2][KT], vf[VT];
#pragma unroll
    for (int i = 0; i < 2; ++i)
#pragma unroll
      for (int c = 0; c < KT; ++c)
        if (c < kt)
          kf[i][c] =
              *reinterpret_cast<const gqa_bf16x8*>(kb + (long)(b * 32 + i * 16) * kd + c * 32);
#pragma unroll
    for (int c = 0; c < VT; ++c)
      if (c < vt)
        vf[c] = *reinterpret_cast<const gqa_bf16x8*>(vb + (long)b * vd * 32 + c * 16 * 32);
    float s[8];
    float top = -INFINITY;
#pragma unroll
    for (int i = 0; i < 2; ++i) {
      gqa_f32x4 a = gqa_f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int c = 0; c < KT; ++c)
        if (c < kt) a = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf[i][c], qf[c], a, 0, 0, 0);
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        const int key = b * 32 + i * 16 + lg * 4 + j;
        s[i * 4 + j] = key < n ? a[j] * scale : -INFINITY;
        top = fmaxf(top, s[i * 4 + j]);
      }
    }
    top = fmaxf(top, __shfl_xor(top, 16));
    top = fmaxf(top, __shfl_xor(top, 32));
    const float mn = fmaxf(m, top);                 // a block has a key: finite
    const float alpha = __expf(m - mn);
    float sum = 0.f;
    gqa_bf16x8 pf;
#pragma unroll
    for (int j = 0; j < 8; ++j) {
      const float e = __expf(s[j] - mn);
      sum += e;
      pf[j] = (__bf16)e;
    }
    l = l * alpha + sum;
    m = mn;
#pragma unroll
    for (int c = 0; c < VT; ++c) {
      if (c >= vt) break;
#pragma unroll
      for (int j = 0; j < 4; ++j) o[c][j] *= alpha;
      o[c] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf[c], pf, o[c], 0, 0, 0);
    }
  }
  l += __shfl_xor(l, 16);
  l += __shfl_xor(l, 32);
  if (!own) return;
  const long at = ((long)r * H + h) * splits + split;
#pragma unroll
  for (int c = 0; c < VT; ++c)
    if (c < vt) *reinterpret_cast<gqa_f32x4*>(part_o + at * vd + c * 16 + lg * 4) = o[c];
  if (lg == 0) {
    part_ml[at * 2] = m;
    part_ml[at * 2 + 1] = l;
  }
}

// One (row, head) per workgroup: the splits' weights once, then their sum with
// every group of vd / 4 threads taking some of the splits.
constexpr int MAX_SPLITS = 256;
__global__ __launch_bounds__(256) void gqa_decode_merge_kernel(
    const float* __restrict__ part_o, const float* __restrict__ part_ml,
    const bf16* __restrict__ sink, bf16* __restrict__ out, int H, int splits, int vd, int dv) {
  __shared__ float w[MAX_SPLITS], red[8];
  __shared__ __attribute__((aligned(16))) float sum[1024];
  const int h = blockIdx.x, tid = threadIdx.x;
  const long rh = (long)blockIdx.y * H + h;
  const float* ml = part_ml + rh * splits * 2;
  const float sk = sink ? bf2f(sink[h]) : -INFINITY;
  const float ms = tid < splits ? ml[2 * tid] : -INFINITY;
  const float ls = tid < splits ? ml[2 * tid + 1] : 0.f;
  const float wm = wave_reduce_max(ms);
  if ((tid & 63) == 0) red[tid >> 6] = wm;
  __syncthreads();
  float m = fmaxf(fmaxf(fmaxf(red[0], red[1]), fmaxf(red[2], red[3])), sk);
  m = m > -INFINITY ? m : 0.f;
  const float e = __expf(ms - m);
  w[tid] = e;
  const float l = block_reduce_sum(ls * e, red + 4) + __expf(sk - m);   // w is written
  const float inv = l > 0.f ? 1.f / l : 0.f;
  const int units = vd / 4, ng = 256 / units, u = tid % units, g = tid / units;
  if (g < ng) {
    float4 a{0.f, 0.f, 0.f, 0.f};
#pragma unroll 4
    for (int s = g; s < splits; s += ng) {
      const float4 o = *reinterpret_cast<const float4*>(part_o + (rh * splits + s) * vd + u * 4);
      a.x = fmaf(o.x, w[s], a.x);
      a.y = fmaf(o.y, w[s], a.y);
      a.z = fmaf(o.z, w[s], a.z);
      a.w = fmaf(o.w, w[s], a.w);
    }
    *reinterpret_cast<float4*>(sum + (g * units + u) * 4) = a;
  }
  __syncthreads();
  for (int c = tid; c < dv; c += 256) {
    float a = 0.f;
    for (int i = 0; i < ng; ++i) a += sum[i * vd + c];
    out[rh * dv + c] = f2bf(a * inv);
  }
}

void check_i32(const at::Tensor& x, int64_t n, const char* what) {
  TORCH_CHECK(x.is_cuda() && x.is_contiguous() && x.scalar_type() == at::kInt && x.numel() == n,
              what, ": contiguous int32 GPU tensor of ", n, " expected");
}

// Checks a cache pair against the head sizes and says how it is laid out.
GqaCache cache_of(const at::Tensor& k, const at::Tensor& v, at::ScalarType dt, int64_t G,
                  int64_t d, int64_t dv) {
  TORCH_CHECK(k.is_cuda() && v.is_cuda() && k.is_contiguous() && v.is_contiguous() &&
                  k.scalar_type() == dt && v.scalar_type() == dt && k.dim() == 4,
              "gqa cache: contiguous GPU tensors of the activation dtype");
  GqaCache c{k.data_ptr(), v.data_ptr(), (int)k.size(0), 0, 0, 0, v.dim() == 5};
  if (c.blocked) {
    c.rows = (int)k.size(2);
    c.kd = (int)k.size(3);
    c.vd = (int)v.size(3);
    TORCH_CHECK(dt == at::kBFloat16 && k.size(1) == G && c.rows % 32 == 0 && c.kd % 32 == 0 &&
                    c.kd >= d && c.vd % 16 == 0 && c.vd >= dv && v.size(0) == k.size(0) &&
                    v.size(1) == G && v.size(2) == c.rows / 32 && v.size(4) == 32,
                "gqa cache: blocked shapes");
  } else {
    c.rows = (int)k.size(1);
    c.kd = (int)d;
    c.vd = (int)dv;
    TORCH_CHECK(k.size(2) == G && k.size(3) == d && v.dim() == 4 && v.size(0) == k.size(0) &&
                    v.size(1) == c.rows && v.size(2) == G && v.size(3) == dv,
                "gqa cache: plain shapes");
  }
  return c;
}

}  // namespace

#define PTR(t) reinterpret_cast<scalar*>((t).data_ptr())

// proj [T, >= H*d + G*(d+dv)] begins with q, k and v. Prompt steps give
// seq_end and get q, k, v padded to (head_pad, v_pad) and rows_pad rows; decode
// steps get q only.
std::tuple<at::Tensor, at::Tensor, at::Tensor> gqa_prep(
    const at::Tensor& proj, const at::Tensor& cos, const at::Tensor& sin, const at::Tensor& pos,
    const std::optional<at::Tensor>& slot, const std::optional<at::Tensor>& seq_end,
    const std::optional<at::Tensor>& cu_seqlens, const std::optional<at::Tensor>& k_cache,
    const std::optional<at::Tensor>& v_cache, int64_t chunk, int64_t heads, int64_t kv_heads,
    int64_t d, int64_t dv, int64_t head_pad, int64_t v_pad, int64_t rows_pad, bool decode) {
  const int64_t T = proj.size(0), ld = proj.size(1);
  const auto dt = proj.scalar_type();
  TORCH_CHECK(proj.is_cuda() && proj.dim() == 2 && proj.is_contiguous() &&
                  (dt == at::kBFloat16 || dt == at::kFloat),
              "gqa_prep: proj must be a contiguous [T, n] bf16/f32 GPU tensor");
  TORCH_CHECK(heads >= 1 && kv_heads >= 1 && heads % kv_heads == 0 && d >= 1 && dv >= 1 &&
                  ld >= heads * d + kv_heads * (d + dv) && head_pad >= d && v_pad >= dv &&
                  rows_pad >= T && chunk >= 1 && chunk <= INT_MAX,
              "gqa_prep: sizes");
  TORCH_CHECK(cos.is_cuda() && sin.is_cuda() && cos.dim() == 2 && cos.is_contiguous() &&
                  sin.is_contiguous() && cos.sizes() == sin.sizes() &&
                  cos.scalar_type() == at::kFloat && sin.scalar_type() == at::kFloat &&
                  2 * cos.size(1) <= d && cos.size(0) >= 1,
              "gqa_prep: cos/sin [positions, rotated / 2] f32");
  check_i32(pos, T, "gqa_prep pos");
  GqaCache cache{nullptr, nullptr, 0, 0, 0, 0, false};
  if (k_cache) {
    TORCH_CHECK(v_cache && slot && (decode || (seq_end && cu_seqlens)),
                "gqa_prep: a cache needs slots, a prompt also its bounds");
    check_i32(*slot, T, "gqa_prep slot");
    cache = cache_of(*k_cache, *v_cache, dt, kv_heads, d, dv);
  }
  if (seq_end) check_i32(*seq_end, T, "gqa_prep seq_end");
  if (cu_seqlens) {
    TORCH_CHECK(cu_seqlens->numel() >= 2, "gqa_prep: cu_seqlens [n + 1]");
    check_i32(*cu_seqlens, cu_seqlens->numel(), "gqa_prep cu_seqlens");
  }
  TORCH_CHECK(!decode || k_cache, "gqa_prep: decoding needs a cache");
  const int half = (int)cos.size(1);
  auto q = at::empty({rows_pad, heads, head_pad}, proj.options());
  auto k = at::empty({decode ? 0 : rows_pad, kv_heads, head_pad}, proj.options());
  auto v = at::empty({decode ? 0 : rows_pad, kv_heads, v_pad}, proj.options());
  if (T == 0) return {q, k, v};
  auto stream = c10::hip::getCurrentHIPStream();
  bool vec = true;
  for (int64_t n : {(int64_t)half, d, dv, head_pad, v_pad, ld}) vec = vec && n % 8 == 0;
  AMD_DISPATCH_T_V(dt, vec, {
    gqa_prep_kernel<scalar, V><<<dim3(rows_pad), dim3(256), 0, stream>>>(
        PTR(proj), ld, cos.data_ptr<float>(), sin.data_ptr<float>(), (int)cos.size(0),
        pos.data_ptr<int>(), slot ? slot->data_ptr<int>() : nullptr,
        decode || !seq_end ? nullptr : seq_end->data_ptr<int>(), cache, (int)chunk, PTR(q),
        decode ? nullptr : PTR(k), decode ? nullptr : PTR(v), (int)T, (int)heads, (int)kv_heads,
        (int)d, (int)dv, half, (int)head_pad, (int)v_pad);
  });
  HIP_CHECK_KERNEL();
  if (!decode && cache.k && cache.blocked) {
    const int64_t n = cu_seqlens->numel() - 1;
    TORCH_CHECK(n <= 65535 && kv_heads <= 65535, "gqa_prep: too many sequences");
    const int blocks = (int)std::min<int64_t>(cache.rows / 32, (T + 31) / 32);
    gqa_store_v_kernel<<<dim3(blocks, kv_heads, n), dim3(256), 0, stream>>>(
        reinterpret_cast<const bf16*>(v.data_ptr()), (int)v_pad, cu_seqlens->data_ptr<int>(),
        slot->data_ptr<int>(), cache, (int)chunk, (int)kv_heads, (int)dv);
    HIP_CHECK_KERNEL();
  }
  return {q, k, v};
}

// q [R, H, kd] against a blocked cache -> [R, H * dv] bf16
at::Tensor gqa_decode_attn(const at::Tensor& q, const at::Tensor& k_cache,
                           const at::Tensor& v_cache, const at::Tensor& slot,
                           const at::Tensor& pos, const std::optional<at::Tensor>& sink,
                           int64_t chunk, int64_t dv, double scale, int64_t splits) {
  TORCH_CHECK(q.is_cuda() && q.dim() == 3 && q.is_contiguous() && q.scalar_type() == at::kBFloat16,
              "gqa_decode_attn: q [R, H, kd] bf16");
  const int64_t R = q.size(0), H = q.size(1), kd = q.size(2), G = k_cache.size(1);
  GqaCache cache = cache_of(k_cache, v_cache, at::kBFloat16, G, kd, dv);
  TORCH_CHECK(cache.blocked && cache.kd == kd && H % G == 0, "gqa_decode_attn: cache shapes");
  TORCH_CHECK(splits >= 1 && splits <= MAX_SPLITS && chunk >= 1 && chunk <= INT_MAX && R <= 65535,
              "gqa_decode_attn: sizes");
  check_i32(slot, R, "gqa_decode_attn slot");
  check_i32(pos, R, "gqa_decode_attn pos");
  if (sink)
    TORCH_CHECK(sink->is_cuda() && sink->is_contiguous() && sink->numel() == H &&
                    sink->scalar_type() == at::kBFloat16, "gqa_decode_attn: sink [H] bf16");
  const int D = std::max(cache.kd, cache.vd);
  TORCH_CHECK(D <= 256, "gqa_decode_attn: head sizes up to 256");
  auto out = at::empty({R, H * dv}, q.options());
  if (R == 0) return out;
  auto part = at::empty({R, H, splits, cache.vd}, q.options().dtype(at::kFloat));
  auto ml = at::empty({R, H, splits, 2}, q.options().dtype(at::kFloat));
  auto stream = c10::hip::getCurrentHIPStream();
  const int hbs = (int)((H / G + 15) / 16);
  const dim3 grid((splits + 3) / 4, G * hbs, R);
#define LAUNCH(DD)                                                                            \
  gqa_decode_attn_kernel<DD><<<grid, dim3(splits < 4 ? 64 * splits : 256), 0, stream>>>(      \
      reinterpret_cast<const bf16*>(q.data_ptr()), cache, slot.data_ptr<int>(),               \
      pos.data_ptr<int>(), (int)chunk, (int)H, (int)G, (float)scale, (int)splits,             \
      part.data_ptr<float>(), ml.data_ptr<float>())
  if (D <= 32) LAUNCH(32);
  else if (D <= 64) LAUNCH(64);
  else if (D <= 96) LAUNCH(96);
  else if (D <= 128) LAUNCH(128);
  else if (D <= 192) LAUNCH(192);
  else LAUNCH(256);
#undef LAUNCH
  HIP_CHECK_KERNEL();
  gqa_decode_merge_kernel<<<dim3(H, R), dim3(256), 0, stream>>>(
      part.data_ptr<float>(), ml.data_ptr<float>(),
      sink ? reinterpret_cast<const bf16*>(sink->data_ptr()) : nullptr,
      reinterpret_cast<bf16*>(out.data_ptr()), (int)H, (int)splits, cache.vd, (int)dv);
  HIP_CHECK_KERNEL();
  return out;
}

#undef PTR

}  // namespace amd_ops
