// Latent attention, decode side: a few query rows against the latent cache,
// with the key and value up-projections absorbed into query and output so that
// only the cache row (latent + shared rotated key) is ever read per key.
//
//   latent_decode_prep     q'[r,h] = [ W_uk[h]^T q_unrot | rotated q ], and the
//                          new token's cache row, in one launch
//   latent_decode_attn     split-KV attention of all heads over the cache:
//                          the heads are the M dimension of 16x16x32 MFMAs, so
//                          one staged key tile serves them all
//   latent_decode_combine  merges the splits, then applies W_uv per head
//
// Lengths and slots are device tensors: a captured step replays for every
// position. Keys are split evenly over the row's own length.

#include <torch/library.h>
#include <ATen/ATen.h>
#include <c10/hip/HIPStream.h>

#include "common.h"
#include "latent_attn.h"
#include "ops_api.h"

namespace amd_ops {

void latent_check_rope(const at::Tensor& cos, const at::Tensor& sin, int64_t rot);
void latent_check_cache(const at::Tensor& cache, at::ScalarType dt, int64_t rank, int64_t rot);

// ---------------------------------------------------------------------------
// prep: blockIdx.x < H * NC absorbs 16*V latent columns of one head for RT
// rows (16 column groups x 16 slices of the head dim, then a reduction);
// the last blockIdx.x writes the rows' latents into the cache.
// ---------------------------------------------------------------------------
template <typename T, int V, int RT>
__global__ __launch_bounds__(256) void latent_decode_prep_kernel(
    const T* __restrict__ qkv, const T* __restrict__ w_uk, const T* __restrict__ w_norm, float eps,
    const float* __restrict__ cosb, const float* __restrict__ sinb, int n_pos, int cs_stride,
    const int* __restrict__ pos, const int* __restrict__ slot, T* __restrict__ cache, int n_slots,
    int max_len, T* __restrict__ q_out, int R, int H, int dn, int dr, int rank, int NC) {
  extern __shared__ float sm[];
  const int tid = threadIdx.x;
  const int r0 = blockIdx.y * RT;
  const int hd = dn + dr, RP = pad32(rank), C = RP + pad32(dr);
  const long N = (long)H * hd + rank + dr;
  if ((int)blockIdx.x == H * NC) {
    for (int r = r0; r < min(r0 + RT, R); ++r) {
      const int p = min(max(pos[r], 0), n_pos - 1);
      const long cr = cache_row(slot[r], pos[r], n_slots, max_len);
      latent_token<T>(qkv + r * N + (long)H * hd, w_norm, eps, cosb + (long)p * cs_stride,
                      sinb + (long)p * cs_stride, rank, dr, cr >= 0 ? cache + cr * C : nullptr,
                      (T*)nullptr, (T*)nullptr, sm);
    }
    return;
  }
  const int h = blockIdx.x / NC, nc = blockIdx.x % NC;
  float* qs = sm;                                 // [RT][dn]
  float* part = sm + RT * dn;                     // [4 waves][RT][16*V]
  for (int i = tid; i < RT * dn; i += 256) {
    const int r = r0 + i / dn;
    qs[i] = r < R ? lat_f(qkv[r * N + h * hd + i % dn]) : 0.f;
  }
  if (nc == 0) {                                  // rotated part and zero padding
    const int half = dr / 2;
    for (int rr = 0; rr < RT; ++rr) {
      const int r = r0 + rr;
      if (r >= R) break;
      T* o = q_out + ((long)r * H + h) * C;
      const T* src = qkv + r * N + h * hd + dn;
      const int p = min(max(pos[r], 0), n_pos - 1);
      for (int i = tid; i < half; i += 256) {
        const float c = cosb[(long)p * cs_stride + i], s = sinb[(long)p * cs_stride + i];
        const float u = lat_f(src[i]), v = lat_f(src[half + i]);
        o[RP + i] = lat_t<T>(u * c - v * s);
        o[RP + half + i] = lat_t<T>(v * c + u * s);
      }
      for (int i = rank + tid; i < RP; i += 256) o[i] = lat_t<T>(0.f);
      for (int i = RP + dr + tid; i < C; i += 256) o[i] = lat_t<T>(0.f);
    }
  }
  __syncthreads();
  const int vec = tid & 15, slice = tid >> 4;     // 16 columns groups x 16 slices
  const int col = (nc * 16 + vec) * V;
  float acc[RT][V];
#pragma unroll
  for (int r = 0; r < RT; ++r)
#pragma unroll
    for (int j = 0; j < V; ++j) acc[r][j] = 0.f;
  if (col < rank) {                               // V divides rank
    const T* wp = w_uk + (long)h * dn * rank + col;
#pragma unroll 4
    for (int d = slice; d < dn; d += 16) {
      const LatPack<T, V> w = *reinterpret_cast<const LatPack<T, V>*>(wp + (long)d * rank);
#pragma unroll
      for (int r = 0; r < RT; ++r) {
        const float qv = qs[r * dn + d];
#pragma unroll
        for (int j = 0; j < V; ++j) acc[r][j] = fmaf(qv, lat_f(w.v[j]), acc[r][j]);
      }
    }
  }
  const int lane = tid & 63, wid = tid >> 6;
#pragma unroll
  for (int r = 0; r < RT; ++r)
#pragma unroll
    for (int j = 0; j < V; ++j) {
      float a = acc[r][j];
      a += __shfl_xor(a, 16);
      a += __shfl_xor(a, 32);
      if (lane < 16) part[(wid * RT + r) * 16 * V + vec * V + j] = a;
    }
  __syncthreads();
  for (int i = tid; i < RT * 16 * V; i += 256) {
    const int r = r0 + i / (16 * V), c = nc * 16 * V + i % (16 * V);
    if (r >= R || c >= rank) continue;
    float a = 0.f;
#pragma unroll
    for (int w = 0; w < 4; ++w) a += part[w * RT * 16 * V + i];
    q_out[((long)r * H + h) * C + c] = lat_t<T>(a);
  }
}

// ---------------------------------------------------------------------------
// attention over the cache. grid (splits, head groups of 16*HT, rows)
// ---------------------------------------------------------------------------
typedef __bf16 lat_bf16x8 __attribute__((ext_vector_type(8)));
typedef __bf16 lat_bf16x4 __attribute__((ext_vector_type(4)));
typedef float lat_f32x4 __attribute__((ext_vector_type(4)));
typedef unsigned lat_u32x4 __attribute__((ext_vector_type(4)));    // 16 bytes in flight

constexpr int LD_KEYS = 64;           // keys per tile: 4 waves x 16
constexpr int LD_PSTRIDE = LD_KEYS * 2 + 16;

// hardware-transposed read: 16 lanes fetch a [4 keys][16 columns] block, lane g
// receives column g (each lane supplies the address of its own 8 bytes)
__device__ __forceinline__ lat_bf16x4 lds_tr16(const char* p) {
  typedef __attribute__((address_space(3))) lat_bf16x4* lds_ptr;
  return __builtin_amdgcn_ds_read_tr16_b64_v4bf16(
      (lds_ptr)(__attribute__((address_space(3))) char*)const_cast<char*>(p));
}

// HT: head tiles (of 16 heads) per workgroup, four waves each; they share the
// staged keys. NCT: 16-column value tiles per wave (4 waves cover RP <= 64 *
// NCT). NPM: bound on the 16-byte pieces of a key tile per thread. The next
// tile travels through registers while the current one is used.
template <int HT, int NCT, int NPM>
__global__ __launch_bounds__(256 * HT) void latent_decode_attn_kernel(
    const bf16* __restrict__ q, const bf16* __restrict__ cache, const int* __restrict__ slot,
    const int* __restrict__ pos, float* __restrict__ part_o, float* __restrict__ part_ml,
    int n_slots, int max_len, int H, int RP, int C, float scale) {
  constexpr int NT = 256 * HT;
  extern __shared__ __attribute__((aligned(16))) char lds[];
  const int KS = C * 2 + 16;                      // LDS row stride: conflict-free b128 reads
  char* kt = lds;                                 // [64][KS]
  char* qt = kt + LD_KEYS * KS;                   // [16 HT][KS]
  char* pt = qt + 16 * HT * KS;                   // [16 HT][LD_PSTRIDE]
  float* red = reinterpret_cast<float*>(pt + 16 * HT * LD_PSTRIDE);   // [HT][4][16]

  const int tid = threadIdx.x, lane = tid & 63, wid = (tid >> 6) & 3, ht = tid >> 8;
  const int lo16 = lane & 15, hi4 = lane >> 4;
  const int split = blockIdx.x, n_split = gridDim.x;
  const int h0 = blockIdx.y * 16 * HT;
  const int r = blockIdx.z;

  const int sl = slot[r];
  const int n = (sl < 0 || sl >= n_slots) ? 0 : min(max(pos[r] + 1, 0), max_len);
  const int tiles = (n + LD_KEYS - 1) / LD_KEYS;
  const int per = (tiles + n_split - 1) / n_split;
  const int t_lo = split * per, t_hi = min(t_lo + per, tiles);
  const bf16* base = cache + (long)(n > 0 ? sl : 0) * max_len * C;

  const int vecs = C / 8;                         // 16-byte pieces per row
  const int pieces = LD_KEYS * vecs, np = (pieces + NT - 1) / NT;
  const unsigned magic = ((1u << 20) + vecs - 1) / vecs;    // i / vecs, exact for i < 128 vecs
  lat_u32x4 pre[NPM];
  auto fetch = [&](int t) {
#pragma unroll
    for (int j = 0; j < NPM; ++j) {
      if (j < np) {                               // uniform
        const unsigned i = tid + j * NT, row = (i * magic) >> 20, c = i - row * vecs;
        const int key = min(t * LD_KEYS + (int)row, n - 1);   // rows past the end: masked below
        pre[j] = *reinterpret_cast<const lat_u32x4*>(base + (long)key * C + c * 8);
      }
    }
  };
  if (t_lo < t_hi) fetch(t_lo);
  for (int i0 = tid; i0 < 16 * HT * vecs; i0 += 4 * NT) {      // this workgroup's queries
    lat_u32x4 x[4];
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      const unsigned i = i0 + j * NT, row = (i * magic) >> 20, c = i - row * vecs;
      x[j] = lat_u32x4{0u, 0u, 0u, 0u};
      if (i < 16u * HT * vecs && h0 + (int)row < H)
        x[j] = *reinterpret_cast<const lat_u32x4*>(q + ((long)r * H + h0 + row) * C + c * 8);
    }
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      const unsigned i = i0 + j * NT, row = (i * magic) >> 20, c = i - row * vecs;
      if (i < 16u * HT * vecs) *reinterpret_cast<lat_u32x4*>(qt + row * KS + c * 16) = x[j];
    }
  }

  lat_f32x4 acc[NCT];
  float m_run[4], l_run[4];
#pragma unroll
  for (int c = 0; c < NCT; ++c) acc[c] = lat_f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
  for (int i = 0; i < 4; ++i) m_run[i] = -1e30f, l_run[i] = 0.f;
  float* my_red = red + ht * 64;
  char* my_pt = pt + ht * 16 * LD_PSTRIDE;

  for (int t = t_lo; t < t_hi; ++t) {
    const int k0 = t * LD_KEYS;
#pragma unroll
    for (int j = 0; j < NPM; ++j) {
      if (j < np) {
        const unsigned i = tid + j * NT, row = (i * magic) >> 20, c = i - row * vecs;
        if ((int)i < pieces) *reinterpret_cast<lat_u32x4*>(kt + row * KS + c * 16) = pre[j];
      }
    }
    __syncthreads();
    if (t + 1 < t_hi) fetch(t + 1);

    // scores: D[head = 4*hi4 + i][key = lo16] of this wave's 16 keys
    lat_f32x4 s = {0.f, 0.f, 0.f, 0.f};
    const char* kp = kt + (wid * 16 + lo16) * KS + hi4 * 16;
    const char* qp = qt + (ht * 16 + lo16) * KS + hi4 * 16;
#pragma unroll 6
    for (int c = 0; c < C * 2; c += 64) {
      const lat_bf16x8 b = *reinterpret_cast<const lat_bf16x8*>(kp + c);
      const lat_bf16x8 x = *reinterpret_cast<const lat_bf16x8*>(qp + c);
      s = __builtin_amdgcn_mfma_f32_16x16x32_bf16(x, b, s, 0, 0, 0);
    }
    const bool live = k0 + wid * 16 + lo16 < n;
    float mx[4];
#pragma unroll
    for (int i = 0; i < 4; ++i) s[i] = mx[i] = live ? s[i] * scale : -1e30f;
#pragma unroll
    for (int d = 1; d < 16; d *= 2)
#pragma unroll
      for (int i = 0; i < 4; ++i) mx[i] = fmaxf(mx[i], __shfl_xor(mx[i], d));
    if (lo16 == 0)
#pragma unroll
      for (int i = 0; i < 4; ++i) my_red[wid * 16 + hi4 * 4 + i] = mx[i];
    __syncthreads();
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int row = hi4 * 4 + i;
      float mn = m_run[i];
#pragma unroll
      for (int w = 0; w < 4; ++w) mn = fmaxf(mn, my_red[w * 16 + row]);
      const float alpha = __expf(m_run[i] - mn);
      const float p = live ? __expf(s[i] - mn) : 0.f;
      l_run[i] = l_run[i] * alpha + p;
      m_run[i] = mn;
      *reinterpret_cast<bf16*>(my_pt + row * LD_PSTRIDE + (wid * 16 + lo16) * 2) = f2bf(p);
#pragma unroll
      for (int c = 0; c < NCT; ++c) acc[c][i] *= alpha;
    }
    __syncthreads();

    // O[head][column] += P[head][key] V[key][column], V = the tile's latents
#pragma unroll
    for (int ks = 0; ks < LD_KEYS / 32; ++ks) {
      const lat_bf16x8 p = *reinterpret_cast<const lat_bf16x8*>(my_pt + lo16 * LD_PSTRIDE +
                                                                (ks * 32 + hi4 * 8) * 2);
#pragma unroll
      for (int c = 0; c < NCT; ++c) {
        const int n0 = (wid * NCT + c) * 16;
        if (n0 < RP) {                            // wave-uniform
          const char* vp = kt + (ks * 32 + hi4 * 8 + (lo16 >> 2)) * KS + (n0 + (lo16 & 3) * 4) * 2;
          const lat_bf16x4 v0 = lds_tr16(vp), v1 = lds_tr16(vp + 4 * KS);
          const lat_bf16x8 v = __builtin_shufflevector(v0, v1, 0, 1, 2, 3, 4, 5, 6, 7);
          acc[c] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(p, v, acc[c], 0, 0, 0);
        }
      }
    }
    __syncthreads();                              // before the tile is overwritten
  }

  // partial results of this split; an empty split stores zeros
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    float l = l_run[i];
#pragma unroll
    for (int d = 1; d < 16; d *= 2) l += __shfl_xor(l, d);
    if (lo16 == 0) my_red[wid * 16 + hi4 * 4 + i] = l;
  }
  __syncthreads();
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const int row = hi4 * 4 + i, h = h0 + ht * 16 + row;
    if (h >= H) continue;
    const long o = ((long)r * H + h) * n_split + split;
    if (wid == 0 && lo16 == 0) {
      float l = 0.f;
#pragma unroll
      for (int w = 0; w < 4; ++w) l += my_red[w * 16 + row];
      part_ml[o * 2] = m_run[i];
      part_ml[o * 2 + 1] = l;
    }
#pragma unroll
    for (int c = 0; c < NCT; ++c) {
      const int n0 = (wid * NCT + c) * 16;
      if (n0 < RP) part_o[o * RP + n0 + lo16] = acc[c][i];
    }
  }
}

// ---------------------------------------------------------------------------
// merge: grid (column chunks of 128, H, R). Splits -> normalised latent output
// in f32; 32 threads cover the columns, 8 groups of them share the splits.
// ---------------------------------------------------------------------------
constexpr int LM_COLS = 128;
__global__ __launch_bounds__(256) void latent_decode_merge_kernel(
    const float* __restrict__ part_o, const float* __restrict__ part_ml, float* __restrict__ o,
    int H, int RP, int S) {
  extern __shared__ float sm[];
  float* wt = sm;                                 // [S]
  lat_f32x4* half = reinterpret_cast<lat_f32x4*>(sm + (S + 3) / 4 * 4);    // [8][32]
  const int tid = threadIdx.x, lane = tid & 63;
  const long rh = (long)blockIdx.z * H + blockIdx.y;
  const float* ml = part_ml + rh * S * 2;
  if (tid < 64) {                                 // one wave weighs the splits
    float m = -1e30f;
    for (int s = lane; s < S; s += 64) m = fmaxf(m, ml[2 * s]);
    m = wave_reduce_max(m);
    float l = 0.f;
    for (int s = lane; s < S; s += 64) l += __expf(ml[2 * s] - m) * ml[2 * s + 1];
    l = wave_reduce_sum(l);
    const float inv = l > 0.f ? 1.f / l : 0.f;
    for (int s = lane; s < S; s += 64) wt[s] = __expf(ml[2 * s] - m) * inv;
  }
  __syncthreads();
  const int col = blockIdx.x * LM_COLS + (tid & 31) * 4, g = tid >> 5;
  lat_f32x4 a = {0.f, 0.f, 0.f, 0.f};
  if (col < RP) {                                 // RP % 32 == 0
    const float* po = part_o + rh * S * RP + col;
#pragma unroll 8
    for (int s = g; s < S; s += 8)
      a += wt[s] * *reinterpret_cast<const lat_f32x4*>(po + (long)s * RP);
  }
  half[g * 32 + (tid & 31)] = a;
  __syncthreads();
  if (g == 0 && col < RP) {
#pragma unroll
    for (int i = 1; i < 8; ++i) a += half[i * 32 + tid];
    *reinterpret_cast<lat_f32x4*>(o + rh * RP + col) = a;
  }
}

// ---------------------------------------------------------------------------
// value up-projection: grid (value chunks of 32, H, row groups of RT). A wave
// takes 8 rows of W_uv[h] at once against the latent outputs in LDS.
// ---------------------------------------------------------------------------
constexpr int LC_ROWS = 32;
template <typename T, int V, int RT>
__global__ __launch_bounds__(256) void latent_decode_value_kernel(
    const float* __restrict__ o_lat, const T* __restrict__ w_uv, T* __restrict__ out, int R, int H,
    int dv, int rank, int stride) {
  extern __shared__ float sm[];                   // [RT][rank]
  constexpr int NV = LC_ROWS / 4;
  const int tid = threadIdx.x, lane = tid & 63, wid = tid >> 6;
  const int h = blockIdx.y, r0 = blockIdx.z * RT;
  const int nc = rank / V;                        // column c = chunk * V + j sits at [j][chunk]
  for (int i = tid; i < RT * rank; i += 256) {
    const int rr = i / rank, c = i % rank, r = min(r0 + rr, R - 1);
    sm[rr * rank + (c % V) * nc + c / V] = o_lat[((long)r * H + h) * stride + c];
  }
  const int v0 = blockIdx.x * LC_ROWS + wid * NV;
  const T* w[NV];
#pragma unroll
  for (int v = 0; v < NV; ++v) w[v] = w_uv + ((long)h * dv + min(v0 + v, dv - 1)) * rank;
  float acc[NV * RT];
#pragma unroll
  for (int i = 0; i < NV * RT; ++i) acc[i] = 0.f;
  __syncthreads();
  for (int c = lane; c < nc; c += 64) {
    LatPack<T, V> x[NV];
#pragma unroll
    for (int v = 0; v < NV; ++v) x[v] = *reinterpret_cast<const LatPack<T, V>*>(w[v] + c * V);
#pragma unroll
    for (int rr = 0; rr < RT; ++rr)
#pragma unroll
      for (int j = 0; j < V; ++j) {
        const float o = sm[rr * rank + j * nc + c];
#pragma unroll
        for (int v = 0; v < NV; ++v) acc[rr * NV + v] = fmaf(lat_f(x[v].v[j]), o, acc[rr * NV + v]);
      }
  }
  // all NV * RT sums over the wave at once: halve the set at every step, so
  // that lane l ends with sum l / (64 / (NV * RT))
  constexpr int NA = NV * RT;
  int mask = 32;
#pragma unroll
  for (int n = NA; n > 1; n /= 2, mask /= 2) {
    const bool up = lane & mask;
#pragma unroll
    for (int i = 0; i < n / 2; ++i) {
      const float keep = up ? acc[i + n / 2] : acc[i], give = up ? acc[i] : acc[i + n / 2];
      acc[i] = keep + __shfl_xor(give, mask);
    }
  }
  for (; mask > 0; mask /= 2) acc[0] += __shfl_xor(acc[0], mask);
  const int idx = lane / (64 / NA), rr = idx / NV, v = idx % NV;
  if (lane % (64 / NA) == 0 && v0 + v < dv && r0 + rr < R)
    out[((long)(r0 + rr) * H + h) * dv + v0 + v] = lat_t<T>(acc[0]);
}

// ---------------------------------------------------------------------------
namespace {
bool dec_t(const at::Tensor& x) {
  return x.is_cuda() && x.is_contiguous() &&
         (x.scalar_type() == at::kBFloat16 || x.scalar_type() == at::kFloat);
}
bool dec_i32(const at::Tensor& x, int64_t n) {
  return x.is_cuda() && x.is_contiguous() && x.scalar_type() == at::kInt && x.numel() == n;
}
constexpr size_t LDS_MAX = 160 * 1024;
}  // namespace

#define ROW_TILE(R, ...)                                   \
  do {                                                     \
    if ((R) <= 1) { constexpr int RT = 1; __VA_ARGS__ }           \
    else if ((R) <= 2) { constexpr int RT = 2; __VA_ARGS__ }      \
    else if ((R) <= 4) { constexpr int RT = 4; __VA_ARGS__ }      \
    else { constexpr int RT = 8; __VA_ARGS__ }                    \
  } while (0)

at::Tensor latent_decode_prep(const at::Tensor& qkv, const at::Tensor& w_uk,
                              const at::Tensor& w_norm, double eps, const at::Tensor& cos,
                              const at::Tensor& sin, const at::Tensor& pos, const at::Tensor& slot,
                              at::Tensor cache, int64_t heads, int64_t dn, int64_t dr) {
  TORCH_CHECK(dec_t(qkv) && qkv.dim() == 2, "latent_decode_prep: qkv [R, N]");
  const auto dt = qkv.scalar_type();
  const int64_t R = qkv.size(0), rank = w_norm.numel();
  TORCH_CHECK(dec_t(w_uk) && w_uk.scalar_type() == dt && w_uk.dim() == 2 &&
                  w_uk.size(0) == heads * dn && w_uk.size(1) == rank,
              "latent_decode_prep: W_uk [heads * dim, rank]");
  TORCH_CHECK(dec_t(w_norm) && w_norm.scalar_type() == dt, "latent_decode_prep: norm weight");
  TORCH_CHECK(qkv.size(1) == heads * (dn + dr) + rank + dr, "latent_decode_prep: qkv width");
  TORCH_CHECK(dec_i32(pos, R) && dec_i32(slot, R), "latent_decode_prep: pos/slot int32 [R]");
  latent_check_rope(cos, sin, dr);
  latent_check_cache(cache, dt, rank, dr);
  auto q = at::empty({R, heads, cache.size(2)}, qkv.options());
  if (R == 0) return q;
  auto stream = c10::hip::getCurrentHIPStream();
  const bool vec = rank % 8 == 0;
  const int cols = vec ? 128 : 16;
  const int NC = (int)((rank + cols - 1) / cols);
#define LAUNCH(TT, VV)                                                                           \
  latent_decode_prep_kernel<TT, VV, RT>                                                          \
      <<<dim3(heads * NC + 1, (R + RT - 1) / RT), dim3(256), smem, stream>>>(                    \
          reinterpret_cast<const TT*>(qkv.data_ptr()),                                           \
          reinterpret_cast<const TT*>(w_uk.data_ptr()),                                          \
          reinterpret_cast<const TT*>(w_norm.data_ptr()), (float)eps, cos.data_ptr<float>(),     \
          sin.data_ptr<float>(), (int)cos.size(0), (int)cos.size(1), pos.data_ptr<int>(),        \
          slot.data_ptr<int>(), reinterpret_cast<TT*>(cache.data_ptr()), (int)cache.size(0),     \
          (int)cache.size(1), reinterpret_cast<TT*>(q.data_ptr()), (int)R, (int)heads, (int)dn,  \
          (int)dr, (int)rank, NC)
  ROW_TILE(R, {
    const size_t smem = (RT * dn + 4 * RT * cols + 16) * sizeof(float);
    TORCH_CHECK(smem <= 64 * 1024, "latent_decode_prep: head dim too large");
    if (dt == at::kBFloat16) {
      if (vec) LAUNCH(bf16, 8); else LAUNCH(bf16, 1);
    } else {
      if (vec) LAUNCH(float, 8); else LAUNCH(float, 1);
    }
  });
#undef LAUNCH
  HIP_CHECK_KERNEL();
  return q;
}

// q [R, H, C] from latent_decode_prep -> (part_o [R, H, S, RP], part_ml [R, H, S, 2])
std::tuple<at::Tensor, at::Tensor> latent_decode_attn(const at::Tensor& q, const at::Tensor& cache,
                                                      const at::Tensor& slot, const at::Tensor& pos,
                                                      int64_t rank, int64_t rot, double scale,
                                                      int64_t splits) {
  TORCH_CHECK(dec_t(q) && q.dim() == 3 && q.scalar_type() == at::kBFloat16,
              "latent_decode_attn: q [R,H,C] bf16");
  latent_check_cache(cache, at::kBFloat16, rank, rot);
  const int64_t R = q.size(0), H = q.size(1), C = q.size(2), RP = pad32(rank);
  TORCH_CHECK(C == cache.size(2) && RP <= 512, "latent_decode_attn: rank <= 512");
  TORCH_CHECK(dec_i32(pos, R) && dec_i32(slot, R), "latent_decode_attn: pos/slot int32 [R]");
  TORCH_CHECK(splits >= 1 && splits <= 1024 && R <= 65535, "latent_decode_attn: splits/rows");
  auto part_o = at::empty({R, H, splits, RP}, q.options().dtype(at::kFloat));
  auto part_ml = at::empty({R, H, splits, 2}, part_o.options());
  if (R == 0) return {part_o, part_ml};
  auto stream = c10::hip::getCurrentHIPStream();
  // head tiles per workgroup: both share the staged keys, but two workgroups
  // are better where the splits alone leave CUs idle
  const bool two = H > 16 && R * splits * ((H + 31) / 32) >= 256;
#define LAUNCH1(HT, NCT, NPM)                                                                    \
  do {                                                                                           \
    const size_t smem = (LD_KEYS + 16 * HT) * (C * 2 + 16) + 16 * HT * (LD_PSTRIDE + 16);        \
    TORCH_CHECK(smem <= LDS_MAX, "latent_decode_attn: tile exceeds LDS");                        \
    static const hipError_t attr_ = hipFuncSetAttribute(                                         \
        reinterpret_cast<const void*>(&latent_decode_attn_kernel<HT, NCT, NPM>),                 \
        hipFuncAttributeMaxDynamicSharedMemorySize, (int)LDS_MAX);                               \
    TORCH_CHECK(attr_ == hipSuccess, "latent_decode_attn: LDS attribute");                       \
    latent_decode_attn_kernel<HT, NCT, NPM>                                                      \
        <<<dim3(splits, (H + 16 * HT - 1) / (16 * HT), R), dim3(256 * HT), smem, stream>>>(      \
            reinterpret_cast<const bf16*>(q.data_ptr()),                                         \
            reinterpret_cast<const bf16*>(cache.data_ptr()), slot.data_ptr<int>(),               \
            pos.data_ptr<int>(), part_o.data_ptr<float>(), part_ml.data_ptr<float>(),            \
            (int)cache.size(0), (int)cache.size(1), (int)H, (int)RP, (int)C, (float)scale);      \
  } while (0)
#define LAUNCH(NCT, NPM)                                                                         \
  do {                                                                                           \
    if (two) LAUNCH1(2, NCT, (NPM + 1) / 2); else LAUNCH1(1, NCT, NPM);                          \
  } while (0)
  TORCH_CHECK(C / 32 <= 26, "latent_decode_attn: latent and rotated key too wide");
  if (RP <= 128 && C <= 256) LAUNCH(2, 8);
  else if (RP <= 256 && C <= 384) LAUNCH(4, 12);
  else if (C <= 640) LAUNCH(8, 20);
  else LAUNCH(8, 26);
#undef LAUNCH1
#undef LAUNCH
  HIP_CHECK_KERNEL();
  return {part_o, part_ml};
}

// part_o [R, H, S, stride >= rank] f32 (+ part_ml) and W_uv [H * dv, rank] -> [R, H * dv]
at::Tensor latent_decode_combine(const at::Tensor& part_o,
                                 const std::optional<at::Tensor>& part_ml, const at::Tensor& w_uv,
                                 int64_t dv) {
  TORCH_CHECK(part_o.is_cuda() && part_o.is_contiguous() && part_o.dim() == 4 &&
                  part_o.scalar_type() == at::kFloat,
              "latent_decode_combine: part_o [R,H,S,n] f32");
  const int64_t R = part_o.size(0), H = part_o.size(1), S = part_o.size(2), n = part_o.size(3);
  TORCH_CHECK(dec_t(w_uv) && w_uv.dim() == 2 && w_uv.size(0) == H * dv && w_uv.size(1) <= n,
              "latent_decode_combine: W_uv [H * dv, rank]");
  const int64_t rank = w_uv.size(1);
  if (part_ml) {
    TORCH_CHECK(part_ml->is_cuda() && part_ml->is_contiguous() &&
                    part_ml->scalar_type() == at::kFloat && part_ml->numel() == R * H * S * 2,
                "latent_decode_combine: part_ml [R,H,S,2] f32");
  } else {
    TORCH_CHECK(S == 1, "latent_decode_combine: splits need part_ml");
  }
  auto out = at::empty({R, H * dv}, w_uv.options());
  if (R == 0) return out;
  auto stream = c10::hip::getCurrentHIPStream();
  const bool vec = rank % 8 == 0;
  at::Tensor o_lat = part_o;
  if (part_ml) {
    TORCH_CHECK(n % 32 == 0 && S <= 1024, "latent_decode_combine: padded rank, splits <= 1024");
    o_lat = at::empty({R, H, n}, part_o.options());
    latent_decode_merge_kernel<<<dim3((n + LM_COLS - 1) / LM_COLS, H, R), dim3(256),
                                 ((S + 3) / 4 * 4 + 1024) * sizeof(float), stream>>>(
        part_o.data_ptr<float>(), part_ml->data_ptr<float>(), o_lat.data_ptr<float>(), (int)H,
        (int)n, (int)S);
    HIP_CHECK_KERNEL();
  }
#define LAUNCH(TT, VV)                                                                          \
  latent_decode_value_kernel<TT, VV, RT>                                                        \
      <<<dim3((dv + LC_ROWS - 1) / LC_ROWS, H, (R + RT - 1) / RT), dim3(256), smem, stream>>>(  \
          o_lat.data_ptr<float>(), reinterpret_cast<const TT*>(w_uv.data_ptr()),                \
          reinterpret_cast<TT*>(out.data_ptr()), (int)R, (int)H, (int)dv, (int)rank, (int)n)
  ROW_TILE(R, {
    const size_t smem = RT * rank * sizeof(float);
    TORCH_CHECK(smem <= 64 * 1024, "latent_decode_combine: rank too large");
    if (w_uv.scalar_type() == at::kBFloat16) {
      if (vec) LAUNCH(bf16, 8); else LAUNCH(bf16, 1);
    } else {
      if (vec) LAUNCH(float, 8); else LAUNCH(float, 1);
    }
  });
#undef LAUNCH
  HIP_CHECK_KERNEL();
  return out;
}
#undef ROW_TILE

}  // namespace amd_ops
