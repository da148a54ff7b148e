// Skinny-batch bf16 GEMV for KV-cached decode: y[B,N] = x[B,K] @ W[N,K]^T.
//
// Decode-step linears are m<=16 GEMMs — pure weight-streaming. hipBLASLt's
// GEMV path measures ~23% of HBM bandwidth on these shapes (profiled in
// profiles/decode_*.json); this kernel streams each W row once with b128
// loads (guide Guideline 13) and broadcasts the tiny x through L2:
//   * one wave per output row, lanes cover K in 16-byte chunks
//     (lane l reads W[row, l*8 + i*512 .. +8) — 1 KB/instruction/wave,
//     fully coalesced);
//   * batch columns (B) accumulate in registers in the same pass, so W
//     traffic is independent of B;
//   * fp32 dot accumulation + wave reduce, lane 0 stores;
//   * the epilogue can apply max(y, 0)^2 and can store f32 (residual inputs,
//     logits) instead of bf16.
// Grid = N/4 workgroups of 4 waves: N=4096 -> 1024 blocks >> 256 CUs.

#include <torch/library.h>
#include <ATen/ATen.h>
#include <c10/hip/HIPStream.h>

#include "common.h"
#include "ops_api.h"

namespace amd_ops {

typedef __bf16 gemv_bf16x2 __attribute__((ext_vector_type(2)));
typedef __bf16 gemv_bf16x8 __attribute__((ext_vector_type(8)));
typedef float gemv_f32x4 __attribute__((ext_vector_type(4)));

__device__ __forceinline__ float dot2(const bf16x8& a, const bf16x8& b, int j, float c) {
  const gemv_bf16x8 av = __builtin_bit_cast(gemv_bf16x8, a), bv = __builtin_bit_cast(gemv_bf16x8, b);
  return __builtin_amdgcn_fdot2_f32_bf16(gemv_bf16x2{av[2 * j], av[2 * j + 1]},
                                         gemv_bf16x2{bv[2 * j], bv[2 * j + 1]}, c, false);
}

// Two rows per wave: doubles outstanding b128 loads per wave (latency
// hiding for the short 8-iteration K sweep at K=4096).
template <int B>
__global__ __launch_bounds__(256, 4) void gemv_bf16_kernel(
    const bf16* __restrict__ W, const bf16* __restrict__ x,
    const bf16* __restrict__ bias, bf16* __restrict__ y, float* __restrict__ yf, bool relu2,
    int N, int K, int group_n) {
  const int lane = threadIdx.x & (WAVE_SIZE - 1);
  const int wid = blockIdx.x * (blockDim.x / WAVE_SIZE) + (threadIdx.x / WAVE_SIZE);
  const int row0 = 2 * wid;
  if (row0 >= N) return;
  const bool two = row0 + 1 < N;
  float acc0[B], acc1[B];
#pragma unroll
  for (int b = 0; b < B; ++b) acc0[b] = acc1[b] = 0.f;
  const bf16* wrow0 = W + (long)row0 * K;
  const bf16* wrow1 = wrow0 + (two ? K : 0);
  if (group_n) x += (long)(row0 / group_n) * B * K;   // group_n is even
  for (int k = lane * 8; k < K; k += WAVE_SIZE * 8) {
    const bf16x8 w0 = *reinterpret_cast<const bf16x8*>(wrow0 + k);
    const bf16x8 w1 = *reinterpret_cast<const bf16x8*>(wrow1 + k);
#pragma unroll
    for (int b = 0; b < B; ++b) {
      const bf16x8 xv = *reinterpret_cast<const bf16x8*>(x + (long)b * K + k);
      float d0 = 0.f, d1 = 0.f;
#pragma unroll
      for (int j = 0; j < 4; ++j) {               // v_dot2_f32_bf16: f32 accumulation
        d0 = dot2(w0, xv, j, d0);
        d1 = dot2(w1, xv, j, d1);
      }
      acc0[b] += d0;
      acc1[b] += d1;
    }
  }
#pragma unroll
  for (int b = 0; b < B; ++b) {
    const float t0 = wave_reduce_sum(acc0[b]);
    const float t1 = wave_reduce_sum(acc1[b]);
    if (lane == 0) {
#pragma unroll
      for (int i = 0; i < 2; ++i) {
        if (i && !two) break;
        float t = (i ? t1 : t0) + (bias ? bf2f(bias[row0 + i]) : 0.f);
        if (relu2) {
          t = fmaxf(t, 0.f);
          t *= t;
        }
        if (yf) yf[(long)b * N + row0 + i] = t;
        else y[(long)b * N + row0 + i] = f2bf(t);
      }
    }
  }
}

// group_n > 0: x holds several [B, K] inputs one after another, and every
// group_n rows of w take the next one.
at::Tensor gemv_bf16(const at::Tensor& x, const at::Tensor& w,
                     const c10::optional<at::Tensor>& bias, bool relu2, bool out_f32,
                     int64_t group_n) {
  TORCH_CHECK(x.is_cuda() && w.is_cuda(), "gemv_bf16: GPU tensors required");
  TORCH_CHECK(x.dtype() == at::kBFloat16 && w.dtype() == at::kBFloat16,
              "gemv_bf16: bf16 only");
  TORCH_CHECK(x.dim() == 2 && w.dim() == 2, "gemv_bf16: x [B,K], w [N,K]");
  const int K = (int)x.size(1), N = (int)w.size(0);
  const int groups = group_n > 0 ? (int)((N + group_n - 1) / group_n) : 1;
  TORCH_CHECK(group_n >= 0 && group_n % 2 == 0 && x.size(0) % groups == 0,
              "gemv_bf16: an even group_n, and one [B,K] input per group");
  const int B = (int)x.size(0) / groups;
  TORCH_CHECK(w.size(1) == K, "K mismatch");
  TORCH_CHECK(B >= 1 && B <= 16, "gemv_bf16: B in [1,16], got ", B,
              " (larger batches belong on hipBLASLt)");
  TORCH_CHECK(K % 8 == 0, "gemv_bf16: K % 8 == 0, got ", K);
  auto xc = x.contiguous(), wc = w.contiguous();
  auto y = at::empty({B, N}, x.options().dtype(out_f32 ? at::kFloat : at::kBFloat16));
  const bf16* bptr = nullptr;
  if (bias.has_value()) {
    TORCH_CHECK(bias->numel() == N && bias->dtype() == at::kBFloat16, "bias [N] bf16");
    bptr = reinterpret_cast<const bf16*>(bias->contiguous().data_ptr());
  }
  const int waves_per_block = 4;
  const int rows_per_block = 2 * waves_per_block;
  const dim3 grid((N + rows_per_block - 1) / rows_per_block);
  auto stream = c10::hip::getCurrentHIPStream();
#define LAUNCH(BB)                                                             \
  gemv_bf16_kernel<BB><<<grid, dim3(waves_per_block * WAVE_SIZE), 0, stream>>>( \
      reinterpret_cast<const bf16*>(wc.data_ptr()),                            \
      reinterpret_cast<const bf16*>(xc.data_ptr()), bptr,                      \
      out_f32 ? nullptr : reinterpret_cast<bf16*>(y.data_ptr()),               \
      out_f32 ? y.data_ptr<float>() : nullptr, relu2, N, K, (int)group_n)
  switch (B) {
    case 1: LAUNCH(1); break;
    case 2: LAUNCH(2); break;
    case 3: LAUNCH(3); break;
    case 4: LAUNCH(4); break;
    case 8: LAUNCH(8); break;
    case 16: LAUNCH(16); break;
    default: TORCH_CHECK(false, "gemv_bf16: pad B to one of 1,2,3,4,8,16 (python wrapper does)");
  }
#undef LAUNCH
  HIP_CHECK_KERNEL();
  return y;
}

// ---------------------------------------------------------------------------
// Skinny GEMM for decode batches of 5..64 rows: the same weight stream, with
// the products on the matrix cores. A workgroup owns 16 rows of W; its waves
// split K and reduce through LDS at the end, so that even N = 4096 fills the
// chip. Matrix fragments want one row per lane, memory wants consecutive lanes
// on consecutive bytes: each wave moves its 16 x 128 tile of W (and the x rows
// of the same K range) with coalesced loads into LDS of its own, the next
// tile's loads in flight meanwhile. No workgroup barrier in the loop.
// ---------------------------------------------------------------------------
constexpr int SK_KC = 128;                        // K per tile
constexpr int SK_STRIDE = SK_KC * 2 + 16;         // LDS bytes per row

template <int NB, int WAVES>
__global__ __launch_bounds__(WAVES * WAVE_SIZE) void gemm_skinny_kernel(
    const bf16* __restrict__ W, const bf16* __restrict__ x, bf16* __restrict__ y,
    float* __restrict__ yf, bool relu2, int B, int N, int K, int group_n) {
  constexpr int RED = WAVES * 16 * (16 * NB + 1) * 4;
  constexpr int TILE = 16 * (1 + NB) * SK_STRIDE;
  __shared__ __attribute__((aligned(16))) char lds[WAVES * TILE > RED ? WAVES * TILE : RED];
  const int lane = threadIdx.x & (WAVE_SIZE - 1), wid = threadIdx.x / WAVE_SIZE;
  const int lo16 = lane & 15, hi4 = lane >> 4;
  const int n0 = blockIdx.x * 16;
  if (group_n) x += (long)(n0 / group_n) * B * K;       // group_n % 16 == 0
  char* wl = lds + wid * TILE;                    // [16][SK_STRIDE]
  char* xl = wl + 16 * SK_STRIDE;                 // [16 NB][SK_STRIDE]

  gemv_f32x4 acc[NB];
#pragma unroll
  for (int b = 0; b < NB; ++b) acc[b] = gemv_f32x4{0.f, 0.f, 0.f, 0.f};
  const int tiles = (K + SK_KC - 1) / SK_KC;
  const int per = (tiles + WAVES - 1) / WAVES;
  const int t_lo = wid * per, t_hi = min(t_lo + per, tiles);

  // load j covers rows 4j + hi4, 16 bytes per lane at column 8 lo16
  gemv_bf16x8 wr[4], xr[4 * NB];
  auto fetch = [&](int t) {
    const int k = t * SK_KC + lo16 * 8;
    const bool in = k < K;                        // K % 8 == 0: all 8 or none
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      wr[j] = gemv_bf16x8{};
      if (in)
        wr[j] = *reinterpret_cast<const gemv_bf16x8*>(
            W + (long)min(n0 + 4 * j + hi4, N - 1) * K + k);
    }
#pragma unroll
    for (int j = 0; j < 4 * NB; ++j) {
      xr[j] = gemv_bf16x8{};
      if (in)
        xr[j] = *reinterpret_cast<const gemv_bf16x8*>(x + (long)min(4 * j + hi4, B - 1) * K + k);
    }
  };
  if (t_lo < t_hi) fetch(t_lo);
  for (int t = t_lo; t < t_hi; ++t) {
#pragma unroll
    for (int j = 0; j < 4; ++j)
      *reinterpret_cast<gemv_bf16x8*>(wl + (4 * j + hi4) * SK_STRIDE + lo16 * 16) = wr[j];
#pragma unroll
    for (int j = 0; j < 4 * NB; ++j)
      *reinterpret_cast<gemv_bf16x8*>(xl + (4 * j + hi4) * SK_STRIDE + lo16 * 16) = xr[j];
    __builtin_amdgcn_wave_barrier();
    if (t + 1 < t_hi) fetch(t + 1);
#pragma unroll
    for (int kk = 0; kk < SK_KC / 32; ++kk) {
      const int off = lo16 * SK_STRIDE + kk * 64 + hi4 * 16;
      const gemv_bf16x8 w = *reinterpret_cast<const gemv_bf16x8*>(wl + off);
#pragma unroll
      for (int b = 0; b < NB; ++b) {
        const gemv_bf16x8 v = *reinterpret_cast<const gemv_bf16x8*>(xl + b * 16 * SK_STRIDE + off);
        acc[b] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(w, v, acc[b], 0, 0, 0);
      }
    }
    __builtin_amdgcn_wave_barrier();              // the tile is overwritten next
  }
  __syncthreads();                                // tiles become the reduction buffer
  float* red = reinterpret_cast<float*>(lds);
  constexpr int RS = 16 * NB + 1;
#pragma unroll
  for (int b = 0; b < NB; ++b)
#pragma unroll
    for (int i = 0; i < 4; ++i) red[(wid * 16 + hi4 * 4 + i) * RS + b * 16 + lo16] = acc[b][i];
  __syncthreads();
  for (int i = threadIdx.x; i < 256 * NB; i += WAVES * WAVE_SIZE) {
    const int row = i & 15, col = i >> 4;
    if (n0 + row >= N || col >= B) continue;
    float t = 0.f;
#pragma unroll
    for (int w = 0; w < WAVES; ++w) t += red[(w * 16 + row) * RS + col];
    if (relu2) {
      t = fmaxf(t, 0.f);
      t *= t;
    }
    const long o = (long)col * N + n0 + row;
    if (yf) yf[o] = t;
    else y[o] = f2bf(t);
  }
}

at::Tensor gemm_skinny_bf16(const at::Tensor& x, const at::Tensor& w, bool relu2, bool out_f32,
                            int64_t group_n) {
  TORCH_CHECK(x.is_cuda() && w.is_cuda() && x.dtype() == at::kBFloat16 &&
                  w.dtype() == at::kBFloat16 && x.dim() == 2 && w.dim() == 2,
              "gemm_skinny_bf16: x [B,K], w [N,K] bf16 on the GPU");
  const int K = (int)x.size(1), N = (int)w.size(0);
  const int groups = group_n > 0 ? (int)((N + group_n - 1) / group_n) : 1;
  TORCH_CHECK(group_n >= 0 && group_n % 16 == 0 && x.size(0) % groups == 0,
              "gemm_skinny_bf16: group_n in whole tiles of 16, one [B,K] input per group");
  const int B = (int)x.size(0) / groups;
  TORCH_CHECK(w.size(1) == K && K % 8 == 0 && K >= 8 && N >= 1, "gemm_skinny_bf16: K % 8 == 0");
  TORCH_CHECK(B >= 1 && B <= 64, "gemm_skinny_bf16: 1..64 rows, got ", B);
  auto xc = x.contiguous(), wc = w.contiguous();
  auto y = at::empty({B, N}, x.options().dtype(out_f32 ? at::kFloat : at::kBFloat16));
  auto stream = c10::hip::getCurrentHIPStream();
#define LAUNCH(NB, WAVES)                                                                    \
  gemm_skinny_kernel<NB, WAVES>                                                              \
      <<<dim3((N + 15) / 16), dim3(WAVES * WAVE_SIZE), 0, stream>>>(                         \
          reinterpret_cast<const bf16*>(wc.data_ptr()),                                      \
          reinterpret_cast<const bf16*>(xc.data_ptr()),                                      \
          out_f32 ? nullptr : reinterpret_cast<bf16*>(y.data_ptr()),                         \
          out_f32 ? y.data_ptr<float>() : nullptr, relu2, B, N, K, (int)group_n)
  // waves per workgroup: enough of them across the chip, each with K left to
  // stream; LDS grows with the x rows
  const bool deep = K >= 2048;
  if (B <= 16) { if (deep) LAUNCH(1, 8); else LAUNCH(1, 4); }
  else if (B <= 32) { LAUNCH(2, 4); }
  else { LAUNCH(4, 2); }
#undef LAUNCH
  HIP_CHECK_KERNEL();
  return y;
}

}  // namespace amd_ops
