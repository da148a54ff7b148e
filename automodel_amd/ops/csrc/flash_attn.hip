// Flash attention fwd+bwd (CDNA4, gfx950) — BSHD + packed varlen (THD),
// causal, GQA, head dims {64, 96, 128, 192, 256} and split-dim MLA (qk 192 /
// v 128). Deterministic backward (no atomics).
//
// MI355X-native replacement for the reference's TE DotProductAttention /
// flash-attn backends (te_attention.py:352 arbitrary
// dims, distributed/thd_utils.py:85 THD varlen). Structure follows the CDNA4
// guide's fused-attention recipe (cdna_hip_programming.md Appendix B):
//   * swapped QK^T — mfma_f32_32x32x16_bf16 computing mfma(K, Q) so each
//     lane holds a P column for ONE q row -> softmax is in-register
//     (16 regs + one __shfl_xor(32) cross-half exchange)
//   * online softmax (running m, l per q row)
//   * P -> bf16 via packed cvt + __builtin_amdgcn_permlane32_swap to build
//     the PV A-fragment without LDS round trips (guide T12)
//   * K tile LDS-staged with XOR swizzle (guide T2 / Guideline 4), row
//     stride padded to a multiple of 256 B so the ((row&15)<<4) swizzle is
//     conflict-free at every head dim
//   * V tile staged TRANSPOSED in LDS (vt[d][k]) with its own XOR swizzle
//     so PV B-fragments are contiguous ds_read_b128
//
// Varlen (packed THD): per-token doc_start/doc_end arrays (precomputed from
// cu_seqlens in ops/attention.py) gate the causal mask to the query's own
// document; KV-tile ranges are clipped per block/wave so cross-document
// tiles are skipped, giving ONE kernel launch per packed batch.
//
// Backward determinism: the dKV kernel's grid is (kv tiles, Hk, B) and each
// block loops over the GQA query-head group, accumulating dK/dV in registers
// across the whole q loop — plain stores, no atomicAdd, bitwise
// run-to-run-identical grads (reference determinism discipline,
// moe/experts.py:66).

#include <torch/library.h>
#include <ATen/ATen.h>
#include <c10/hip/HIPStream.h>

#include "common.h"
#include "flash_attn.h"
#include "ops_api.h"

namespace amd_ops {

// ===========================================================================
// Forward
// ===========================================================================

template <int DQK, int DV, int WAVES, bool VARLEN>
__global__ __launch_bounds__(WAVES * WAVE_SIZE, 2) void flash_fwd_kernel(
    const bf16* __restrict__ q, const bf16* __restrict__ k, const bf16* __restrict__ v,
    bf16* __restrict__ out, float* __restrict__ lse, const int* __restrict__ doc_start,
    const bf16* __restrict__ sink, int B, int Sq, int Skv, int Hq, int Hk, int q_start,
    float scale, bool causal) {
  constexpr int KB = pad256(DQK * 2);     // K tile row stride (bytes)
  extern __shared__ __attribute__((aligned(16))) char smem[];
  char* k_lds = smem;                               // KVBLK*KB
  char* v_img = smem + KVBLK * KB;                  // subtiled [DV/16][32][16]
  float* bcast = reinterpret_cast<float*>(smem + KVBLK * KB + sub_img_bytes<DV>());
  int* bcast_skip = reinterpret_cast<int*>(bcast + WAVES * 32);

  const int tid = threadIdx.x;
  const int lane = tid & (WAVE_SIZE - 1);
  const int wid = tid / WAVE_SIZE;
  const int col = lane & 31;           // q row within wave tile (QK layout)
  const int half = lane >> 5;

  const int qblk0 = blockIdx.x * (WAVES * QBLK);
  const int h = blockIdx.y;
  const int b = blockIdx.z;
  const int kvh = h / (Hq / Hk);

  const long q_base = (((long)b * Sq) * Hq + h) * DQK;
  const long k_base = (((long)b * Skv) * Hk + kvh) * DQK;
  const long v_base = (((long)b * Skv) * Hk + kvh) * DV;
  const long o_base = (((long)b * Sq) * Hq + h) * DV;
  const long q_rs = (long)Hq * DQK, k_rs = (long)Hk * DQK;
  const long v_rs = (long)Hk * DV, o_rs = (long)Hq * DV;

  const int q0 = qblk0 + wid * QBLK;   // this wave's first q row

  // ---- load Q fragments to registers: lane holds Q[q0+col][8*half + j + 16*c]
  bf16x8_v qfrag[DQK / 16];
#pragma unroll
  for (int c = 0; c < DQK / 16; ++c) {
    const bf16* src = q + q_base + (long)(q0 + col) * q_rs + c * 16 + half * 8;
    qfrag[c] = *reinterpret_cast<const bf16x8_v*>(src);
  }

  // varlen doc bounds: lane's q row is fixed for the whole kernel
  const int qg_lane = q_start + q0 + col;
  const int ds_lane = VARLEN ? doc_start[qg_lane] : 0;        // lane's doc start
  const int ds_wave = VARLEN ? doc_start[q_start + q0] : 0;   // wave min (non-decreasing)

  // ---- accumulators
  f32x16 o_acc[DV / 32];
#pragma unroll
  for (int t = 0; t < DV / 32; ++t)
#pragma unroll
    for (int r = 0; r < 16; ++r) o_acc[t][r] = 0.f;
  float m_run = -1e30f, l_run = 0.f;

  const int q_block_max = q_start + qblk0 + WAVES * QBLK - 1;
  const int n_tiles = causal ? (min(q_block_max, Skv - 1) / KVBLK + 1)
                             : (Skv + KVBLK - 1) / KVBLK;
  // block-uniform start tile (varlen: nothing before the block's first doc)
  const int jt0 = VARLEN ? doc_start[q_start + qblk0] / KVBLK : 0;

  for (int jt = jt0; jt < n_tiles; ++jt) {
    const int k0 = jt * KVBLK;
    // ---- stage K tile (swizzled) and V^T tile cooperatively
    {
      constexpr int KCH = DQK / 8;     // 16-B chunks per K row
      for (int idx = tid; idx < KVBLK * KCH; idx += WAVES * WAVE_SIZE) {
        const int row = idx / KCH, c0 = (idx % KCH) * 8;
        const int ks = min(k0 + row, Skv - 1);  // overhang rows masked later
        *reinterpret_cast<bf16x8*>(k_lds + row_lds_off(row, c0 * 2, KB)) =
            *reinterpret_cast<const bf16x8*>(k + k_base + (long)ks * k_rs + c0);
      }
      constexpr int VCH = DV / 8;
      for (int idx = tid; idx < KVBLK * VCH; idx += WAVES * WAVE_SIZE) {
        const int row = idx / VCH, c0 = (idx % VCH) * 8;
        const int ks = min(k0 + row, Skv - 1);
        // vectorized subtile store (the round-1 path scatter-stored 8
        // scalars per vector to build a transposed image)
        *reinterpret_cast<bf16x8*>(v_img + sub_off(row, c0)) =
            *reinterpret_cast<const bf16x8*>(v + v_base + (long)ks * v_rs + c0);
      }
    }
    __syncthreads();

    const bool tile_live = (!causal || (k0 <= q_start + q0 + QBLK - 1)) &&
                           (!VARLEN || (k0 + KVBLK > ds_wave));
    float alpha = 1.f;
    bf16x8_v pa0, pa1;
    if (tile_live) {
      // ---- QK^T swapped: P[k][q] = sum_d K[k][d] * Q[q][d]
      f32x16 p;
#pragma unroll
      for (int r = 0; r < 16; ++r) p[r] = 0.f;
#pragma unroll
      for (int c = 0; c < DQK / 16; ++c) {
        bf16x8_v ka = *reinterpret_cast<const bf16x8_v*>(
            k_lds + row_lds_off(col, (c * 16 + half * 8) * 2, KB));
        p = __builtin_amdgcn_mfma_f32_32x32x16_bf16(ka, qfrag[c], p, 0, 0, 0);
      }

      // ---- masked online softmax, IN PLACE in the p accumulator
      const int qg = qg_lane;
      float tile_max = -1e30f;
#pragma unroll
      for (int r = 0; r < 16; ++r) {
        const int kg = k0 + (r & 3) + 8 * (r >> 2) + 4 * half;
        float sv = p[r] * scale;
        if ((causal && kg > qg) || kg >= Skv || (VARLEN && kg < ds_lane)) sv = -1e30f;
        p[r] = sv;
        tile_max = fmaxf(tile_max, sv);
      }
      tile_max = fmaxf(tile_max, __shfl_xor(tile_max, 32));
      // defer-max (guide T13, THR=8): if no row's max grew past m+THR, keep
      // the old max and skip the O-wide rescale pass — P is then bounded by
      // e^8 instead of 1, which the f32 accumulator tolerates. Wave-uniform
      // decision taken BEFORE this tile's P is exponentiated (the textbook-
      // safe order; guide T13 correctness hazard).
      const bool need_rescale = !__all(tile_max <= m_run + 8.0f);
      const float m_new = need_rescale ? fmaxf(m_run, tile_max) : m_run;
      alpha = need_rescale ? __expf(m_run - m_new) : 1.f;
      float psum = 0.f;
#pragma unroll
      for (int r = 0; r < 16; ++r) {
        float e = __expf(p[r] - m_new);
        p[r] = e;
        psum += e;
      }
      psum += __shfl_xor(psum, 32);
      l_run = l_run * alpha + psum;
      m_run = m_new;

      // ---- P f32 -> bf16 packed pairs, permlane32_swap into A-fragment layout
      unsigned int pk[8];
#pragma unroll
      for (int i = 0; i < 8; ++i) {
        unsigned lo = __builtin_bit_cast(unsigned short, f2bf(p[2 * i]));
        unsigned hi = __builtin_bit_cast(unsigned short, f2bf(p[2 * i + 1]));
        pk[i] = lo | (hi << 16);
      }
#pragma unroll
      for (int i = 0; i < 2; ++i) {
        auto r02 = __builtin_amdgcn_permlane32_swap(pk[4 * i + 0], pk[4 * i + 2], false, false);
        auto r13 = __builtin_amdgcn_permlane32_swap(pk[4 * i + 1], pk[4 * i + 3], false, false);
        unsigned frag[4] = {(unsigned)r02[0], (unsigned)r13[0], (unsigned)r02[1], (unsigned)r13[1]};
        if (i == 0) pa0 = __builtin_bit_cast(bf16x8_v, *reinterpret_cast<ulonglong2*>(frag));
        else pa1 = __builtin_bit_cast(bf16x8_v, *reinterpret_cast<ulonglong2*>(frag));
      }

      // ---- broadcast alpha to O layout via LDS (sign bit of slot 0 set
      // when the whole wave deferred, so the rescale pass can be skipped)
      if (lane < 32) bcast[wid * 32 + lane] = alpha;
      if (lane == 0) bcast_skip[wid] = need_rescale ? 1 : 0;
    }
    // (waves with dead tiles skip compute but still hit the barriers)
    __syncthreads();

    if (tile_live) {
      // ---- rescale O by alpha (skipped on deferred tiles, guide T13)
      if (bcast_skip[wid]) {
#pragma unroll
        for (int t = 0; t < DV / 32; ++t) {
#pragma unroll
          for (int r = 0; r < 16; ++r) {
            const int row = (r & 3) + 8 * (r >> 2) + 4 * half;
            o_acc[t][r] *= bcast[wid * 32 + row];
          }
        }
      }
      // software-pipelined tr16 PV: tile t+1's four transpose reads are in
      // flight during tile t's MFMAs; the counted s_waitcnt takes the
      // fragment registers as "+v" operands so the consuming MFMAs cannot
      // be scheduled past it. lgkmcnt(4) is conservative-safe: compiler-
      // issued LDS ops between ours only strengthen the wait.
      const unsigned v_base_a = lds_addr(v_img);
      if constexpr (DV > 128) {
#pragma unroll
        for (int t = 0; t < DV / 32; ++t) {
          bf16x8_v vb0 = tr16_frag(v_base_a, t, half, lane);
          bf16x8_v vb1 = tr16_frag(v_base_a, t, half + 2, lane);
          o_acc[t] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(pa0, vb0, o_acc[t], 0, 0, 0);
          o_acc[t] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(pa1, vb1, o_acc[t], 0, 0, 0);
        }
      } else {
      unsigned long long f0a, f0b, f1a, f1b, g0a, g0b, g1a, g1b;
      auto tr_issue = [&](int t, unsigned long long& r0a, unsigned long long& r0b,
                          unsigned long long& r1a, unsigned long long& r1b) {
        const unsigned base = v_base_a +
            (unsigned)((t * 2 + ((lane >> 4) & 1)) * 1152 + (lane & 15) * 8);
        const unsigned klo = (unsigned)(8 * half) * 32;
        const unsigned khi = (unsigned)(8 * (half + 2)) * 32;
        asm volatile("ds_read_b64_tr_b16 %0, %4\n\t"
                     "ds_read_b64_tr_b16 %1, %4 offset:128\n\t"
                     "ds_read_b64_tr_b16 %2, %5\n\t"
                     "ds_read_b64_tr_b16 %3, %5 offset:128"
                     : "=v"(r0a), "=v"(r0b), "=v"(r1a), "=v"(r1b)
                     : "v"(base + klo), "v"(base + khi));
      };
      tr_issue(0, f0a, f0b, f1a, f1b);
#pragma unroll
      for (int t = 0; t < DV / 32; ++t) {
        unsigned long long& c0a = (t & 1) ? g0a : f0a;
        unsigned long long& c0b = (t & 1) ? g0b : f0b;
        unsigned long long& c1a = (t & 1) ? g1a : f1a;
        unsigned long long& c1b = (t & 1) ? g1b : f1b;
        if (t + 1 < DV / 32) {
          tr_issue(t + 1, (t & 1) ? f0a : g0a, (t & 1) ? f0b : g0b,
                   (t & 1) ? f1a : g1a, (t & 1) ? f1b : g1b);
          asm volatile("s_waitcnt lgkmcnt(4)"
                       : "+v"(c0a), "+v"(c0b), "+v"(c1a), "+v"(c1b));
        } else {
          asm volatile("s_waitcnt lgkmcnt(0)"
                       : "+v"(c0a), "+v"(c0b), "+v"(c1a), "+v"(c1b));
        }
        ulonglong2 u0{c0a, c0b}, u1{c1a, c1b};
        bf16x8_v vb0 = __builtin_bit_cast(bf16x8_v, u0);
        bf16x8_v vb1 = __builtin_bit_cast(bf16x8_v, u1);
        o_acc[t] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(pa0, vb0, o_acc[t], 0, 0, 0);
        o_acc[t] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(pa1, vb1, o_acc[t], 0, 0, 0);
      }
      }
    }
    __syncthreads();
  }

  // ---- epilogue: normalize by l, write O and LSE. A sink is one more logit in
  // the denominator, without a key (m_run bounds the scores, so that only a
  // sink far above all of them can overflow: the output is 0 then, as it is)
  if (sink) l_run += __expf(bf2f(sink[h]) - m_run);
  if (lane < 32) bcast[wid * 32 + lane] = (l_run > 0.f) ? 1.f / l_run : 0.f;
  __syncthreads();

  const int qg = q0 + col;
  if (lane < 32 && qg < Sq) {
    lse[((long)b * Hq + h) * Sq + qg] = (l_run > 0.f) ? m_run + __logf(l_run) : -1e30f;
  }
#pragma unroll
  for (int t = 0; t < DV / 32; ++t) {
#pragma unroll
    for (int r = 0; r < 16; ++r) {
      const int row = (r & 3) + 8 * (r >> 2) + 4 * half;  // q row in wave tile
      const int qrow = q0 + row;
      if (qrow < Sq) {
        const float inv_l = bcast[wid * 32 + row];
        out[o_base + (long)qrow * o_rs + t * 32 + col] = f2bf(o_acc[t][r] * inv_l);
      }
    }
  }
}

template <int DQK, int DV, int WAVES, bool VARLEN>
static void launch_fwd(const at::Tensor& q, const at::Tensor& k, const at::Tensor& v,
                       at::Tensor& out, at::Tensor& lse, const int* doc_start,
                       const bf16* sink, int B, int Sq, int Skv, int Hq, int Hk, int q_start,
                       float scale, bool causal, hipStream_t stream) {
  const dim3 grid(Sq / (WAVES * QBLK), Hq, B);
  const size_t smem = KVBLK * pad256(DQK * 2) + sub_img_bytes<DV>() +
                      WAVES * 33 * sizeof(float);
  hipLaunchKernelGGL((flash_fwd_kernel<DQK, DV, WAVES, VARLEN>), grid,
                     dim3(WAVES * WAVE_SIZE), smem, stream,
                     reinterpret_cast<const bf16*>(q.data_ptr()),
                     reinterpret_cast<const bf16*>(k.data_ptr()),
                     reinterpret_cast<const bf16*>(v.data_ptr()),
                     reinterpret_cast<bf16*>(out.data_ptr()), lse.data_ptr<float>(),
                     doc_start, sink, B, Sq, Skv, Hq, Hk, q_start, scale, causal);
  HIP_CHECK_KERNEL();
}

std::tuple<at::Tensor, at::Tensor> flash_attn_fwd(
    const at::Tensor& q, const at::Tensor& k, const at::Tensor& v, double scale,
    bool causal, int64_t q_start, const std::optional<at::Tensor>& doc_start,
    const std::optional<at::Tensor>& sink) {
  TORCH_CHECK(q.is_cuda() && q.dim() == 4 && q.scalar_type() == at::kBFloat16,
              "flash_attn_fwd: q must be [B,S,Hq,D] bf16");
  const int B = q.size(0), Sq = q.size(1), Hq = q.size(2), Dqk = q.size(3);
  const int Skv = k.size(1), Hk = k.size(2), Dv = v.size(3);
  TORCH_CHECK(Hq % Hk == 0, "flash_attn_fwd: Hq must be divisible by Hk");
  TORCH_CHECK(Sq % (4 * QBLK) == 0, "flash_attn_fwd: Sq must be a multiple of 128");
  TORCH_CHECK(Skv % KVBLK == 0, "flash_attn_fwd: Skv must be a multiple of 32");
  const bool varlen = doc_start.has_value();
  const int* ds_ptr = varlen ? doc_start->data_ptr<int>() : nullptr;
  if (varlen) TORCH_CHECK(causal && B == 1, "varlen flash is causal with B==1");
  if (sink)
    TORCH_CHECK(sink->is_cuda() && sink->is_contiguous() && sink->numel() == Hq &&
                    sink->scalar_type() == at::kBFloat16, "flash_attn_fwd: sink [Hq] bf16");
  const bf16* sk_ptr = sink ? reinterpret_cast<const bf16*>(sink->data_ptr()) : nullptr;
  auto out = at::empty({B, Sq, Hq, Dv}, q.options());
  auto lse = at::empty({B, Hq, Sq}, q.options().dtype(at::kFloat));
  auto stream = c10::hip::getCurrentHIPStream().stream();

  bool done = false;
#define FA_FWD_CASE(A, C)                                                             \
  if (!done && Dqk == A && Dv == C) {                                                 \
    done = true;                                                                      \
    if (varlen && Sq % (8 * QBLK) == 0) {                                             \
      launch_fwd<A, C, 8, true>(q, k, v, out, lse, ds_ptr, sk_ptr, B, Sq, Skv, Hq, Hk, \
                                (int)q_start, (float)scale, causal, stream);          \
    } else if (varlen) {                                                              \
      launch_fwd<A, C, 4, true>(q, k, v, out, lse, ds_ptr, sk_ptr, B, Sq, Skv, Hq, Hk, \
                                (int)q_start, (float)scale, causal, stream);          \
    } else if (Sq % (8 * QBLK) == 0) {                                                \
      launch_fwd<A, C, 8, false>(q, k, v, out, lse, nullptr, sk_ptr, B, Sq, Skv, Hq, Hk, \
                                 (int)q_start, (float)scale, causal, stream);         \
    } else {                                                                          \
      launch_fwd<A, C, 4, false>(q, k, v, out, lse, nullptr, sk_ptr, B, Sq, Skv, Hq, Hk, \
                                 (int)q_start, (float)scale, causal, stream);         \
    }                                                                                 \
  }
  FA_FWD_CASE(64, 64)
  FA_FWD_CASE(96, 96)
  FA_FWD_CASE(128, 128)
  FA_FWD_CASE(192, 128)
  FA_FWD_CASE(192, 192)
  FA_FWD_CASE(256, 256)
#undef FA_FWD_CASE
  TORCH_CHECK(done, "flash_attn_fwd: unsupported head dims (Dqk=", Dqk, ", Dv=", Dv,
              "); supported pairs: (64,64),(96,96),(128,128),(192,128),(192,192),(256,256)");
  return {out, lse};
}

}  // namespace amd_ops
