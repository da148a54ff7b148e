// Flash attention backward (CDNA4, gfx950): deterministic dKV (kv-parallel) and
// dQ (q-parallel) kernels of the forward in flash_attn.hip, plus the MFMA and
// transpose-read layout probes.

#include <torch/library.h>
#include <ATen/ATen.h>
#include <c10/hip/HIPStream.h>

#include "common.h"
#include "flash_attn.h"
#include "ops_api.h"

namespace amd_ops {

// ===========================================================================
// Backward: flash-attention-2 style split.
//   delta kernel: delta[b,h,s] = rowsum(dO * O)
//   kernel A (kv-parallel, DETERMINISTIC): grid over (kv tiles, Hk, B); each
//     block loops the GQA query-head group and all q tiles, accumulating
//     dK/dV in registers; plain bf16 stores (no atomics -> bitwise
//     reproducible grads).
//   kernel B (q-parallel): recompute S in [q][k] layout, accumulate dQ.
// ===========================================================================

__global__ void fa_delta_kernel(const bf16* __restrict__ dout, const bf16* __restrict__ o,
                                float* __restrict__ delta, int S, int Hq, int DV,
                                long rows) {
  // row r = ((b*S + s)*Hq + h); one wave per row
  const long row = ((long)blockIdx.x * blockDim.x + threadIdx.x) / WAVE_SIZE;
  if (row >= rows) return;
  const int lane = threadIdx.x & (WAVE_SIZE - 1);
  const bf16* dp = dout + row * DV;
  const bf16* op = o + row * DV;
  float acc = 0.f;
  for (int j = lane * 2; j < DV; j += 2 * WAVE_SIZE) {
    acc += bf2f(dp[j]) * bf2f(op[j]) + bf2f(dp[j + 1]) * bf2f(op[j + 1]);
  }
  acc = wave_reduce_sum(acc);
  if (lane == 0) {
    const long h = row % Hq;
    const long bs = row / Hq;
    const long b = bs / S, s = bs % S;
    delta[(b * Hq + h) * S + s] = acc;
  }
}

template <int DQK, int DV, int WAVES, bool VARLEN>
__global__ __launch_bounds__(WAVES * WAVE_SIZE, occ_dkv(DQK, DV)) void flash_bwd_dkv_kernel(
    const bf16* __restrict__ dout, const bf16* __restrict__ q, const bf16* __restrict__ k,
    const bf16* __restrict__ v, const float* __restrict__ lse, const float* __restrict__ delta,
    bf16* __restrict__ dk, bf16* __restrict__ dv, const int* __restrict__ doc_end,
    int B, int Sq, int Skv, int Hq, int Hk, int q_start, float scale, bool causal) {
  extern __shared__ __attribute__((aligned(16))) char smem[];
  char* q_img = smem;                                    // subtiled [DQK/16][32][16]
  char* do_img = smem + sub_img_bytes<DQK>();            // subtiled [DV/16][32][16]
  char* tbuf = do_img + sub_img_bytes<DV>();             // WAVES*2048

  const int tid = threadIdx.x;
  const int lane = tid & 63;
  const int wid = tid / 64;
  const int col = lane & 31;
  const int half = lane >> 5;

  const int kvb = blockIdx.x * (WAVES * 32);
  const int kvh = blockIdx.y;
  const int b = blockIdx.z;
  const int G = Hq / Hk;               // GQA group size
  const int kv0 = kvb + wid * 32;      // this wave's kv rows

  const long k_base = (((long)b * Skv) * Hk + kvh) * DQK;
  const long v_base = (((long)b * Skv) * Hk + kvh) * DV;
  const long k_rs = (long)Hk * DQK, v_rs = (long)Hk * DV;
  const long q_rs = (long)Hq * DQK, do_rs = (long)Hq * DV;

  // K/V rows of this wave -> A fragments in registers
  bf16x8_v kfrag[DQK / 16], vfrag[DV / 16];
#pragma unroll
  for (int c = 0; c < DQK / 16; ++c)
    kfrag[c] = *reinterpret_cast<const bf16x8_v*>(
        k + k_base + (long)(kv0 + col) * k_rs + c * 16 + half * 8);
#pragma unroll
  for (int c = 0; c < DV / 16; ++c)
    vfrag[c] = *reinterpret_cast<const bf16x8_v*>(
        v + v_base + (long)(kv0 + col) * v_rs + c * 16 + half * 8);

  // varlen: per-element doc_end for this wave's 16 kv rows (fixed all kernel)
  int dend[16];
  int dend_wave = Sq;                  // max over the wave's rows
  if (VARLEN) {
#pragma unroll
    for (int r = 0; r < 16; ++r) {
      const int kg = kv0 + (r & 3) + 8 * (r >> 2) + 4 * half;
      dend[r] = doc_end[min(kg, Skv - 1)];
    }
    dend_wave = doc_end[min(kv0 + 31, Skv - 1)];
  }

  f32x16 dk_acc[DQK / 32], dv_acc[DV / 32];
#pragma unroll
  for (int t = 0; t < DQK / 32; ++t)
#pragma unroll
    for (int r = 0; r < 16; ++r) dk_acc[t][r] = 0.f;
#pragma unroll
  for (int t = 0; t < DV / 32; ++t)
#pragma unroll
    for (int r = 0; r < 16; ++r) dv_acc[t][r] = 0.f;

  char* tb = tbuf + wid * 2048;
  const int jq_start = causal ? (kvb > q_start ? (kvb - q_start) / 32 : 0) : 0;
  // block-uniform end (varlen: nothing after the block's last doc)
  int jq_end = Sq / 32;
  if (VARLEN) {
    const int de_blk = doc_end[min(kvb + WAVES * 32 - 1, Skv - 1)];
    jq_end = min(jq_end, (de_blk - q_start + 31) / 32);
  }

  for (int g = 0; g < G; ++g) {
    const int h = kvh * G + g;
    const long q_base = (((long)b * Sq) * Hq + h) * DQK;
    const long do_base = (((long)b * Sq) * Hq + h) * DV;
    const float* lse_row = lse + ((long)b * Hq + h) * Sq;
    const float* dlt_row = delta + ((long)b * Hq + h) * Sq;

    for (int jq = jq_start; jq < jq_end; ++jq) {
      const int q0 = jq * 32;
      // ---- cooperative stage: ONE subtiled image per tensor (serves both
      // the row-chunk B-frags and the tr16 transposed B-frags — the round-1
      // kernel kept a row image AND a scalar-scattered transposed image)
      {
        constexpr int QCH = DQK / 8;
        for (int idx = tid; idx < 32 * QCH; idx += WAVES * 64) {
          const int rr = idx / QCH, c0 = (idx % QCH) * 8;
          *reinterpret_cast<bf16x8*>(q_img + sub_off(rr, c0)) =
              *reinterpret_cast<const bf16x8*>(q + q_base + (long)(q0 + rr) * q_rs + c0);
        }
        constexpr int OCH = DV / 8;
        for (int idx = tid; idx < 32 * OCH; idx += WAVES * 64) {
          const int rr = idx / OCH, c0 = (idx % OCH) * 8;
          *reinterpret_cast<bf16x8*>(do_img + sub_off(rr, c0)) =
              *reinterpret_cast<const bf16x8*>(
                  dout + do_base + (long)(q0 + rr) * do_rs + c0);
        }
      }
      __syncthreads();

      const bool live = (!causal || (q_start + q0 + 31 >= kv0)) &&
                        (!VARLEN || (q_start + q0 < dend_wave));
      if (live) {
        const int ql = q0 + col;          // local q row (lse/delta index)
        const int qg = q_start + ql;      // global position (mask)
        const float lse_q = lse_row[ql];
        const float dlt_q = dlt_row[ql];

        // ---- S^T = K Q^T (rows = kv, cols = q)
        f32x16 st;
#pragma unroll
        for (int r = 0; r < 16; ++r) st[r] = 0.f;
#pragma unroll
        for (int c = 0; c < DQK / 16; ++c) {
          bf16x8_v qb = *reinterpret_cast<const bf16x8_v*>(
              q_img + sub_off(col, c * 16 + half * 8));
          st = __builtin_amdgcn_mfma_f32_32x32x16_bf16(kfrag[c], qb, st, 0, 0, 0);
        }
        // ---- dP^T = V dO^T
        f32x16 dpt;
#pragma unroll
        for (int r = 0; r < 16; ++r) dpt[r] = 0.f;
#pragma unroll
        for (int c = 0; c < DV / 16; ++c) {
          bf16x8_v db = *reinterpret_cast<const bf16x8_v*>(
              do_img + sub_off(col, c * 16 + half * 8));
          dpt = __builtin_amdgcn_mfma_f32_32x32x16_bf16(vfrag[c], db, dpt, 0, 0, 0);
        }

        // in place: st becomes P^T, dpt becomes dS^T
#pragma unroll
        for (int r = 0; r < 16; ++r) {
          const int kg = kv0 + (r & 3) + 8 * (r >> 2) + 4 * half;
          const bool masked = (causal && kg > qg) || kg >= Skv ||
                              (VARLEN && qg >= dend[r]);
          const float pv = masked ? 0.f : __expf(st[r] * scale - lse_q);
          st[r] = pv;
          dpt[r] = pv * (dpt[r] - dlt_q) * scale;
        }

        // ---- transpose P^T -> A-frags via wave-local LDS buffer, accumulate dV
#pragma unroll
        for (int r = 0; r < 16; ++r) {
          const int krow = (r & 3) + 8 * (r >> 2) + 4 * half;
          *reinterpret_cast<bf16*>(tb + tb_off(krow, col * 2)) = f2bf(st[r]);
        }
        __builtin_amdgcn_wave_barrier();
        const unsigned do_base_a = lds_addr(do_img);
        if constexpr (!pipe_ok_dkv(DQK, DV)) {
#pragma unroll
          for (int c2 = 0; c2 < 2; ++c2) {
            bf16x8_v pa = *reinterpret_cast<const bf16x8_v*>(
                tb + tb_off(col, (c2 * 16 + half * 8) * 2));
#pragma unroll
            for (int t = 0; t < DV / 32; ++t) {
              bf16x8_v dob = tr16_frag(do_base_a, t, c2 * 2 + half, lane);
              dv_acc[t] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(pa, dob, dv_acc[t], 0, 0, 0);
            }
          }
        } else {
          bf16x8_v paf[2];
#pragma unroll
          for (int c2 = 0; c2 < 2; ++c2)
            paf[c2] = *reinterpret_cast<const bf16x8_v*>(
                tb + tb_off(col, (c2 * 16 + half * 8) * 2));
          constexpr int NT = DV / 32;
          unsigned long long pA, pB, qA, qB;
          auto addr_f = [&](int i) {
            const int c2 = i / NT, t = i % NT;
            return do_base_a + (unsigned)((t * 2 + ((lane >> 4) & 1)) * 1152 +
                                          (8 * (c2 * 2 + half)) * 32 + (lane & 15) * 8);
          };
          tr16_issue2(addr_f(0), pA, pB);
#pragma unroll
          for (int i = 0; i < 2 * NT; ++i) {
            const bool last = (i + 1 == 2 * NT);
            if (!last) tr16_issue2(addr_f(i + 1), (i & 1) ? pA : qA, (i & 1) ? pB : qB);
            bf16x8_v dob = tr16_take((i & 1) ? qA : pA, (i & 1) ? qB : pB, !last);
            dv_acc[i % NT] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(
                paf[i / NT], dob, dv_acc[i % NT], 0, 0, 0);
          }
        }
        // ---- transpose dS^T, accumulate dK
        __builtin_amdgcn_wave_barrier();
#pragma unroll
        for (int r = 0; r < 16; ++r) {
          const int krow = (r & 3) + 8 * (r >> 2) + 4 * half;
          *reinterpret_cast<bf16*>(tb + tb_off(krow, col * 2)) = f2bf(dpt[r]);
        }
        __builtin_amdgcn_wave_barrier();
        const unsigned q_base_a = lds_addr(q_img);
        if constexpr (!pipe_ok_dkv(DQK, DV)) {
#pragma unroll
          for (int c2 = 0; c2 < 2; ++c2) {
            bf16x8_v da = *reinterpret_cast<const bf16x8_v*>(
                tb + tb_off(col, (c2 * 16 + half * 8) * 2));
#pragma unroll
            for (int t = 0; t < DQK / 32; ++t) {
              bf16x8_v qb2 = tr16_frag(q_base_a, t, c2 * 2 + half, lane);
              dk_acc[t] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(da, qb2, dk_acc[t], 0, 0, 0);
            }
          }
        } else {
          bf16x8_v daf[2];
#pragma unroll
          for (int c2 = 0; c2 < 2; ++c2)
            daf[c2] = *reinterpret_cast<const bf16x8_v*>(
                tb + tb_off(col, (c2 * 16 + half * 8) * 2));
          constexpr int NT = DQK / 32;
          unsigned long long pA, pB, qA, qB;
          auto addr_f = [&](int i) {
            const int c2 = i / NT, t = i % NT;
            return q_base_a + (unsigned)((t * 2 + ((lane >> 4) & 1)) * 1152 +
                                         (8 * (c2 * 2 + half)) * 32 + (lane & 15) * 8);
          };
          tr16_issue2(addr_f(0), pA, pB);
#pragma unroll
          for (int i = 0; i < 2 * NT; ++i) {
            const bool last = (i + 1 == 2 * NT);
            if (!last) tr16_issue2(addr_f(i + 1), (i & 1) ? pA : qA, (i & 1) ? pB : qB);
            bf16x8_v qb2 = tr16_take((i & 1) ? qA : pA, (i & 1) ? qB : pB, !last);
            dk_acc[i % NT] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(
                daf[i / NT], qb2, dk_acc[i % NT], 0, 0, 0);
          }
        }
      }
      __syncthreads();
    }
  }

  // ---- epilogue: plain bf16 stores — each kv row is owned by exactly one
  // wave of one block (grid is per-Hk), so no cross-block accumulation.
#pragma unroll
  for (int r = 0; r < 16; ++r) {
    const int krow = (r & 3) + 8 * (r >> 2) + 4 * half;
    const int kg = kv0 + krow;
    if (kg < Skv) {
#pragma unroll
      for (int t = 0; t < DQK / 32; ++t)
        dk[k_base + (long)kg * k_rs + t * 32 + col] = f2bf(dk_acc[t][r]);
#pragma unroll
      for (int t = 0; t < DV / 32; ++t)
        dv[v_base + (long)kg * v_rs + t * 32 + col] = f2bf(dv_acc[t][r]);
    }
  }
}

template <int DQK, int DV, int WAVES, bool VARLEN>
__global__ __launch_bounds__(WAVES * WAVE_SIZE, occ_dq(DQK, DV)) void flash_bwd_dq_kernel(
    const bf16* __restrict__ dout, const bf16* __restrict__ q, const bf16* __restrict__ k,
    const bf16* __restrict__ v, const float* __restrict__ lse, const float* __restrict__ delta,
    bf16* __restrict__ dq, const int* __restrict__ doc_start, int B, int Sq, int Skv,
    int Hq, int Hk, int q_start, float scale, bool causal) {
  extern __shared__ __attribute__((aligned(16))) char smem[];
  char* k_img = smem;                                  // subtiled [DQK/16][32][16]
  char* v_img = smem + sub_img_bytes<DQK>();           // subtiled [DV/16][32][16]
  char* tbuf = v_img + sub_img_bytes<DV>();            // WAVES*2048
  float* stats = reinterpret_cast<float*>(tbuf + WAVES * 2048);  // 3*WAVES*32

  const int tid = threadIdx.x;
  const int lane = tid & 63;
  const int wid = tid / 64;
  const int col = lane & 31;
  const int half = lane >> 5;

  const int qb_blk = blockIdx.x * (WAVES * 32);
  const int h = blockIdx.y;
  const int b = blockIdx.z;
  const int kvh = h / (Hq / Hk);
  const int q0 = qb_blk + wid * 32;

  const long q_base = (((long)b * Sq) * Hq + h) * DQK;
  const long do_base = (((long)b * Sq) * Hq + h) * DV;
  const long k_base = (((long)b * Skv) * Hk + kvh) * DQK;
  const long v_base = (((long)b * Skv) * Hk + kvh) * DV;
  const long q_rs = (long)Hq * DQK, do_rs = (long)Hq * DV;
  const long k_rs = (long)Hk * DQK, v_rs = (long)Hk * DV;
  const float* lse_row = lse + ((long)b * Hq + h) * Sq;
  const float* dlt_row = delta + ((long)b * Hq + h) * Sq;

  // Q/dO rows of this wave as A-fragments
  bf16x8_v qfrag[DQK / 16], dofrag[DV / 16];
#pragma unroll
  for (int c = 0; c < DQK / 16; ++c)
    qfrag[c] = *reinterpret_cast<const bf16x8_v*>(
        q + q_base + (long)(q0 + col) * q_rs + c * 16 + half * 8);
#pragma unroll
  for (int c = 0; c < DV / 16; ++c)
    dofrag[c] = *reinterpret_cast<const bf16x8_v*>(
        dout + do_base + (long)(q0 + col) * do_rs + c * 16 + half * 8);
  // lse/delta(/doc_start) for the block's q rows -> LDS
  if (tid < WAVES * 32) {
    stats[tid] = lse_row[qb_blk + tid];
    stats[WAVES * 32 + tid] = dlt_row[qb_blk + tid];
    if (VARLEN) stats[2 * WAVES * 32 + tid] = (float)doc_start[q_start + qb_blk + tid];
  }

  f32x16 dq_acc[DQK / 32];
#pragma unroll
  for (int t = 0; t < DQK / 32; ++t)
#pragma unroll
    for (int r = 0; r < 16; ++r) dq_acc[t][r] = 0.f;

  char* tb = tbuf + wid * 2048;
  const int ds_wave = VARLEN ? doc_start[q_start + q0] : 0;
  const int block_q_max = q_start + qb_blk + WAVES * 32 - 1;
  const int n_tiles = causal ? (min(block_q_max, Skv - 1) / 32 + 1) : (Skv + 31) / 32;
  const int jk0 = VARLEN ? doc_start[q_start + qb_blk] / 32 : 0;

  for (int jk = jk0; jk < n_tiles; ++jk) {
    const int k0 = jk * 32;
    // ---- stage K and V as subtiled images (one image serves both the
    // row-chunk and the tr16 transposed reads)
    {
      constexpr int KCH = DQK / 8;
      for (int idx = tid; idx < 32 * KCH; idx += WAVES * 64) {
        const int rr = idx / KCH, c0 = (idx % KCH) * 8;
        const int ks = min(k0 + rr, Skv - 1);  // overhang masked in compute
        *reinterpret_cast<bf16x8*>(k_img + sub_off(rr, c0)) =
            *reinterpret_cast<const bf16x8*>(k + k_base + (long)ks * k_rs + c0);
      }
      constexpr int VCH = DV / 8;
      for (int idx = tid; idx < 32 * VCH; idx += WAVES * 64) {
        const int rr = idx / VCH, c0 = (idx % VCH) * 8;
        const int ks = min(k0 + rr, Skv - 1);
        *reinterpret_cast<bf16x8*>(v_img + sub_off(rr, c0)) =
            *reinterpret_cast<const bf16x8*>(v + v_base + (long)ks * v_rs + c0);
      }
    }
    __syncthreads();

    const bool live = (!causal || (k0 <= q_start + q0 + 31)) &&
                      (!VARLEN || (k0 + 31 >= ds_wave));
    if (live) {
      // ---- S[q][k] = Q K^T : A=Q rows, B from k_rows (contiguous d)
      f32x16 s;
#pragma unroll
      for (int r = 0; r < 16; ++r) s[r] = 0.f;
#pragma unroll
      for (int c = 0; c < DQK / 16; ++c) {
        bf16x8_v kb = *reinterpret_cast<const bf16x8_v*>(
            k_img + sub_off(col, c * 16 + half * 8));
        s = __builtin_amdgcn_mfma_f32_32x32x16_bf16(qfrag[c], kb, s, 0, 0, 0);
      }
      // ---- dP[q][k] = dO V^T
      f32x16 dp;
#pragma unroll
      for (int r = 0; r < 16; ++r) dp[r] = 0.f;
#pragma unroll
      for (int c = 0; c < DV / 16; ++c) {
        bf16x8_v vb = *reinterpret_cast<const bf16x8_v*>(
            v_img + sub_off(col, c * 16 + half * 8));
        dp = __builtin_amdgcn_mfma_f32_32x32x16_bf16(dofrag[c], vb, dp, 0, 0, 0);
      }

      const int kg = k0 + col;   // cols = k here
#pragma unroll
      for (int r = 0; r < 16; ++r) {
        const int qrow = (r & 3) + 8 * (r >> 2) + 4 * half;  // block-local + wid*32
        const int qg = q_start + q0 + qrow;
        const bool masked = (causal && kg > qg) || kg >= Skv ||
                            (VARLEN && kg < (int)stats[2 * WAVES * 32 + wid * 32 + qrow]);
        const float p = masked ? 0.f : __expf(s[r] * scale - stats[wid * 32 + qrow]);
        s[r] = p * (dp[r] - stats[WAVES * 32 + wid * 32 + qrow]) * scale;  // dS in place
      }

      // ---- transpose dS (cols=k -> A-frag rows=q), accumulate dQ
#pragma unroll
      for (int r = 0; r < 16; ++r) {
        const int qrow = (r & 3) + 8 * (r >> 2) + 4 * half;
        *reinterpret_cast<bf16*>(tb + tb_off(qrow, col * 2)) = f2bf(s[r]);
      }
      __builtin_amdgcn_wave_barrier();
      const unsigned k_base_a = lds_addr(k_img);
      if constexpr (!pipe_ok_dq(DQK, DV)) {
#pragma unroll
        for (int c2 = 0; c2 < 2; ++c2) {
          bf16x8_v da = *reinterpret_cast<const bf16x8_v*>(
              tb + tb_off(col, (c2 * 16 + half * 8) * 2));
#pragma unroll
          for (int t = 0; t < DQK / 32; ++t) {
            bf16x8_v ktb = tr16_frag(k_base_a, t, c2 * 2 + half, lane);
            dq_acc[t] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(da, ktb, dq_acc[t], 0, 0, 0);
          }
        }
      } else {
        bf16x8_v daf[2];
#pragma unroll
        for (int c2 = 0; c2 < 2; ++c2)
          daf[c2] = *reinterpret_cast<const bf16x8_v*>(
              tb + tb_off(col, (c2 * 16 + half * 8) * 2));
        constexpr int NT = DQK / 32;
        unsigned long long pA, pB, qA, qB;
        auto addr_f = [&](int i) {
          const int c2 = i / NT, t = i % NT;
          return k_base_a + (unsigned)((t * 2 + ((lane >> 4) & 1)) * 1152 +
                                       (8 * (c2 * 2 + half)) * 32 + (lane & 15) * 8);
        };
        tr16_issue2(addr_f(0), pA, pB);
#pragma unroll
        for (int i = 0; i < 2 * NT; ++i) {
          const bool last = (i + 1 == 2 * NT);
          if (!last) tr16_issue2(addr_f(i + 1), (i & 1) ? pA : qA, (i & 1) ? pB : qB);
          bf16x8_v ktb = tr16_take((i & 1) ? qA : pA, (i & 1) ? qB : pB, !last);
          dq_acc[i % NT] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(
              daf[i / NT], ktb, dq_acc[i % NT], 0, 0, 0);
        }
      }
      __builtin_amdgcn_wave_barrier();
    }
    __syncthreads();
  }

  // ---- epilogue: plain bf16 stores (q rows exclusive to this block)
#pragma unroll
  for (int t = 0; t < DQK / 32; ++t) {
#pragma unroll
    for (int r = 0; r < 16; ++r) {
      const int qrow = q0 + (r & 3) + 8 * (r >> 2) + 4 * half;
      if (qrow < Sq) {
        dq[q_base + (long)qrow * q_rs + t * 32 + col] = f2bf(dq_acc[t][r]);
      }
    }
  }
}

template <int DQK, int DV, int WAVES, bool VARLEN>
static void launch_dkv(const at::Tensor& dout, const at::Tensor& q, const at::Tensor& k,
                       const at::Tensor& v, const at::Tensor& lse, const at::Tensor& delta,
                       at::Tensor& dk, at::Tensor& dv, const int* doc_end, int B, int Sq,
                       int Skv, int Hq, int Hk, int q_start, float scale, bool causal,
                       hipStream_t stream) {
  const dim3 grid(Skv / (WAVES * 32), Hk, B);
  const size_t smem = sub_img_bytes<DQK>() + sub_img_bytes<DV>() + WAVES * 2048;
  hipLaunchKernelGGL((flash_bwd_dkv_kernel<DQK, DV, WAVES, VARLEN>), grid,
                     dim3(WAVES * WAVE_SIZE), smem, stream,
                     reinterpret_cast<const bf16*>(dout.data_ptr()),
                     reinterpret_cast<const bf16*>(q.data_ptr()),
                     reinterpret_cast<const bf16*>(k.data_ptr()),
                     reinterpret_cast<const bf16*>(v.data_ptr()),
                     lse.data_ptr<float>(), delta.data_ptr<float>(),
                     reinterpret_cast<bf16*>(dk.data_ptr()),
                     reinterpret_cast<bf16*>(dv.data_ptr()), doc_end,
                     B, Sq, Skv, Hq, Hk, q_start, scale, causal);
  HIP_CHECK_KERNEL();
}

template <int DQK, int DV, int WAVES, bool VARLEN>
static void launch_dq(const at::Tensor& dout, const at::Tensor& q, const at::Tensor& k,
                      const at::Tensor& v, const at::Tensor& lse, const at::Tensor& delta,
                      at::Tensor& dq, const int* doc_start, int B, int Sq, int Skv, int Hq,
                      int Hk, int q_start, float scale, bool causal, hipStream_t stream) {
  const dim3 grid(Sq / (WAVES * 32), Hq, B);
  const size_t smem = sub_img_bytes<DQK>() + sub_img_bytes<DV>() +
                      WAVES * 2048 + 3 * WAVES * 32 * sizeof(float);
  hipLaunchKernelGGL((flash_bwd_dq_kernel<DQK, DV, WAVES, VARLEN>), grid,
                     dim3(WAVES * WAVE_SIZE), smem, stream,
                     reinterpret_cast<const bf16*>(dout.data_ptr()),
                     reinterpret_cast<const bf16*>(q.data_ptr()),
                     reinterpret_cast<const bf16*>(k.data_ptr()),
                     reinterpret_cast<const bf16*>(v.data_ptr()),
                     lse.data_ptr<float>(), delta.data_ptr<float>(),
                     reinterpret_cast<bf16*>(dq.data_ptr()), doc_start,
                     B, Sq, Skv, Hq, Hk, q_start, scale, causal);
  HIP_CHECK_KERNEL();
}

std::tuple<at::Tensor, at::Tensor, at::Tensor> flash_attn_bwd(
    const at::Tensor& dout, const at::Tensor& q, const at::Tensor& k, const at::Tensor& v,
    const at::Tensor& o, const at::Tensor& lse, double scale, bool causal, int64_t q_start,
    const std::optional<at::Tensor>& doc_start, const std::optional<at::Tensor>& doc_end) {
  const int B = q.size(0), Sq = q.size(1), Hq = q.size(2), Dqk = q.size(3);
  const int Skv = k.size(1), Hk = k.size(2), Dv = v.size(3);
  TORCH_CHECK(Sq % 128 == 0 && Skv % 128 == 0,
              "flash_attn_bwd: Sq%128==0, Skv%128==0 required");
  const bool varlen = doc_start.has_value();
  TORCH_CHECK(varlen == doc_end.has_value(), "doc_start and doc_end go together");
  const int* ds_ptr = varlen ? doc_start->data_ptr<int>() : nullptr;
  const int* de_ptr = varlen ? doc_end->data_ptr<int>() : nullptr;
  auto stream = c10::hip::getCurrentHIPStream().stream();

  auto delta = at::empty({B, Hq, Sq}, q.options().dtype(at::kFloat));
  {
    const long rows = (long)B * Sq * Hq;
    const int block = 256;
    const long grid = (rows * WAVE_SIZE + block - 1) / block;
    hipLaunchKernelGGL(fa_delta_kernel, dim3((unsigned)grid), dim3(block), 0, stream,
                       reinterpret_cast<const bf16*>(dout.data_ptr()),
                       reinterpret_cast<const bf16*>(o.data_ptr()),
                       delta.data_ptr<float>(), Sq, Hq, Dv, rows);
    HIP_CHECK_KERNEL();
  }

  auto dq = at::empty_like(q);
  auto dk = at::empty_like(k);
  auto dv = at::empty_like(v);

  bool done = false;
  // kv-parallel dKV: 8-wave only where two waves/SIMD fit (occ_dkv == 2)
#define FA_BWD_CASE(A, C)                                                                \
  if (!done && Dqk == A && Dv == C) {                                                    \
    done = true;                                                                         \
    if (varlen) {                                                                        \
      launch_dkv<A, C, 4, true>(dout, q, k, v, lse, delta, dk, dv, de_ptr, B, Sq, Skv,   \
                                Hq, Hk, (int)q_start, (float)scale, causal, stream);     \
      launch_dq<A, C, 4, true>(dout, q, k, v, lse, delta, dq, ds_ptr, B, Sq, Skv, Hq,    \
                               Hk, (int)q_start, (float)scale, causal, stream);          \
    } else {                                                                             \
      if (occ_dkv(A, C) == 2 && Skv % 256 == 0) {                                        \
        launch_dkv<A, C, (occ_dkv(A, C) == 2 ? 8 : 4), false>(                           \
            dout, q, k, v, lse, delta, dk, dv, nullptr, B, Sq, Skv, Hq, Hk,              \
            (int)q_start, (float)scale, causal, stream);                                 \
      } else {                                                                           \
        launch_dkv<A, C, 4, false>(dout, q, k, v, lse, delta, dk, dv, nullptr, B, Sq,    \
                                   Skv, Hq, Hk, (int)q_start, (float)scale, causal,      \
                                   stream);                                              \
      }                                                                                  \
      if (occ_dq(A, C) == 2 && Sq % 256 == 0) {                                          \
        launch_dq<A, C, (occ_dq(A, C) == 2 ? 8 : 4), false>(                             \
            dout, q, k, v, lse, delta, dq, nullptr, B, Sq, Skv, Hq, Hk, (int)q_start,    \
            (float)scale, causal, stream);                                               \
      } else {                                                                           \
        launch_dq<A, C, 4, false>(dout, q, k, v, lse, delta, dq, nullptr, B, Sq, Skv,    \
                                  Hq, Hk, (int)q_start, (float)scale, causal, stream);   \
      }                                                                                  \
    }                                                                                    \
  }
  FA_BWD_CASE(64, 64)
  FA_BWD_CASE(96, 96)
  FA_BWD_CASE(128, 128)
  FA_BWD_CASE(192, 128)
  FA_BWD_CASE(192, 192)
  FA_BWD_CASE(256, 256)
#undef FA_BWD_CASE
  TORCH_CHECK(done, "flash_attn_bwd: unsupported head dims (Dqk=", Dqk, ", Dv=", Dv, ")");
  return {dq, dk, dv};
}

// ---- MFMA layout self-test: d[32,32] = a[32,16] @ b[16,32] via one mfma.
__global__ void mfma_probe_kernel(const bf16* a, const bf16* b, float* d) {
  const int lane = threadIdx.x & 63;
  const int half = lane >> 5;
  bf16x8_v af, bf_;
#pragma unroll
  for (int j = 0; j < 8; ++j) {
    af[j] = (__bf16)a[(lane & 31) * 16 + half * 8 + j];   // A[i=l&31][k=8*half+j]
    bf_[j] = (__bf16)b[(half * 8 + j) * 32 + (lane & 31)];  // B[k=8*half+j][j=l&31]
  }
  f32x16 acc;
#pragma unroll
  for (int r = 0; r < 16; ++r) acc[r] = 0.f;
  acc = __builtin_amdgcn_mfma_f32_32x32x16_bf16(af, bf_, acc, 0, 0, 0);
#pragma unroll
  for (int r = 0; r < 16; ++r) {
    const int row = (r & 3) + 8 * (r >> 2) + 4 * half;
    d[row * 32 + (lane & 31)] = acc[r];
  }
}

// ---- ds_read_b64_tr_b16 layout probe: fill LDS with a linear pattern and
// dump what each lane receives for reads at stride-8B lane addresses.
// Guide T10: the gather is hardware-defined; verify on silicon before
// building kernels on it (cdna_hip_programming.md §5.4 rule 27).
__global__ void tr16_probe_kernel(const bf16* __restrict__ in, float* __restrict__ out,
                                  int n) {
  __shared__ __attribute__((aligned(16))) bf16 lds[2048];
  const int l = threadIdx.x & 63;
  for (int i = threadIdx.x; i < n; i += 64) lds[i] = in[i];
  __syncthreads();
  // two reads cover 1024 B: lanes at 8-B stride (address = LDS base + offset)
  const unsigned base = (unsigned)(unsigned long long)(uintptr_t)(&lds[0]);
  for (int rd = 0; rd < 2; ++rd) {
    unsigned off = base + (unsigned)(l * 8 + rd * 512);
    unsigned long long v;
    asm volatile("ds_read_b64_tr_b16 %0, %1\n\ts_waitcnt lgkmcnt(0)"
                 : "=v"(v) : "v"(off));
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      unsigned short u = (unsigned short)(v >> (16 * j));
      out[(rd * 64 + l) * 4 + j] = bf2f(__builtin_bit_cast(bf16, u));
    }
  }
}

at::Tensor tr16_probe(const at::Tensor& pattern) {
  TORCH_CHECK(pattern.is_cuda() && pattern.scalar_type() == at::kBFloat16 &&
              pattern.numel() <= 2048, "tr16_probe: bf16, <=2048 elems");
  auto out = at::empty({2, 64, 4}, pattern.options().dtype(at::kFloat));
  auto stream = c10::hip::getCurrentHIPStream();
  hipLaunchKernelGGL(tr16_probe_kernel, dim3(1), dim3(64), 0, stream.stream(),
                     reinterpret_cast<const bf16*>(pattern.data_ptr()),
                     out.data_ptr<float>(), (int)pattern.numel());
  HIP_CHECK_KERNEL();
  return out;
}

at::Tensor mfma_probe(const at::Tensor& a, const at::Tensor& b) {
  TORCH_CHECK(a.is_cuda() && a.sizes() == at::IntArrayRef({32, 16}), "a must be [32,16]");
  TORCH_CHECK(b.sizes() == at::IntArrayRef({16, 32}), "b must be [16,32]");
  auto d = at::empty({32, 32}, a.options().dtype(at::kFloat));
  auto stream = c10::hip::getCurrentHIPStream();
  hipLaunchKernelGGL(mfma_probe_kernel, dim3(1), dim3(64), 0, stream.stream(),
                     reinterpret_cast<const bf16*>(a.data_ptr()),
                     reinterpret_cast<const bf16*>(b.data_ptr()), d.data_ptr<float>());
  HIP_CHECK_KERNEL();
  return d;
}

}  // namespace amd_ops
