// Shared device helpers of the flash-attention forward and backward kernels:
// LDS tile layouts, hardware-transpose fragment reads and occupancy bounds.
#pragma once

#include "common.h"

namespace amd_ops {

typedef __bf16 bf16x8_v __attribute__((ext_vector_type(8)));
typedef float f32x16 __attribute__((ext_vector_type(16)));

#define QBLK 32
#define KVBLK 32

// LDS row-major tile offsets: row stride padded to a multiple of 256 B so
// every row starts at bank 0; ((row&15)<<4) rotates the 16-B slot per row ->
// a 16-lane ds_read_b128 group (16 distinct rows, same in-row byte) hits 16
// distinct slots (guide Guideline 4). PMC evidence: profiles/r1_pmc_*.csv.
__host__ __device__ constexpr int pad256(int bytes) { return ((bytes + 255) / 256) * 256; }

__device__ __forceinline__ int row_lds_off(int row, int byte_in_row, int stride_b) {
  return row * stride_b + (byte_in_row ^ ((row & 15) << 4));
}
// V^T-style tile: [D][KVBLK] bf16, 64 B rows (16 words). Rows d and d+4 share
// the same 16-word bank window; ((d>>2)^(d>>3))&3 rotation separates the four
// colliding rows for reads AND spreads the transpose-store writers.
__device__ __forceinline__ int vt_lds_off(int d, int byte_in_row) {
  return d * 64 + (byte_in_row ^ ((((d >> 2) ^ (d >> 3)) & 3) << 4));
}

// ---- gfx950 hardware-transpose (ds_read_b64_tr_b16) tile images -----------
// Probe-verified semantics (benchmarks/tr16_map.py, guide T10): each 16-lane
// group reads a contiguous 128-B region as a [4 row][16 col] bf16 block and
// lane g receives COLUMN g (one value per row). A [32 k][D] tile stored as
// [D/16 subtiles][32 k rows][16 d cols] therefore serves BOTH access
// patterns with no scalar transposes:
//   * row-chunk b128 reads (A-style: lane = k row, 8 consecutive d)
//   * transposed B-fragments via two tr16 reads (lane = d col, 8 k rows)
// Subtile stride 1152 B (not 1024): adjacent subtiles land 32 banks apart,
// so the two 16-lane halves of a wave (reading subtiles 2t and 2t+1) never
// share a bank window (b64 conflict groups are 32 lanes).
__device__ __forceinline__ int sub_off(int k, int d) {
  return (d >> 4) * 1152 + k * 32 + (d & 15) * 2;
}
template <int D>
__host__ __device__ constexpr int sub_img_bytes() { return (D / 16) * 1152; }

__device__ __forceinline__ unsigned lds_addr(const void* p) {
  return (unsigned)(unsigned long long)(uintptr_t)p;
}

// B-fragment for mfma_32x32x16: element j = T[k = 8*khalf + j][col =
// tile32*32 + (lane&31)] from a subtiled image, via two hardware-transpose
// reads (k rows 8h..8h+3 and 8h+4..8h+7). The trailing s_waitcnt rides in
// the second asm so the consuming mfma (which needs both halves) cannot be
// scheduled before the data lands.
// pipelined form: issue one fragment's two reads; wait-and-take later with
// a counted lgkmcnt (the "+v" operands order the consuming MFMAs after it)
__device__ __forceinline__ void tr16_issue2(unsigned addr, unsigned long long& r0,
                                            unsigned long long& r1) {
  asm volatile("ds_read_b64_tr_b16 %0, %2\n\tds_read_b64_tr_b16 %1, %2 offset:128"
               : "=v"(r0), "=v"(r1) : "v"(addr));
}
__device__ __forceinline__ bf16x8_v tr16_take(unsigned long long& r0,
                                              unsigned long long& r1, bool newer2) {
  if (newer2) {
    asm volatile("s_waitcnt lgkmcnt(2)" : "+v"(r0), "+v"(r1));
  } else {
    asm volatile("s_waitcnt lgkmcnt(0)" : "+v"(r0), "+v"(r1));
  }
  ulonglong2 u{r0, r1};
  return __builtin_bit_cast(bf16x8_v, u);
}

__device__ __forceinline__ bf16x8_v tr16_frag(unsigned img_base, int tile32,
                                              int khalf, int lane) {
  const unsigned a0 = img_base + (unsigned)((tile32 * 2 + ((lane >> 4) & 1)) * 1152 +
                                            (8 * khalf) * 32 + (lane & 15) * 8);
  unsigned long long v0, v1;
  // single asm block: outputs are fully landed when it retires, so the
  // register allocator can never spill an in-flight read (a real silent-
  // corruption hazard caught at (192,192) under register pressure)
  asm volatile("ds_read_b64_tr_b16 %0, %2\n\t"
               "ds_read_b64_tr_b16 %1, %2 offset:128\n\t"
               "s_waitcnt lgkmcnt(0)"
               : "=v"(v0), "=v"(v1) : "v"(a0));
  ulonglong2 u{v0, v1};
  return __builtin_bit_cast(bf16x8_v, u);
}

// Pipelining across other code is only safe when nothing spills: gate the
// pipelined tr16 paths to instantiations comfortably inside the register
// budget; the big-D variants take the self-contained tr16_frag instead.
__host__ __device__ constexpr bool pipe_ok_dkv(int DQK, int DV) {
  return 3 * (DQK + DV) / 4 + 16 <= 208;
}
__host__ __device__ constexpr bool pipe_ok_dq(int DQK, int DV) {
  return DQK / 4 + DV / 4 + DQK / 2 + 48 <= 208;
}
// per-wave transpose buffer: [32][64 B]
__device__ __forceinline__ int tb_off(int row, int byte_in_row) {
  return row * 64 + (byte_in_row ^ ((((row >> 2) ^ (row >> 3)) & 3) << 4));
}

// Min-waves-per-SIMD for the backward kernels: the f32 accumulators scale
// with head dim; past ~240 VGPR/lane two waves/SIMD would spill heavily, so
// the big-D instantiations run one wave/SIMD (4-wave workgroups).
__host__ __device__ constexpr int occ_dkv(int DQK, int DV) {
  return (3 * (DQK + DV) / 4 + 16) <= 240 ? 2 : 1;
}
__host__ __device__ constexpr int occ_dq(int DQK, int DV) {
  return (DQK / 4 + DV / 4 + DQK / 2 + 48) <= 240 ? 2 : 1;
}

}  // namespace amd_ops
