// Linear recurrences with a matrix state per head, over packed prompts and one
// token at a time (inference). The state S [K, P] is f32 throughout.
//
//   state space   S_t = a_t S_(t-1) + dt_t B_t x_t^T,   y_t = S_t^T C_t + D x_t
//                 one decay a_t = exp(-exp(A_log) dt_t) per head
//   wkv           o_t = (S_(t-1) + diag(u) k_t v_t^T)^T r_t,
//                 S_t = diag(w_t) S_(t-1) + k_t v_t^T, a decay per key channel
//
//   causal_conv_silu    short convolution per channel, with its cached inputs
//   token_shift         h + (h' - h) * mu for several mu, h' the token before
//   decay_cumsum / step_cumsum   log decays summed within blocks of 16 tokens
//   ssd_prompt / wkv_prompt   blocks of 16 tokens on the f32 matrix cores
//   ssd_decode / wkv_decode   one token per sequence
//   gated_group_norm    rms norm in equal groups, gated before or after
//
// The prompt kernels hold S in the accumulators of 16x16 MFMAs with f32 operands
// (or with bf16 ones where that is exact): a wave owns 16 columns of one head and
// walks its sequence. A lane (g, c) of S has
// keys 4g..4g+3 of a tile, which is an MFMA operand once the summed index is
// permuted in both operands alike; so S, the values and the 16x16 matrix within
// a block are all used where they are, and only queries and keys pass through
// LDS. Every exponent taken is of a non-positive sum, however strong the decay.

#include <torch/library.h>
#include <ATen/ATen.h>
#include <c10/hip/HIPStream.h>

#include "elem.h"
#include "ops_api.h"

namespace amd_ops {

typedef float scan_f32x4 __attribute__((ext_vector_type(4)));
typedef short scan_s16x4 __attribute__((ext_vector_type(4)));
typedef __bf16 scan_bf16x8 __attribute__((ext_vector_type(8)));

namespace {

constexpr int TB = 16;                 // tokens per block
// A log decay below this is a factor of 0 in f32; the bound keeps sums of log
// decays (of which differences are taken) accurate.
constexpr float MIN_LOG = -90.f;

__device__ __forceinline__ scan_f32x4 mfma4(float a, float b, scan_f32x4 c) {
  return __builtin_amdgcn_mfma_f32_16x16x4f32(a, b, c, 0, 0, 0);
}

// ---------------------------------------------------------------------------
// short convolution and token shift
// ---------------------------------------------------------------------------
constexpr int CONV_TOKENS = 16;        // per workgroup: taps and inputs stay in registers

// Prompts. TAPS 0: any number of taps, weights and inputs from memory.
template <typename T, int V, int TAPS>
__global__ __launch_bounds__(256) void conv_prompt_kernel(
    const T* __restrict__ in, long ld, const T* __restrict__ w, const T* __restrict__ bias,
    const int* __restrict__ pos, const int* __restrict__ slot, const int* __restrict__ seq_end,
    T* __restrict__ state, int n_slots, T* __restrict__ out, int n_tok, int C, int taps_) {
  const int taps = TAPS ? TAPS : taps_;
  const int c = (blockIdx.y * 256 + threadIdx.x) * V;
  if (c >= C) return;
  const int t0 = blockIdx.x * CONV_TOKENS, t1 = min(n_tok, t0 + CONV_TOKENS);
  float b[V];
  load_vec<T, V>(bias + c, b);
  auto finish = [&](int t, float (&acc)[V], const float (&own)[V]) {
    if (state && taps > 1 && t + taps - 1 >= seq_end[t]) {
      const int sl = slot[t];
      if (sl >= 0 && sl < n_slots)
        store_vec<T, V>(state + ((long)sl * (taps - 1) + pos[t] % (taps - 1)) * C + c, own);
    }
#pragma unroll
    for (int e = 0; e < V; ++e) acc[e] = silu_f(acc[e]);
    store_vec<T, V>(out + (long)t * C + c, acc);
  };
  if constexpr (TAPS > 0) {
    float wr[TAPS][V], x[TAPS][V];                 // x[j]: the input of tap j
#pragma unroll
    for (int j = 0; j < TAPS; ++j)
#pragma unroll
      for (int e = 0; e < V; ++e) wr[j][e] = to_f32(w[(long)(c + e) * TAPS + j]);
#pragma unroll
    for (int j = 0; j + 1 < TAPS; ++j)             // before the tile: j = TAPS - 1 is t0
      load_vec<T, V>(in + (long)max(t0 - (TAPS - 1 - j), 0) * ld + c, x[j]);
#pragma unroll 4
    for (int t = t0; t < t1; ++t) {
      load_vec<T, V>(in + t * ld + c, x[TAPS - 1]);
      const int p = pos[t];
      float acc[V];
#pragma unroll
      for (int e = 0; e < V; ++e) acc[e] = b[e];
#pragma unroll
      for (int j = 0; j < TAPS; ++j)
#pragma unroll
        for (int e = 0; e < V; ++e)
          acc[e] = fmaf(wr[j][e], p >= TAPS - 1 - j ? x[j][e] : 0.f, acc[e]);
      finish(t, acc, x[TAPS - 1]);
#pragma unroll
      for (int j = 0; j + 1 < TAPS; ++j)
#pragma unroll
        for (int e = 0; e < V; ++e) x[j][e] = x[j + 1][e];
    }
  } else {
    for (int t = t0; t < t1; ++t) {
      float acc[V], x[V];
#pragma unroll
      for (int e = 0; e < V; ++e) acc[e] = b[e];
      for (int j = max(0, taps - 1 - pos[t]); j < taps; ++j) {
        load_vec<T, V>(in + (t - (taps - 1 - j)) * ld + c, x);
#pragma unroll
        for (int e = 0; e < V; ++e)
          acc[e] = fmaf(to_f32(w[(long)(c + e) * taps + j]), x[e], acc[e]);
      }
      finish(t, acc, x);                           // x: the last tap's, the token's own
    }
  }
}

// One token per sequence, the earlier inputs from the state; V columns a thread.
template <typename T, int V>
__global__ __launch_bounds__(256) void conv_decode_kernel(
    const T* __restrict__ in, long ld, const T* __restrict__ w, const T* __restrict__ bias,
    const int* __restrict__ pos, const int* __restrict__ slot, T* __restrict__ state, int n_slots,
    T* __restrict__ out, int C, int taps) {
  const long t = blockIdx.x;
  const int c = (blockIdx.y * 256 + threadIdx.x) * V, sl = slot[t], p = pos[t];
  if (c >= C || sl < 0 || sl >= n_slots || p < 0) return;
  T* st = state + (long)sl * (taps - 1) * C + c;
  float acc[V], own[V];
  load_vec<T, V>(bias + c, acc);
  load_vec<T, V>(in + t * ld + c, own);
#pragma unroll 4
  for (int j = max(0, taps - 1 - p); j < taps - 1; ++j) {
    float x[V];
    load_vec<T, V>(st + (long)((p - (taps - 1 - j)) % (taps - 1)) * C, x);
#pragma unroll
    for (int e = 0; e < V; ++e) acc[e] = fmaf(to_f32(w[(long)(c + e) * taps + j]), x[e], acc[e]);
  }
#pragma unroll
  for (int e = 0; e < V; ++e)
    acc[e] = silu_f(fmaf(to_f32(w[(long)(c + e) * taps + taps - 1]), own[e], acc[e]));
  if (taps > 1) store_vec<T, V>(st + (long)(p % (taps - 1)) * C, own);
  store_vec<T, V>(out + t * C + c, acc);
}

template <typename T, int V>
__global__ __launch_bounds__(256) void token_shift_kernel(
    const T* __restrict__ h, const T* __restrict__ mu, int n_mix, const int* __restrict__ pos,
    const int* __restrict__ slot, const int* __restrict__ seq_end, T* __restrict__ state,
    int n_slots, T* __restrict__ out, int W) {
  const long t = blockIdx.x, n_tok = gridDim.x;
  const bool decode = seq_end == nullptr;
  const int sl = state ? slot[t] : -1;
  T* st = sl >= 0 && sl < n_slots ? state + (long)sl * W : nullptr;
  const int i = (blockIdx.y * blockDim.x + threadIdx.x) * V;
  if (i < W) {
    float a[V], d[V];
    load_vec<T, V>(h + t * W + i, a);
#pragma unroll
    for (int e = 0; e < V; ++e) d[e] = 0.f;
    if (pos[t] > 0) {
      if (!decode) load_vec<T, V>(h + (t - 1) * W + i, d);
      else if (st) load_vec<T, V>(st + i, d);
    }
#pragma unroll
    for (int e = 0; e < V; ++e) d[e] -= a[e];
    if (st && (decode || t + 1 == seq_end[t])) store_vec<T, V>(st + i, a);
    for (int s = 0; s < n_mix; ++s) {
      float m[V];
      load_vec<T, V>(mu + (long)s * W + i, m);
#pragma unroll
      for (int e = 0; e < V; ++e) m[e] = fmaf(d[e], m[e], a[e]);
      store_vec<T, V>(out + (s * n_tok + t) * W + i, m);
    }
  }
}

// low [T, C] -> sums of the log decays -exp(low + w0) from each block's start,
// in place; blocks of TB tokens counted from every sequence's first.
template <typename T>
__global__ __launch_bounds__(256) void decay_cumsum_kernel(float* __restrict__ low,
                                                           const T* __restrict__ w0,
                                                           const int* __restrict__ cu, int C) {
  const int c = blockIdx.z * 256 + threadIdx.x;
  const int t0 = cu[blockIdx.y] + blockIdx.x * TB, t1 = min(t0 + TB, cu[blockIdx.y + 1]);
  if (c >= C) return;
  const float b = to_f32(w0[c]);
  float s = 0.f;
  for (int t = t0; t < t1; ++t) {
    s += fmaxf(-expf(low[(long)t * C + c] + b), MIN_LOG);
    low[(long)t * C + c] = s;
  }
}

// dt [T, H] -> steps softplus(dt + bias) and sums of the log decays
// -exp(A_log) * step from each block's start, both [H, T].
template <typename T>
__global__ __launch_bounds__(256) void step_cumsum_kernel(
    const T* __restrict__ dt, long dt_ld, const T* __restrict__ bias, const T* __restrict__ a_log,
    const int* __restrict__ cu, int H, int n_tok, float* __restrict__ steps,
    float* __restrict__ sums) {
  const int h = blockIdx.z * 64 + (threadIdx.x & 63);
  const int t0 = cu[blockIdx.y] + (blockIdx.x * 4 + (threadIdx.x >> 6)) * TB;
  const int t1 = min(t0 + TB, cu[blockIdx.y + 1]);
  if (h >= H) return;
  const float b = to_f32(bias[h]), rate = -expf(to_f32(a_log[h]));
  float s = 0.f;
  for (int t = t0; t < t1; ++t) {
    const float step = softplus_f(to_f32(dt[t * dt_ld + h]) + b);
    s += fmaxf(rate * step, MIN_LOG);
    steps[(long)h * n_tok + t] = step;
    sums[(long)h * n_tok + t] = s;
  }
}

// ---------------------------------------------------------------------------
// prompts: grid (column groups of 64, heads, sequences x segments), one wave per
// 16 columns. Few heads and long sequences leave most of the chip idle, so a
// sequence may be cut into segments: a first pass (STATES) makes every segment's
// state from zero and its decay, scan_link_kernel turns these into the states
// that the segments begin with, and the main pass runs all segments at once.
// ---------------------------------------------------------------------------
// KT consecutive floats of LDS, 16 bytes at a time where there are as many
template <int N>
__device__ __forceinline__ void put(float* p, const float (&x)[N]) {
  if constexpr (N >= 4) {
#pragma unroll
    for (int j = 0; j < N; j += 4)
      *reinterpret_cast<float4*>(p + j) = float4{x[j], x[j + 1], x[j + 2], x[j + 3]};
  } else {
#pragma unroll
    for (int j = 0; j < N; ++j) p[j] = x[j];
  }
}
template <int N>
__device__ __forceinline__ void get(const float* p, float (&x)[N]) {
  if constexpr (N >= 4) {
#pragma unroll
    for (int j = 0; j < N; j += 4) {
      const float4 t = *reinterpret_cast<const float4*>(p + j);
      x[j] = t.x;
      x[j + 1] = t.y;
      x[j + 2] = t.z;
      x[j + 3] = t.w;
    }
  } else {
#pragma unroll
    for (int j = 0; j < N; ++j) x[j] = p[j];
  }
}

template <typename T>
struct ScanArgs {
  const T *q, *k, *v;                  // row t, head h: base + t * ld + ...
  long q_ld, k_ld, v_ld;
  int q_hs, k_hs, per_group;           // head strides; heads per q/k group
  const float* cum;                    // wkv: [T, H * K]
  const T* u;                          // wkv: [H, K]
  const T* d_skip;                     // state space: [H]
  const float *steps, *sums;           // state space: [H, n_tok]
  int n_tok;
  const int *cu, *slot;
  float* state;                        // [slots, H, K, P] or null
  int segs, seg_len;                   // segments per sequence, in whole blocks
  float* seg_state;                    // [seqs, segs, H, K, P] if segs > 1
  float* seg_decay;                    // [seqs, segs, H, K] (wkv) or [seqs, segs, H]
  int n_slots, H, K, P;
  bool vec;                            // K = KT * 16 and rows aligned to 16 bytes
  T* out;                              // [T, H * P]
};

// What a workgroup works on, and the state in MFMA accumulators: lane (g, c) of
// tile kt has keys 16 kt + 4 g + r of column c.
template <typename T, int KT>
struct ScanWork {
  static constexpr int KP = KT * 16;
  const ScanArgs<T>& a;
  int tid, wid, lo, lg, h, seg, s0, len, col, colc;
  int own_i, own_ch;                   // staging: KT neighbouring channels of one token
  bool live, last;
  long sh;                             // index of (sequence, segment, head)
  scan_f32x4 S[KT];

  __device__ __forceinline__ explicit ScanWork(const ScanArgs<T>& args) : a(args) {
    tid = threadIdx.x;
    wid = tid >> 6;
    lo = tid & 15;
    lg = (tid & 63) >> 4;
    own_i = tid >> 4;
    own_ch = (tid & 15) * KT;
    h = blockIdx.y;
    seg = blockIdx.z % a.segs;
    const int seq = blockIdx.z / a.segs;
    const int left = a.cu[seq + 1] - a.cu[seq] - seg * a.seg_len;
    s0 = a.cu[seq] + seg * a.seg_len;
    len = min(left, a.seg_len);
    last = left <= a.seg_len;
    col = (blockIdx.x * 4 + wid) * 16 + lo;
    live = col < a.P;
    colc = live ? col : a.P - 1;
    sh = (long)blockIdx.z * a.H + h;
  }
  __device__ __forceinline__ void begin(bool from_zero) {
#pragma unroll
    for (int i = 0; i < KT; ++i) S[i] = scan_f32x4{0.f, 0.f, 0.f, 0.f};
    if (from_zero || seg == 0) return;
    const float* st = a.seg_state + sh * a.K * a.P + colc;
#pragma unroll
    for (int kt = 0; kt < KT; ++kt)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int key = kt * 16 + lg * 4 + r;
        const float x = st[(long)min(key, a.K - 1) * a.P];
        S[kt][r] = key < a.K ? x : 0.f;
      }
  }
  __device__ __forceinline__ void store(float* st) const {
    if (!live) return;
#pragma unroll
    for (int kt = 0; kt < KT; ++kt)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int key = kt * 16 + lg * 4 + r;
        if (key < a.K) st[(long)key * a.P + col] = S[kt][r];
      }
  }
  __device__ __forceinline__ void store_segment() const { store(a.seg_state + sh * a.K * a.P); }
  __device__ __forceinline__ void store_final() const {
    if (a.state == nullptr || !last) return;
    const int sl = a.slot[s0];
    if (sl >= 0 && sl < a.n_slots) store(a.state + ((long)sl * a.H + h) * a.K * a.P);
  }
  __device__ __forceinline__ void store_out(int c0, int nt, const scan_f32x4& o) const {
#pragma unroll
    for (int r = 0; r < 4; ++r)
      if (live && lg * 4 + r < nt)
        a.out[(long)(s0 + c0 + lg * 4 + r) * a.H * a.P + (long)h * a.P + col] = from_f32<T>(o[r]);
  }
  // This thread's channels of a token's row, as they are. Places are clamped
  // rather than skipped: all loads of a block are then in flight at once.
  template <typename E>
  __device__ __forceinline__ void fetch_row(const E* row, E (&to)[KT]) const {
    if (a.vec) {
      constexpr int N = KT * sizeof(E) > 16 ? 16 / sizeof(E) : KT;   // elements per load
#pragma unroll
      for (int j = 0; j < KT; j += N) {
        const ElemPack<E, N> t = *reinterpret_cast<const ElemPack<E, N>*>(row + own_ch + j);
#pragma unroll
        for (int e = 0; e < N; ++e) to[j + e] = t.v[e];
      }
    } else {
#pragma unroll
      for (int j = 0; j < KT; ++j) to[j] = row[min(own_ch + j, a.K - 1)];
    }
  }
  __device__ __forceinline__ void fetch_values(int c0, int nt, T (&to)[4]) const {
    const T* vb = a.v + (long)h * a.P + colc;
#pragma unroll
    for (int r = 0; r < 4; ++r) to[r] = vb[(long)(s0 + c0 + min(lg * 4 + r, nt - 1)) * a.v_ld];
  }
  __device__ __forceinline__ bool own_in(int j, int nt) const {
    return own_i < nt && own_ch + j < a.K;
  }
};

// STATES: the segment's state from zero and its decay, without outputs.
template <typename T, int KT, bool STATES>
__global__ __launch_bounds__(256) void wkv_prompt_kernel(ScanArgs<T> a) {
  constexpr int KP = KT * 16, LD = KP + 4;
  extern __shared__ __attribute__((aligned(16))) float lds[];
  float* qs = lds;                     // [TB][LD]
  float* ks = qs + TB * LD;
  float* cm = ks + TB * LD;            // sums of log decays
  float* qd = cm + TB * LD;            // r times the decay since the block's start
  float* kd = qd + TB * LD;            // k times the decay up to the block's end
  float* es = kd + TB * LD;            // [KP] decay over the block
  float* us = es + KP;                 // [KP]
  float* am = us + KP;                 // [TB][TB + 4] weights within the block

  ScanWork<T, KT> wk(a);
  if (wk.len <= 0 || (STATES && wk.last)) return;  // uniform over the block
  const int tid = wk.tid, lo = wk.lo, lg = wk.lg;
  const T* qb = a.q + (long)wk.h * a.q_hs;
  const T* kb = a.k + (long)wk.h * a.k_hs;
  const float* cb = a.cum + (long)wk.h * a.K;
  if constexpr (!STATES) {
    for (int i = tid; i < KP; i += 256) us[i] = i < a.K ? to_f32(a.u[(long)wk.h * a.K + i]) : 0.f;
    for (int i = tid; i < TB * (TB + 4); i += 256) am[i] = 0.f;
  }
  wk.begin(STATES);
  float log_decay = 0.f;                           // STATES: of channel tid

  T qr[KT], kr[KT], vr[4];                         // the next block's operands
  float cr[KT];
  auto fetch = [&](int c0) {
    const int nt = min(TB, wk.len - c0);
    const long t = wk.s0 + c0 + min(wk.own_i, nt - 1);
    if constexpr (!STATES) wk.fetch_row(qb + t * a.q_ld, qr);
    wk.fetch_row(kb + t * a.k_ld, kr);
    // past the end the sum of log decays stays where it is
    wk.fetch_row(cb + t * ((long)a.H * a.K), cr);
    wk.fetch_values(c0, nt, vr);
  };
  fetch(0);
  for (int c0 = 0; c0 < wk.len; c0 += TB) {
    const int nt = min(TB, wk.len - c0), at = wk.own_i * LD + wk.own_ch;
    __syncthreads();                               // the last block has been read
    float x[KT], y[KT], c[KT];
#pragma unroll
    for (int j = 0; j < KT; ++j) {
      x[j] = !STATES && wk.own_in(j, nt) ? to_f32(qr[j]) : 0.f;
      y[j] = wk.own_in(j, nt) ? to_f32(kr[j]) : 0.f;
      c[j] = wk.own_ch + j < a.K ? cr[j] : 0.f;
    }
    if constexpr (!STATES) put(qs + at, x);
    put(ks + at, y);
    put(cm + at, c);
    float v[4];
#pragma unroll
    for (int r = 0; r < 4; ++r) v[r] = lg * 4 + r < nt ? to_f32(vr[r]) : 0.f;
    __syncthreads();
    if (c0 + TB < wk.len) fetch(c0 + TB);

    float end[KT];
    get(cm + (TB - 1) * LD + wk.own_ch, end);
    if constexpr (!STATES) {
      float before[KT];
      get(cm + max(at - LD, wk.own_ch), before);
#pragma unroll
      for (int j = 0; j < KT; ++j) x[j] *= wk.own_i > 0 ? __expf(before[j]) : 1.f;
      put(qd + at, x);
    } else if (tid < KP) {
      log_decay += cm[(TB - 1) * LD + tid];
    }
#pragma unroll
    for (int j = 0; j < KT; ++j) {
      y[j] *= __expf(end[j] - c[j]);
      end[j] = __expf(end[j]);
    }
    put(kd + at, y);
    if (wk.own_i == 0) put(es + wk.own_ch, end);

    if constexpr (!STATES) {
      // Weights of earlier tokens j for i within the block. Wave `wid` takes the
      // pairs that part at half size hs: j in the lower, i in the upper half of
      // a group of 2 hs, both measured against the group's middle.
      const int hs = 8 >> wk.wid;
      const int mid = lo / (2 * hs) * (2 * hs) + hs - 1;
      const bool upper = (lo & hs) != 0;
      scan_f32x4 g = scan_f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int kt = 0; kt < KT; ++kt) {
        const int ch = kt * 16 + lg * 4;
        const float4 p = *reinterpret_cast<const float4*>((upper ? qs : ks) + lo * LD + ch);
        const float4 cmid = *reinterpret_cast<const float4*>(cm + mid * LD + ch);
        const float4 cown =
            *reinterpret_cast<const float4*>(cm + (upper ? lo - 1 : lo) * LD + ch);
        const float ps[4] = {p.x, p.y, p.z, p.w};
        const float ds[4] = {cown.x - cmid.x, cown.y - cmid.y, cown.z - cmid.z, cown.w - cmid.w};
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const float w = ps[r] * __expf(upper ? ds[r] : -ds[r]);
          g = mfma4(upper ? 0.f : w, upper ? w : 0.f, g);   // row j, column i
        }
      }
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int j = lg * 4 + r, i = lo;
        if (upper && !(j & hs) && i / (2 * hs) == j / (2 * hs)) am[i * (TB + 4) + j] = g[r];
      }
      // the token itself, with the bonus: 16 threads each
      float d = 0.f;
      for (int ch = lo; ch < KP; ch += 16)
        d = fmaf(qs[wk.own_i * LD + ch] * us[ch], ks[wk.own_i * LD + ch], d);
#pragma unroll
      for (int off = 8; off > 0; off >>= 1) d += __shfl_xor(d, off);
      if (lo == 0) am[wk.own_i * (TB + 4) + wk.own_i] = d;
    }
    __syncthreads();
    if constexpr (!STATES) {
      scan_f32x4 o = scan_f32x4{0.f, 0.f, 0.f, 0.f}, o2 = o;
#pragma unroll
      for (int kt = 0; kt < KT; ++kt) {
        const float4 p = *reinterpret_cast<const float4*>(qd + lo * LD + kt * 16 + lg * 4);
        o = mfma4(p.x, wk.S[kt][0], o);
        o2 = mfma4(p.y, wk.S[kt][1], o2);
        o = mfma4(p.z, wk.S[kt][2], o);
        o2 = mfma4(p.w, wk.S[kt][3], o2);
      }
      const float4 w = *reinterpret_cast<const float4*>(am + lo * (TB + 4) + lg * 4);
      o = mfma4(w.x, v[0], o);
      o2 = mfma4(w.y, v[1], o2);
      o = mfma4(w.z, v[2], o);
      o2 = mfma4(w.w, v[3], o2);
      o += o2;
      wk.store_out(c0, nt, o);
    }
#pragma unroll
    for (int kt = 0; kt < KT; ++kt) {
      const float4 e = *reinterpret_cast<const float4*>(es + kt * 16 + lg * 4);
      wk.S[kt][0] *= e.x;
      wk.S[kt][1] *= e.y;
      wk.S[kt][2] *= e.z;
      wk.S[kt][3] *= e.w;
    }
#pragma unroll
    for (int r = 0; r < 4; ++r)
#pragma unroll
      for (int kt = 0; kt < KT; ++kt)
        wk.S[kt] = mfma4(kd[(lg * 4 + r) * LD + kt * 16 + lo], v[r], wk.S[kt]);
  }
  if constexpr (STATES) {
    if (blockIdx.x == 0 && tid < a.K) a.seg_decay[wk.sh * a.K + tid] = __expf(log_decay);
    wk.store_segment();
  } else {
    wk.store_final();
  }
}

// Queries and keys in LDS for the state-space kernel, and the products with them.
// f32: both as [TB][KP + 4].
template <typename T, int KT>
struct SsdOperands {
  static constexpr int KP = KT * 16, LD = KP + 4;
  static constexpr size_t BYTES = 2 * TB * LD * sizeof(float);
  float *qs, *ks;
  __device__ __forceinline__ explicit SsdOperands(char* lds)
      : qs(reinterpret_cast<float*>(lds)), ks(qs + TB * LD) {}
  template <typename W>
  __device__ __forceinline__ void stage(const W& wk, const T (&q)[KT], const T (&k)[KT], int nt,
                                        bool queries) {
    float x[KT], y[KT];
#pragma unroll
    for (int j = 0; j < KT; ++j) {
      x[j] = queries && wk.own_in(j, nt) ? to_f32(q[j]) : 0.f;
      y[j] = wk.own_in(j, nt) ? to_f32(k[j]) : 0.f;
    }
    if (queries) put(qs + wk.own_i * LD + wk.own_ch, x);
    put(ks + wk.own_i * LD + wk.own_ch, y);
  }
  // row j, column i: k_j . q_i
  __device__ __forceinline__ scan_f32x4 gram(int lo, int lg) const {
    scan_f32x4 g = scan_f32x4{0.f, 0.f, 0.f, 0.f}, g2 = g;
#pragma unroll
    for (int kt = 0; kt < KT; ++kt) {
      const float4 x = *reinterpret_cast<const float4*>(qs + lo * LD + kt * 16 + lg * 4);
      const float4 y = *reinterpret_cast<const float4*>(ks + lo * LD + kt * 16 + lg * 4);
      g = mfma4(y.x, x.x, g);
      g2 = mfma4(y.y, x.y, g2);
      g = mfma4(y.z, x.z, g);
      g2 = mfma4(y.w, x.w, g2);
    }
    return g + g2;
  }
  __device__ __forceinline__ float4 query4(int lo, int ch) const {
    return *reinterpret_cast<const float4*>(qs + lo * LD + ch);
  }
  // S += k^T v, v[r] the value of token 4 lg + r
  __device__ __forceinline__ void add(scan_f32x4 (&S)[KT], const float (&v)[4], int lo,
                                      int lg) const {
#pragma unroll
    for (int r = 0; r < 4; ++r)
#pragma unroll
      for (int kt = 0; kt < KT; ++kt)
        S[kt] = mfma4(ks[(lg * 4 + r) * LD + kt * 16 + lo], v[r], S[kt]);
  }
};

// bf16: products of two bf16 operands are exact in f32, and an f32 value is the
// sum of three bf16 parts, so the bf16 matrix cores give f32 results here at a
// multiple of the f32 rate. Keys also transposed, [KP][TB + 4].
template <int KT>
struct SsdOperands<bf16, KT> {
  static constexpr int KP = KT * 16, LD = KP + 8, TD = TB + 4;
  static constexpr size_t BYTES = (2 * TB * LD + KP * TD) * sizeof(bf16);
  bf16 *qs, *ks, *kt_;
  __device__ __forceinline__ explicit SsdOperands(char* lds)
      : qs(reinterpret_cast<bf16*>(lds)), ks(qs + TB * LD), kt_(ks + TB * LD) {}
  template <typename W>
  __device__ __forceinline__ void stage(const W& wk, const bf16 (&q)[KT], const bf16 (&k)[KT],
                                        int nt, bool queries) {
    const bf16 zero = f2bf(0.f);
    ElemPack<bf16, KT> x, y;
#pragma unroll
    for (int j = 0; j < KT; ++j) {
      x.v[j] = queries && wk.own_in(j, nt) ? q[j] : zero;
      y.v[j] = wk.own_in(j, nt) ? k[j] : zero;
      kt_[(wk.own_ch + j) * TD + wk.own_i] = y.v[j];
    }
    if (!queries) return;
    *reinterpret_cast<ElemPack<bf16, KT>*>(qs + wk.own_i * LD + wk.own_ch) = x;
    *reinterpret_cast<ElemPack<bf16, KT>*>(ks + wk.own_i * LD + wk.own_ch) = y;
  }
  __device__ __forceinline__ scan_f32x4 gram(int lo, int lg) const {
    scan_f32x4 g = scan_f32x4{0.f, 0.f, 0.f, 0.f};
    if constexpr (KT == 1) {
      const scan_s16x4 y = *reinterpret_cast<const scan_s16x4*>(ks + lo * LD + lg * 4);
      const scan_s16x4 x = *reinterpret_cast<const scan_s16x4*>(qs + lo * LD + lg * 4);
      return __builtin_amdgcn_mfma_f32_16x16x16bf16_1k(y, x, g, 0, 0, 0);
    } else {
#pragma unroll
      for (int c = 0; c < KP / 32; ++c) {
        const scan_bf16x8 y = *reinterpret_cast<const scan_bf16x8*>(ks + lo * LD + c * 32 + lg * 8);
        const scan_bf16x8 x = *reinterpret_cast<const scan_bf16x8*>(qs + lo * LD + c * 32 + lg * 8);
        g = __builtin_amdgcn_mfma_f32_16x16x32_bf16(y, x, g, 0, 0, 0);
      }
      return g;
    }
  }
  __device__ __forceinline__ float4 query4(int lo, int ch) const {
    float x[4];
    load_vec<bf16, 4>(qs + lo * LD + ch, x);
    return float4{x[0], x[1], x[2], x[3]};
  }
  __device__ __forceinline__ void add(scan_f32x4 (&S)[KT], const float (&v)[4], int lo,
                                      int lg) const {
    // Both products are the same instruction: a chain through one accumulator of
    // 16x16x32 and 16x16x16 steps right after one another lost results here.
    scan_bf16x8 b;                                 // leading parts, then the middle ones
    scan_bf16x8 b3{};                              // the rest
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const __bf16 v1 = (__bf16)v[r];
      const float rest = v[r] - (float)v1;
      const __bf16 v2 = (__bf16)rest;
      b[r] = v1;
      b[4 + r] = v2;
      b3[r] = (__bf16)(rest - (float)v2);
    }
    scan_bf16x8 k8[KT];                            // the tokens' keys, twice
#pragma unroll
    for (int kt = 0; kt < KT; ++kt) {
      const scan_s16x4 k4 =
          *reinterpret_cast<const scan_s16x4*>(kt_ + (kt * 16 + lo) * TD + lg * 4);
      k8[kt] = __builtin_bit_cast(scan_bf16x8,
                                  __builtin_shufflevector(k4, k4, 0, 1, 2, 3, 4, 5, 6, 7));
    }
#pragma unroll
    for (int kt = 0; kt < KT; ++kt)
      S[kt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(k8[kt], b, S[kt], 0, 0, 0);
#pragma unroll
    for (int kt = 0; kt < KT; ++kt)
      S[kt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(k8[kt], b3, S[kt], 0, 0, 0);
  }
};

template <typename T, int KT, bool STATES>
__global__ __launch_bounds__(256) void ssd_prompt_kernel(ScanArgs<T> a) {
  extern __shared__ __attribute__((aligned(16))) float lds[];
  SsdOperands<T, KT> op(reinterpret_cast<char*>(lds));
  ScanWork<T, KT> wk(a);
  if (wk.len <= 0 || (STATES && wk.last)) return;  // uniform over the block
  const int lo = wk.lo, lg = wk.lg;
  const T* qb = a.q + (long)(wk.h / a.per_group) * a.q_hs;
  const T* kb = a.k + (long)(wk.h / a.per_group) * a.k_hs;
  const float* steps = a.steps + (long)wk.h * a.n_tok + wk.s0;
  const float* sums = a.sums + (long)wk.h * a.n_tok + wk.s0;
  const float skip = to_f32(a.d_skip[wk.h]);
  wk.begin(STATES);
  float log_decay = 0.f;                           // over the segment

  T qr[KT], kr[KT], vr[4];                         // the next block's operands
  float step_r[4], sum_r[4], own_r, total_r;
  auto fetch = [&](int c0) {
    const int nt = min(TB, wk.len - c0);
    const long t = wk.s0 + c0 + min(wk.own_i, nt - 1);
    if constexpr (!STATES) wk.fetch_row(qb + t * a.q_ld, qr);
    wk.fetch_row(kb + t * a.k_ld, kr);
    wk.fetch_values(c0, nt, vr);
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      step_r[r] = steps[c0 + min(lg * 4 + r, nt - 1)];
      sum_r[r] = sums[c0 + min(lg * 4 + r, nt - 1)];
    }
    own_r = sums[c0 + min(lo, nt - 1)];
    total_r = sums[c0 + nt - 1];
  };
  fetch(0);
  for (int c0 = 0; c0 < wk.len; c0 += TB) {
    const int nt = min(TB, wk.len - c0);
    __syncthreads();                               // the last block has been read
    op.stage(wk, qr, kr, nt, !STATES);
    float v[4];
#pragma unroll
    for (int r = 0; r < 4; ++r) v[r] = lg * 4 + r < nt ? to_f32(vr[r]) : 0.f;
    // of token lo, of tokens 4 lg + r (whose value is 0 past the end), of the block
    const float cs = own_r, total = total_r;
    float csj[4], f[4];
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      csj[r] = sum_r[r];
      f[r] = step_r[r];
    }
    __syncthreads();
    if (c0 + TB < wk.len) fetch(c0 + TB);

    log_decay += total;
    if constexpr (!STATES) {
      scan_f32x4 o = scan_f32x4{0.f, 0.f, 0.f, 0.f}, o2 = o;
      scan_f32x4 g = op.gram(lo, lg);
#pragma unroll
      for (int kt = 0; kt < KT; ++kt) {
        const float4 x = op.query4(lo, kt * 16 + lg * 4);
        o = mfma4(x.x, wk.S[kt][0], o);
        o2 = mfma4(x.y, wk.S[kt][1], o2);
        o = mfma4(x.z, wk.S[kt][2], o);
        o2 = mfma4(x.w, wk.S[kt][3], o2);
      }
      o += o2;
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        g[r] = lg * 4 + r <= lo ? g[r] * __expf(cs - csj[r]) * f[r] : 0.f;
        o[r] *= __expf(csj[r]);
      }
#pragma unroll
      for (int r = 0; r < 4; ++r) o = mfma4(g[r], v[r], o);
#pragma unroll
      for (int r = 0; r < 4; ++r) o[r] = fmaf(skip, v[r], o[r]);
      wk.store_out(c0, nt, o);
    }
#pragma unroll
    for (int r = 0; r < 4; ++r) v[r] *= __expf(total - csj[r]) * f[r];
    const float e = __expf(total);
#pragma unroll
    for (int kt = 0; kt < KT; ++kt) wk.S[kt] *= e;
    op.add(wk.S, v, lo, lg);
  }
  if constexpr (STATES) {
    if (blockIdx.x == 0 && wk.tid == 0) a.seg_decay[wk.sh] = __expf(log_decay);
    wk.store_segment();
  } else {
    wk.store_final();
  }
}

// Segments' own states -> the states they begin with, in place. A thread has one
// element of one head; key_decay: a decay per key, else one per head.
__global__ __launch_bounds__(256) void scan_link_kernel(float* __restrict__ seg_state,
                                                        const float* __restrict__ seg_decay,
                                                        const int* __restrict__ cu, int segs,
                                                        int seg_len, int H, int K, int P,
                                                        bool key_decay) {
  const long n = (long)H * K * P, i = (long)blockIdx.x * 256 + threadIdx.x;
  if (i >= n) return;
  const int seq = blockIdx.y, len = cu[seq + 1] - cu[seq];
  const long at = key_decay ? i / P : i / ((long)K * P), decays = key_decay ? (long)H * K : H;
  float s = 0.f;
  for (int g = 0; g * seg_len < len; ++g) {
    float* p = seg_state + ((long)seq * segs + g) * n + i;
    const bool last = (g + 1) * seg_len >= len;    // has no state of its own
    const float own = last ? 0.f : *p;
    *p = s;
    if (!last) s = fmaf(seg_decay[((long)seq * segs + g) * decays + at], s, own);
  }
}

// ---------------------------------------------------------------------------
// one token: grid (heads, rows); a thread owns V columns and every ng-th key
// ---------------------------------------------------------------------------
// A thread's share of one head's state: V columns of every ng-th key. The first
// PRE of them are loaded early, while the step's vectors are still being made.
constexpr int PRE = 8;
template <int V>
struct StatePart {
  float* st;
  int K, P, units, wide, ng, p, g;
  float s[PRE][V];
  __device__ __forceinline__ StatePart(float* st_, int K_, int P_) : st(st_), K(K_), P(P_) {
    units = P / V;
    wide = min(units, 256);
    ng = 256 / wide;
    p = threadIdx.x % wide;
    g = threadIdx.x / wide;
#pragma unroll
    for (int j = 0; j < PRE; ++j)
      load_vec<float, V>(st + (long)min(g % ng + j * ng, K - 1) * P + p * V, s[j]);
  }
  // y[p] of the step in red[p]; S <- decay * S + k x^T. READ_OLD: y from the
  // state before the update, else after it.
  template <bool READ_OLD>
  __device__ __forceinline__ void step(const float* __restrict__ decay, bool per_key,
                                       const float* __restrict__ k, const float* __restrict__ q,
                                       const float* __restrict__ x, float* __restrict__ red) {
    for (int u0 = 0; u0 < units; u0 += wide) {
      const int u = u0 + p;
      if (g >= ng || u >= units) continue;
      float y[V], xv[V];
#pragma unroll
      for (int j = 0; j < V; ++j) {
        y[j] = 0.f;
        xv[j] = x[u * V + j];
      }
      auto one = [&](int key, float (&v)[V]) {
        const float dc = decay[per_key ? key : 0], kk = k[key], qq = q[key];
#pragma unroll
        for (int j = 0; j < V; ++j) {
          if (READ_OLD) y[j] = fmaf(qq, v[j], y[j]);
          v[j] = fmaf(dc, v[j], kk * xv[j]);
          if (!READ_OLD) y[j] = fmaf(qq, v[j], y[j]);
        }
        store_vec<float, V>(st + (long)key * P + u * V, v);
      };
      int key = g;
      if (u0 == 0) {
#pragma unroll
        for (int j = 0; j < PRE; ++j)
          if (g + j * ng < K) one(g + j * ng, s[j]);
        key = g + PRE * ng;
      }
#pragma unroll 4
      for (; key < K; key += ng) {
        float v[V];
        load_vec<float, V>(st + (long)key * P + u * V, v);
        one(key, v);
      }
#pragma unroll
      for (int j = 0; j < V; ++j) red[g * P + u * V + j] = y[j];
    }
    __syncthreads();
    for (int i = threadIdx.x; i < P; i += 256) {
      float y = 0.f;
      for (int e = 0; e < ng; ++e) y += red[e * P + i];
      red[i] = y;                                  // column i is this thread's alone
    }
    __syncthreads();
  }
};

// Floats of red that StatePart::step needs.
int64_t step_scratch(int64_t P, int64_t V) {
  const int64_t wide = std::min<int64_t>(P / V, 256);
  return 256 / wide * P;
}

template <typename T, int V>
__global__ __launch_bounds__(256) void ssd_decode_kernel(
    const T* __restrict__ xbc, int C, const T* __restrict__ dt_in, long dt_ld,
    const T* __restrict__ dt_bias, const T* __restrict__ a_log, const T* __restrict__ d_skip,
    const int* __restrict__ slot, float* __restrict__ state, int n_slots, int H, int G, int N,
    int P, T* __restrict__ out) {
  extern __shared__ __attribute__((aligned(16))) float lds[];
  float *k = lds, *q = k + N, *x = q + N, *dec = x + P, *red = dec + 4;
  const int h = blockIdx.x, tid = threadIdx.x;
  const long r = blockIdx.y;
  const int sl = slot[r];
  if (sl < 0 || sl >= n_slots) return;             // uniform over the block
  StatePart<V> part(state + ((long)sl * H + h) * N * P, N, P);
  const float dt = softplus_f(to_f32(dt_in[r * dt_ld + h]) + to_f32(dt_bias[h]));
  const T* row = xbc + r * C;
  const T* b = row + (long)H * P + (long)(h / (H / G)) * N;
  for (int i = tid; i < N; i += 256) {
    k[i] = dt * to_f32(b[i]);
    q[i] = to_f32(b[(long)G * N + i]);
  }
  for (int i = tid; i < P; i += 256) x[i] = to_f32(row[(long)h * P + i]);
  if (tid == 0) dec[0] = expf(-expf(to_f32(a_log[h])) * dt);
  __syncthreads();
  part.template step<false>(dec, false, k, q, x, red);
  const float d = to_f32(d_skip[h]);
  for (int i = tid; i < P; i += 256)
    out[(r * H + h) * P + i] = from_f32<T>(fmaf(d, x[i], red[i]));
}

// proj row: [r | k | v | g : H n each | low : rank]. Decay, recurrence, norm and
// gate of one head.
template <typename T, int V>
__global__ __launch_bounds__(256) void wkv_decode_kernel(
    const T* __restrict__ proj, long ld, const T* __restrict__ w2, int rank,
    const T* __restrict__ w0, const T* __restrict__ u, const T* __restrict__ w_norm, float eps,
    const int* __restrict__ slot, float* __restrict__ state, int n_slots, int H, int n,
    T* __restrict__ out) {
  extern __shared__ __attribute__((aligned(16))) float lds[];
  float *q = lds, *k = q + n, *x = k + n, *dec = x + n, *low = dec + n;
  float *sm = low + rank, *red = sm + 8;
  const int h = blockIdx.x, tid = threadIdx.x;
  const long r = blockIdx.y, hn = (long)H * n;
  const int sl = slot[r];
  if (sl < 0 || sl >= n_slots) return;             // uniform over the block
  StatePart<V> part(state + ((long)sl * H + h) * n * n, n, n);
  const T* row = proj + r * ld;
  for (int i = tid; i < rank; i += 256) low[i] = tanhf(to_f32(row[4 * hn + i]));
  float ruk = 0.f;
  for (int i = tid; i < n; i += 256) {
    q[i] = to_f32(row[h * n + i]);
    k[i] = to_f32(row[hn + h * n + i]);
    x[i] = to_f32(row[2 * hn + h * n + i]);
    ruk = fmaf(q[i] * to_f32(u[h * n + i]), k[i], ruk);
  }
  ruk = block_reduce_sum(ruk, sm);                 // also: low, q, k, x are written
  for (int c = tid >> 2; c < (n + 63) / 64 * 64; c += 64) {
    float d = 0.f;
    if (c < n && rank % 32 == 0) {                 // a quarter of the row per lane
      for (int j = (tid & 3) * 8; j < rank; j += 32) {
        float w[8];
        load_vec<T, 8>(w2 + ((long)h * n + c) * rank + j, w);
#pragma unroll
        for (int e = 0; e < 8; ++e) d = fmaf(w[e], low[j + e], d);
      }
    } else if (c < n) {
      for (int j = tid & 3; j < rank; j += 4)
        d = fmaf(to_f32(w2[((long)h * n + c) * rank + j]), low[j], d);
    }
    d += __shfl_xor(d, 1);
    d += __shfl_xor(d, 2);
    if (c < n && (tid & 3) == 0)
      dec[c] = expf(fmaxf(-expf(d + to_f32(w0[h * n + c])), MIN_LOG));
  }
  __syncthreads();
  part.template step<true>(dec, true, k, q, x, red);
  float ss = 0.f;
  for (int i = tid; i < n; i += 256) {
    const float o = fmaf(ruk, x[i], red[i]);
    red[i] = o;
    ss = fmaf(o, o, ss);
  }
  const float inv = 1.0f / sqrtf(block_reduce_sum(ss, sm) / (float)n + eps);
  for (int i = tid; i < n; i += 256)
    out[r * hn + h * n + i] = from_f32<T>(red[i] * inv * to_f32(w_norm[h * n + i]) *
                                          silu_f(to_f32(row[3 * hn + h * n + i])));
}

// Groups of `size` columns, TPG threads each; up to NIT vectors of a thread stay
// in registers (NIT 0: any size, read twice).
template <typename T, int V, int TPG, int NIT>
__global__ __launch_bounds__(256) void gated_group_norm_kernel(
    const T* __restrict__ y, const T* __restrict__ z, long z_ld, const T* __restrict__ w,
    T* __restrict__ out, long n_groups, int groups, int size, float eps, bool gate_first) {
  __shared__ float red[4];
  const long gi = (long)blockIdx.x * (256 / TPG) + threadIdx.x / TPG;
  const bool live = gi < n_groups;                 // else it helps with the shuffles only
  const long t = live ? gi / groups : 0;
  const int c0 = live ? (int)(gi % groups) * size : 0;
  const int lane = threadIdx.x % TPG;
  const T* yr = y + t * groups * size + c0;
  const T* zr = z + t * z_ld + c0;
  T* to = out + t * groups * size + c0;
  float ss = 0.f;
  float kept[NIT ? NIT : 1][V], gate[NIT ? NIT : 1][V];
  auto read = [&](int i, float (&a)[V], float (&b)[V]) {
    load_vec<T, V>(yr + i, a);
    load_vec<T, V>(zr + i, b);
#pragma unroll
    for (int j = 0; j < V; ++j) {
      b[j] = silu_f(b[j]);
      if (gate_first) a[j] *= b[j];
    }
  };
  auto write = [&](int i, float inv, float (&a)[V], float (&b)[V]) {
    float g[V];
    load_vec<T, V>(w + c0 + i, g);
#pragma unroll
    for (int j = 0; j < V; ++j) a[j] = a[j] * inv * g[j] * (gate_first ? 1.f : b[j]);
    store_vec<T, V>(to + i, a);
  };
  if constexpr (NIT > 0) {
#pragma unroll
    for (int n = 0; n < NIT; ++n) {
      const int i = (n * TPG + lane) * V;
      if (i < size) {
        read(i, kept[n], gate[n]);
#pragma unroll
        for (int j = 0; j < V; ++j) ss = fmaf(kept[n][j], kept[n][j], ss);
      }
    }
  } else {
    for (int i = lane * V; i < size; i += TPG * V) {
      read(i, kept[0], gate[0]);
#pragma unroll
      for (int j = 0; j < V; ++j) ss = fmaf(kept[0][j], kept[0][j], ss);
    }
  }
  if constexpr (TPG == 256) {
    ss = block_reduce_sum(ss, red);
  } else {
#pragma unroll
    for (int off = TPG / 2; off > 0; off >>= 1) ss += __shfl_xor(ss, off);
  }
  if (!live) return;
  const float inv = 1.0f / sqrtf(ss / (float)size + eps);
  if constexpr (NIT > 0) {
#pragma unroll
    for (int n = 0; n < NIT; ++n) {
      const int i = (n * TPG + lane) * V;
      if (i < size) write(i, inv, kept[n], gate[n]);
    }
  } else {
    for (int i = lane * V; i < size; i += TPG * V) {
      read(i, kept[0], gate[0]);
      write(i, inv, kept[0], gate[0]);
    }
  }
}

// ---------------------------------------------------------------------------
bool is_elem(const at::Tensor& x) {
  return x.scalar_type() == at::kBFloat16 || x.scalar_type() == at::kFloat;
}
void check_t(const at::Tensor& t, at::ScalarType dt, int64_t n, const char* what) {
  TORCH_CHECK(t.is_cuda() && t.is_contiguous() && t.scalar_type() == dt && t.numel() == n, what,
              ": contiguous GPU tensor of ", n, " ", dt, " elements expected, got ", t.sizes());
}
// rows of a wider matrix: unit column stride
void check_rows(const at::Tensor& t, at::ScalarType dt, int64_t T, int64_t n, const char* what) {
  TORCH_CHECK(t.is_cuda() && t.dim() == 2 && t.size(0) == T && t.size(1) == n &&
                  (n == 1 || t.stride(1) == 1) && t.stride(0) >= n && t.scalar_type() == dt,
              what, ": [", T, ", ", n, "] rows of the activation dtype expected");
}
void check_i32(const at::Tensor& x, int64_t n, const char* what) {
  TORCH_CHECK(x.is_cuda() && x.is_contiguous() && x.scalar_type() == at::kInt && x.numel() == n,
              what, ": contiguous int32 GPU tensor of ", n, " expected");
}
bool aligned16(const at::Tensor& t) {
  return reinterpret_cast<uintptr_t>(t.data_ptr()) % 16 == 0 &&
         (t.dim() < 2 || t.stride(0) * t.element_size() % 16 == 0);
}
constexpr int64_t MAX_KEYS = 256;
constexpr int64_t TARGET_GROUPS = 512;  // workgroups of a prompt pass: two per CU

template <typename T, bool WKV>
void launch_scan(ScanArgs<T> a, int64_t n_seqs, int64_t max_len, const at::TensorOptions& f32,
                 hipStream_t stream) {
  auto ok = [](const void* p, int64_t ld) {
    return reinterpret_cast<uintptr_t>(p) % 16 == 0 && ld * sizeof(T) % 16 == 0;
  };
  a.vec = (a.K == 16 || a.K == 32 || a.K == 64 || a.K == 128 || a.K == 256) && ok(a.q, a.q_ld) &&
          ok(a.k, a.k_ld) && ok(a.cum, 16);
  // segments of at least 8 blocks, as many as fill the chip
  const int64_t groups = (a.P + 63) / 64 * a.H * n_seqs, blocks = (max_len + TB - 1) / TB;
  const int64_t want = std::min<int64_t>((TARGET_GROUPS + groups - 1) / groups, blocks / 8);
  a.seg_len = (int)((blocks + std::max<int64_t>(want, 1) - 1) / std::max<int64_t>(want, 1)) * TB;
  a.segs = (int)((max_len + a.seg_len - 1) / a.seg_len);
  TORCH_CHECK(n_seqs * a.segs <= 65535, "recurrence: too many sequences");
  at::Tensor seg_state, seg_decay;
  if (a.segs > 1) {
    seg_state = at::empty({n_seqs * a.segs, a.H, a.K, a.P}, f32);
    seg_decay = at::empty({n_seqs * a.segs, a.H, WKV ? a.K : 1}, f32);
    a.seg_state = seg_state.data_ptr<float>();
    a.seg_decay = seg_decay.data_ptr<float>();
  }
  const dim3 grid((a.P + 63) / 64, a.H, n_seqs * a.segs);
#define LAUNCH_PASS(KT, STATES)                                                                 \
  do {                                                                                          \
    if constexpr (WKV) {                                                                        \
      const size_t n = 5 * TB * (KT * 16 + 4) + 2 * KT * 16 + TB * (TB + 4);                    \
      wkv_prompt_kernel<T, KT, STATES><<<grid, dim3(256), n * sizeof(float), stream>>>(a);      \
    } else {                                                                                    \
      ssd_prompt_kernel<T, KT, STATES>                                                          \
          <<<grid, dim3(256), SsdOperands<T, KT>::BYTES, stream>>>(a);                          \
    }                                                                                           \
  } while (0)
#define LAUNCH(KT)                                                                              \
  do {                                                                                          \
    if (a.segs > 1) {                                                                           \
      LAUNCH_PASS(KT, true);                                                                    \
      scan_link_kernel<<<dim3(ceil_div_i((long)a.H * a.K * a.P, 256), n_seqs), dim3(256), 0,    \
                         stream>>>(a.seg_state, a.seg_decay, a.cu, a.segs, a.seg_len, a.H, a.K, \
                                   a.P, WKV);                                                   \
    }                                                                                           \
    LAUNCH_PASS(KT, false);                                                                     \
  } while (0)
  if (a.K <= 16) LAUNCH(1);
  else if (a.K <= 32) LAUNCH(2);
  else if (a.K <= 64) LAUNCH(4);
  else if (a.K <= 128) LAUNCH(8);
  else LAUNCH(16);
#undef LAUNCH
#undef LAUNCH_PASS
}

int64_t check_bounds(const at::Tensor& cu, int64_t T, const std::optional<at::Tensor>& slot,
                     const std::optional<at::Tensor>& state, const char* who) {
  const int64_t n = cu.numel() - 1;
  TORCH_CHECK(n >= 1 && n <= 65535, who, ": cu_seqlens [n + 1]");
  check_i32(cu, n + 1, who);
  if (state) {
    TORCH_CHECK(slot, who, ": a state needs slots");
    check_i32(*slot, T, who);
  }
  return n;
}

}  // namespace

#define PTR(t) reinterpret_cast<scalar*>((t).data_ptr())
#define OPT_I(t) ((t).has_value() ? (t)->data_ptr<int>() : nullptr)

// x [T, C] (rows may be strided) -> silu(conv) [T, C]. Prompt steps give
// seq_end; decode steps take the earlier inputs from state [slots, taps-1, C].
at::Tensor causal_conv_silu(const at::Tensor& x, const at::Tensor& w, const at::Tensor& bias,
                            const at::Tensor& pos, const std::optional<at::Tensor>& slot,
                            const std::optional<at::Tensor>& seq_end,
                            const std::optional<at::Tensor>& state) {
  TORCH_CHECK(x.dim() == 2 && w.dim() == 2 && is_elem(x), "causal_conv_silu: x [T, C], w [C, n]");
  const int64_t T = x.size(0), C = x.size(1), taps = w.size(1);
  const auto dt = x.scalar_type();
  check_rows(x, dt, T, C, "causal_conv_silu x");
  check_t(w, dt, C * taps, "causal_conv_silu w");
  check_t(bias, dt, C, "causal_conv_silu bias");
  check_i32(pos, T, "causal_conv_silu pos");
  TORCH_CHECK(taps >= 1 && taps <= 1024, "causal_conv_silu: 1..1024 taps");
  int64_t n_slots = 0;
  if (state) {
    TORCH_CHECK(slot && state->dim() == 3, "causal_conv_silu: state [slots, taps-1, C]");
    n_slots = state->size(0);
    check_t(*state, dt, n_slots * (taps - 1) * C, "causal_conv_silu state");
    check_i32(*slot, T, "causal_conv_silu slot");
  }
  TORCH_CHECK(seq_end || state, "causal_conv_silu: decoding needs a state");
  if (seq_end) check_i32(*seq_end, T, "causal_conv_silu seq_end");
  auto out = at::empty({T, C}, x.options());
  if (T == 0) return out;
  auto stream = c10::hip::getCurrentHIPStream();
#define LAUNCH(TAPS)                                                                          \
  conv_prompt_kernel<scalar, V, TAPS>                                                         \
      <<<dim3((T + CONV_TOKENS - 1) / CONV_TOKENS, ceil_div_i(C, 256 * V)), dim3(256), 0,     \
         stream>>>(PTR(x), x.stride(0), PTR(w), PTR(bias), pos.data_ptr<int>(), OPT_I(slot),  \
                   OPT_I(seq_end), state && taps > 1 ? PTR(*state) : nullptr, (int)n_slots,   \
                   PTR(out), (int)T, (int)C, (int)taps)
  const bool vec = C % 8 == 0 && aligned16(x);
  if (seq_end) {
    AMD_DISPATCH_T_V(dt, vec, {
      if (taps == 2) LAUNCH(2);
      else if (taps == 3) LAUNCH(3);
      else if (taps == 4) LAUNCH(4);
      else LAUNCH(0);
    });
  } else {
    AMD_DISPATCH_T(dt, {
      if (vec) conv_decode_kernel<scalar, 2><<<dim3(T, ceil_div_i(C, 512)), dim3(256), 0, stream>>>(
          PTR(x), x.stride(0), PTR(w), PTR(bias), pos.data_ptr<int>(), slot->data_ptr<int>(),
          PTR(*state), (int)n_slots, PTR(out), (int)C, (int)taps);
      else conv_decode_kernel<scalar, 1><<<dim3(T, ceil_div_i(C, 256)), dim3(256), 0, stream>>>(
          PTR(x), x.stride(0), PTR(w), PTR(bias), pos.data_ptr<int>(), slot->data_ptr<int>(),
          PTR(*state), (int)n_slots, PTR(out), (int)C, (int)taps);
    });
  }
#undef LAUNCH
  HIP_CHECK_KERNEL();
  return out;
}

// h [T, W], mu [n, W] -> [n, T, W]
at::Tensor token_shift(const at::Tensor& h, const at::Tensor& mu, const at::Tensor& pos,
                       const std::optional<at::Tensor>& slot,
                       const std::optional<at::Tensor>& seq_end,
                       const std::optional<at::Tensor>& state) {
  TORCH_CHECK(h.dim() == 2 && mu.dim() == 2 && is_elem(h), "token_shift: h [T, W], mu [n, W]");
  const int64_t T = h.size(0), W = h.size(1), n = mu.size(0);
  const auto dt = h.scalar_type();
  check_t(h, dt, T * W, "token_shift h");
  check_t(mu, dt, n * W, "token_shift mu");
  check_i32(pos, T, "token_shift pos");
  int64_t n_slots = 0;
  if (state) {
    TORCH_CHECK(slot && state->dim() == 2, "token_shift: state [slots, W]");
    n_slots = state->size(0);
    check_t(*state, dt, n_slots * W, "token_shift state");
    check_i32(*slot, T, "token_shift slot");
  }
  TORCH_CHECK(seq_end || state, "token_shift: decoding needs a state");
  if (seq_end) check_i32(*seq_end, T, "token_shift seq_end");
  auto out = at::empty({n, T, W}, h.options());
  if (T == 0) return out;
  auto stream = c10::hip::getCurrentHIPStream();
  AMD_DISPATCH_T_V(dt, W % 8 == 0, {
    const int threads = std::min(256, ceil_div_i(W, V * WAVE_SIZE) * WAVE_SIZE);
    token_shift_kernel<scalar, V>
        <<<dim3(T, ceil_div_i(W, V * threads)), dim3(threads), 0, stream>>>(
        PTR(h), PTR(mu), (int)n, pos.data_ptr<int>(), OPT_I(slot), OPT_I(seq_end),
        state ? PTR(*state) : nullptr, (int)n_slots, PTR(out), (int)W);
  });
  HIP_CHECK_KERNEL();
  return out;
}

// z [T, I] may be strided rows of a wider matrix.
at::Tensor gated_group_norm(const at::Tensor& y, const at::Tensor& z, const at::Tensor& w,
                            int64_t groups, double eps, bool gate_first) {
  TORCH_CHECK(y.dim() == 2 && is_elem(y), "gated_group_norm: y [T, I]");
  const int64_t T = y.size(0), I = y.size(1);
  const auto dt = y.scalar_type();
  check_t(y, dt, T * I, "gated_group_norm y");
  check_rows(z, dt, T, I, "gated_group_norm z");
  check_t(w, dt, I, "gated_group_norm w");
  TORCH_CHECK(groups >= 1 && I % groups == 0, "gated_group_norm: groups");
  const int64_t size = I / groups, n = T * groups;
  auto out = at::empty_like(y);
  if (n == 0) return out;
  auto stream = c10::hip::getCurrentHIPStream();
#define LAUNCH(TPG, NIT)                                                                       \
  gated_group_norm_kernel<scalar, V, TPG, NIT>                                                 \
      <<<dim3((n + 256 / TPG - 1) / (256 / TPG)), dim3(256), 0, stream>>>(                     \
          PTR(y), PTR(z), z.stride(0), PTR(w), PTR(out), n, (int)groups, (int)size, (float)eps, \
          gate_first)
  AMD_DISPATCH_T_V(dt, size % 8 == 0 && aligned16(z), {
    if (size <= 8 * V) LAUNCH(8, 1);
    else if (size <= 64 * V) LAUNCH(64, 1);
    else if (size <= 128 * V) LAUNCH(64, 2);
    else if (size <= 1024 * V) LAUNCH(256, 4);
    else LAUNCH(256, 0);
  });
#undef LAUNCH
  HIP_CHECK_KERNEL();
  return out;
}

// xbc [T, H*P + 2*G*N] = [x | B | C]; dt [T, H] rows before bias and softplus
at::Tensor ssd_prompt(const at::Tensor& xbc, const at::Tensor& dt_in, const at::Tensor& dt_bias,
                      const at::Tensor& a_log, const at::Tensor& d_skip, const at::Tensor& cu,
                      const std::optional<at::Tensor>& slot,
                      const std::optional<at::Tensor>& state, int64_t groups, int64_t N,
                      int64_t max_len) {
  TORCH_CHECK(xbc.dim() == 2 && is_elem(xbc), "ssd_prompt: xbc [T, C]");
  const int64_t T = xbc.size(0), H = a_log.numel(), C = xbc.size(1);
  const int64_t P = H > 0 ? (C - 2 * groups * N) / H : 0;
  const auto dt = xbc.scalar_type();
  TORCH_CHECK(H >= 1 && groups >= 1 && H % groups == 0 && N >= 1 && N <= MAX_KEYS && P >= 1 &&
                  C == H * P + 2 * groups * N && H <= 65535 && max_len >= 1,
              "ssd_prompt: sizes (state up to ", MAX_KEYS, ")");
  check_t(xbc, dt, T * C, "ssd_prompt xbc");
  check_rows(dt_in, dt, T, H, "ssd_prompt dt");
  check_t(dt_bias, dt, H, "ssd_prompt dt_bias");
  check_t(a_log, dt, H, "ssd_prompt A_log");
  check_t(d_skip, dt, H, "ssd_prompt D");
  const int64_t n = check_bounds(cu, T, slot, state, "ssd_prompt");
  if (state) check_t(*state, at::kFloat, state->size(0) * H * N * P, "ssd_prompt state");
  auto out = at::empty({T, H * P}, xbc.options());
  if (T == 0) return out;
  auto steps = at::empty({H, T}, xbc.options().dtype(at::kFloat)), sums = at::empty_like(steps);
  auto stream = c10::hip::getCurrentHIPStream().stream();
  AMD_DISPATCH_T(dt, {
    ScanArgs<scalar> a{};
    a.v = PTR(xbc);
    a.k = PTR(xbc) + H * P;
    a.q = a.k + groups * N;
    a.q_ld = a.k_ld = a.v_ld = C;
    a.q_hs = a.k_hs = (int)N;
    a.per_group = (int)(H / groups);
    step_cumsum_kernel<scalar>
        <<<dim3(ceil_div_i(max_len, 4 * TB), n, ceil_div_i(H, 64)), dim3(256), 0, stream>>>(
            PTR(dt_in), dt_in.stride(0), PTR(dt_bias), PTR(a_log), cu.data_ptr<int>(), (int)H,
            (int)T, steps.data_ptr<float>(), sums.data_ptr<float>());
    a.steps = steps.data_ptr<float>();
    a.sums = sums.data_ptr<float>();
    a.n_tok = (int)T;
    a.d_skip = PTR(d_skip);
    a.cu = cu.data_ptr<int>();
    a.slot = OPT_I(slot);
    a.state = state ? state->data_ptr<float>() : nullptr;
    a.n_slots = state ? (int)state->size(0) : 0;
    a.H = (int)H;
    a.K = (int)N;
    a.P = (int)P;
    a.out = PTR(out);
    launch_scan<scalar, false>(a, n, max_len, xbc.options().dtype(at::kFloat), stream);
  });
  HIP_CHECK_KERNEL();
  return out;
}

at::Tensor ssd_decode(const at::Tensor& xbc, const at::Tensor& dt_in, const at::Tensor& dt_bias,
                      const at::Tensor& a_log, const at::Tensor& d_skip, const at::Tensor& slot,
                      at::Tensor state, int64_t groups, int64_t N) {
  TORCH_CHECK(xbc.dim() == 2 && is_elem(xbc), "ssd_decode: xbc [R, C]");
  const int64_t R = xbc.size(0), H = a_log.numel(), C = xbc.size(1);
  const int64_t P = H > 0 ? (C - 2 * groups * N) / H : 0;
  const auto dt = xbc.scalar_type();
  TORCH_CHECK(H >= 1 && groups >= 1 && H % groups == 0 && N >= 1 && P >= 1 && P <= 2048 &&
                  N <= 4096 && C == H * P + 2 * groups * N && R <= 65535,
              "ssd_decode: sizes");
  check_t(xbc, dt, R * C, "ssd_decode xbc");
  check_rows(dt_in, dt, R, H, "ssd_decode dt");
  check_t(dt_bias, dt, H, "ssd_decode dt_bias");
  check_t(a_log, dt, H, "ssd_decode A_log");
  check_t(d_skip, dt, H, "ssd_decode D");
  check_i32(slot, R, "ssd_decode slot");
  check_t(state, at::kFloat, state.size(0) * H * N * P, "ssd_decode state");
  auto out = at::empty({R, H * P}, xbc.options());
  if (R == 0) return out;
  auto stream = c10::hip::getCurrentHIPStream();
#define LAUNCH(V)                                                                              \
  ssd_decode_kernel<scalar, V>                                                                 \
      <<<dim3(H, R), dim3(256), (2 * N + P + 4 + step_scratch(P, V)) * sizeof(float),          \
         stream>>>(PTR(xbc), (int)C, PTR(dt_in), dt_in.stride(0), PTR(dt_bias), PTR(a_log),    \
                   PTR(d_skip), slot.data_ptr<int>(), state.data_ptr<float>(),                 \
                   (int)state.size(0), (int)H, (int)groups, (int)N, (int)P, PTR(out))
  AMD_DISPATCH_T(dt, {
    if (P % 4 == 0) LAUNCH(4);
    else LAUNCH(1);
  });
#undef LAUNCH
  HIP_CHECK_KERNEL();
  return out;
}

// r, k, v [T, H*n] (rows may be strided) of the activation dtype, low [T, H*n]
// f32 (overwritten) the decay's projection before w0
at::Tensor wkv_prompt(const at::Tensor& r, const at::Tensor& k, const at::Tensor& v,
                      at::Tensor low, const at::Tensor& w0, const at::Tensor& u,
                      const at::Tensor& cu, const std::optional<at::Tensor>& slot,
                      const std::optional<at::Tensor>& state, int64_t max_len) {
  TORCH_CHECK(r.dim() == 2 && u.dim() == 2 && is_elem(r), "wkv_prompt: r [T, H*n], u [H, n]");
  const int64_t T = r.size(0), H = u.size(0), n = u.size(1);
  const auto dt = r.scalar_type();
  TORCH_CHECK(n >= 1 && n <= MAX_KEYS && H >= 1 && H <= 65535 && max_len >= 1,
              "wkv_prompt: heads of up to ", MAX_KEYS);
  check_rows(r, dt, T, H * n, "wkv_prompt r");
  check_rows(k, dt, T, H * n, "wkv_prompt k");
  check_rows(v, dt, T, H * n, "wkv_prompt v");
  check_t(low, at::kFloat, T * H * n, "wkv_prompt low");
  check_t(w0, dt, H * n, "wkv_prompt w0");
  check_t(u, dt, H * n, "wkv_prompt u");
  const int64_t seqs = check_bounds(cu, T, slot, state, "wkv_prompt");
  if (state) check_t(*state, at::kFloat, state->size(0) * H * n * n, "wkv_prompt state");
  auto out = at::empty({T, H * n}, r.options());
  if (T == 0) return out;
  auto stream = c10::hip::getCurrentHIPStream().stream();
  AMD_DISPATCH_T(dt, {
    decay_cumsum_kernel<scalar>
        <<<dim3((max_len + TB - 1) / TB, seqs, (H * n + 255) / 256), dim3(256), 0, stream>>>(
            low.data_ptr<float>(), PTR(w0), cu.data_ptr<int>(), (int)(H * n));
    ScanArgs<scalar> a{};
    a.q = PTR(r);
    a.k = PTR(k);
    a.v = PTR(v);
    a.q_ld = r.stride(0);
    a.k_ld = k.stride(0);
    a.v_ld = v.stride(0);
    a.q_hs = a.k_hs = (int)n;
    a.per_group = 1;
    a.cum = low.data_ptr<float>();
    a.u = PTR(u);
    a.cu = cu.data_ptr<int>();
    a.slot = OPT_I(slot);
    a.state = state ? state->data_ptr<float>() : nullptr;
    a.n_slots = state ? (int)state->size(0) : 0;
    a.H = (int)H;
    a.K = a.P = (int)n;
    a.out = PTR(out);
    launch_scan<scalar, true>(a, seqs, max_len, low.options(), stream);
  });
  HIP_CHECK_KERNEL();
  return out;
}

// proj [R, 4*H*n + rank] = [r | k | v | g | low] -> gated, normed heads [R, H*n]
at::Tensor wkv_decode(const at::Tensor& proj, const at::Tensor& w2, const at::Tensor& w0,
                      const at::Tensor& u, const at::Tensor& w_norm, double eps,
                      const at::Tensor& slot, at::Tensor state) {
  TORCH_CHECK(proj.dim() == 2 && w2.dim() == 2 && u.dim() == 2 && is_elem(proj),
              "wkv_decode: proj [R, 4*H*n + rank], w2 [H*n, rank], u [H, n]");
  const int64_t R = proj.size(0), H = u.size(0), n = u.size(1), rank = w2.size(1);
  const auto dt = proj.scalar_type();
  TORCH_CHECK(H >= 1 && n >= 1 && n <= 1024 && rank >= 1 && rank <= 4096 && R <= 65535,
              "wkv_decode: sizes");
  check_t(proj, dt, R * (4 * H * n + rank), "wkv_decode proj");
  check_t(w2, dt, H * n * rank, "wkv_decode w2");
  check_t(w0, dt, H * n, "wkv_decode w0");
  check_t(u, dt, H * n, "wkv_decode u");
  check_t(w_norm, dt, H * n, "wkv_decode norm");
  check_i32(slot, R, "wkv_decode slot");
  check_t(state, at::kFloat, state.size(0) * H * n * n, "wkv_decode state");
  auto out = at::empty({R, H * n}, proj.options());
  if (R == 0) return out;
  auto stream = c10::hip::getCurrentHIPStream();
#define LAUNCH(V)                                                                               \
  wkv_decode_kernel<scalar, V>                                                                  \
      <<<dim3(H, R), dim3(256), (4 * n + rank + 8 + step_scratch(n, V)) * sizeof(float),        \
         stream>>>(PTR(proj), proj.size(1), PTR(w2), (int)rank, PTR(w0), PTR(u), PTR(w_norm),   \
                   (float)eps, slot.data_ptr<int>(), state.data_ptr<float>(),                   \
                   (int)state.size(0), (int)H, (int)n, PTR(out))
  AMD_DISPATCH_T(dt, {
    if (n % 4 == 0) LAUNCH(4);
    else LAUNCH(1);
  });
#undef LAUNCH
  HIP_CHECK_KERNEL();
  return out;
}

#undef PTR
#undef OPT_I

}  // namespace amd_ops
