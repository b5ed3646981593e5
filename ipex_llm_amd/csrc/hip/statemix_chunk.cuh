// Device code that the chunked forms of the matrix-state recurrences share
// (statemix_chunk.hip: one decay per head, chanmix_chunk.hip: one per key
// channel): finding a step's chunks, the 16x16x4 f32 products, the chain over
// the chunks and the read-out.  A lane group g of four takes the summed index
// 16 j + 4 g + i at step (j, i), for both operands alike, so every operand is
// read as 16-byte pieces.
#pragma once
#include "statemix.h"

#include <math.h>

namespace illm {
namespace sx {
namespace {

constexpr int C = kChunk;
typedef float f32x4 __attribute__((ext_vector_type(4)));

template <typename E> __device__ __forceinline__ float ldf(const E* p);
template <> __device__ __forceinline__ float ldf<float>(const float* p) { return *p; }
template <> __device__ __forceinline__ float ldf<__bf16>(const __bf16* p) { return (float)*p; }

__device__ __forceinline__ float wave_sum(float v) {
#pragma unroll
  for (int o = 32; o > 0; o >>= 1) v += __shfl_xor(v, o, 64);
  return v;
}
__device__ __forceinline__ float sigmoidf(float z) { return 1.0f / (1.0f + expf(-z)); }
__device__ __forceinline__ float silu(float z) { return z / (1.0f + expf(-z)); }
__device__ __forceinline__ float softplusf(float z) { return z > 20.f ? z : log1pf(expf(z)); }

// tokens of sequence b inside the segment [seg0, seg0 + seg) of every portion
__device__ __forceinline__ int seg_tokens(const int32_t* cu, int b, int seg0, int seg) {
  const int n = cu[b + 1] - cu[b] - seg0;
  return n < 0 ? 0 : (n > seg ? seg : n);
}
__device__ __forceinline__ int chunks_of(int n) { return (n + C - 1) / C; }

// the x-th chunk of the step: its sequence and its index there (every wave finds it by itself); false: past the end
__device__ __forceinline__ bool find_chunk(const int32_t* cu, int B, int seg0, int seg, int x, int* b_out, int* c_out) {
  const int lane = threadIdx.x & 63;
  int before = 0;
  for (int b0 = 0; b0 < B; b0 += 64) {
    const int n = b0 + lane < B ? chunks_of(seg_tokens(cu, b0 + lane, seg0, seg)) : 0;
    int upto = n;
#pragma unroll
    for (int o = 1; o < 64; o <<= 1) {
      const int v = __shfl_up(upto, o, 64);
      if (lane >= o) upto += v;
    }
    const unsigned long long m = __ballot(before + upto > x);
    if (m) {
      const int l = __ffsll((long long)m) - 1;
      *b_out = b0 + l;
      *c_out = x - (before + __shfl(upto, l, 64) - __shfl(n, l, 64));
      return true;
    }
    before += __shfl(upto, 63, 64);
  }
  return false;
}
// chunks of the sequences in front of b
__device__ __forceinline__ int chunks_before(const int32_t* cu, int b, int seg0, int seg) {
  int n = 0;
  for (int i = threadIdx.x & 63; i < b; i += 64) n += chunks_of(seg_tokens(cu, i, seg0, seg));
#pragma unroll
  for (int o = 32; o > 0; o >>= 1) n += __shfl_xor(n, o, 64);
  return n;
}

__device__ __forceinline__ f32x4 mfma4(const f32x4& a, const f32x4& b, f32x4 c) {
#pragma unroll
  for (int i = 0; i < 4; i++) c = __builtin_amdgcn_mfma_f32_16x16x4f32(a[i], b[i], c, 0, 0, 0);
  return c;
}
__device__ __forceinline__ f32x4 ld4(const float* p) { return *(const f32x4*)p; }
__device__ __forceinline__ void st4(float* p, const f32x4& v) { *(f32x4*)p = v; }

// scratch of one launch sequence, per (chunk, head); DP: d rounded up to ND 16, DV: dv rounded up to 16
struct Scratch {
  float* w;     // [C][DP]
  float* gq;    // [C][DP]   e^(G_t) q_t
  float* kd;    // [DP][C]   e^(G_last - G_s) k_s
  float* p;     // [C][C]    tiles on and below the diagonal
  float* u;     // [DV][C]
  float* s0;    // [DV][DP]  start state
  float* gc;    // e^(G_last): one number, or [DP] with a decay per key channel
};

// x <- (I + A)^-1 x for one column: A strictly lower triangular in LDS (row stride LA, a multiple of 4), x in registers
__device__ __forceinline__ void solve_unit_lower(const float* As, int LA, float (&x)[C]) {
  // four rows at a time: what the rows above contribute (16 columns of A between two scheduling barriers, so that
  // A's values do not all sit in registers at once), then the rows' own triangle
#pragma unroll
  for (int tb = 0; tb < C; tb += 4) {
#pragma unroll
    for (int s = 0; s < tb; s += 4) {
#pragma unroll
      for (int i = 0; i < 4; i++) {
        const f32x4 a = ld4(As + (tb + i) * LA + s);
#pragma unroll
        for (int e = 0; e < 4; e++) x[tb + i] = fmaf(-a[e], x[s + e], x[tb + i]);
      }
      if ((s & 15) == 12) __builtin_amdgcn_sched_barrier(0);
    }
#pragma unroll
    for (int i = 1; i < 4; i++) {
      const f32x4 a = ld4(As + (tb + i) * LA + tb);
#pragma unroll
      for (int e = 0; e < i; e++) x[tb + i] = fmaf(-a[e], x[tb + e], x[tb + i]);
    }
    __builtin_amdgcn_sched_barrier(0);
  }
}

// CHAN: one factor per state row in gc ([DP] per chunk and head) instead of one number
template <int ND, bool DELTA, bool CHAN>
__global__ void __launch_bounds__(256) chunk_chain_k(float* __restrict__ S, const int32_t* __restrict__ cu,
                                                    const int32_t* __restrict__ slots, const int64_t* __restrict__ pos,
                                                    int seg0, int seg, Scratch sc, int H, int d, int dv, int DV) {
  constexpr int DP = 16 * ND, LD = DP + 4, LU = C + 4, NT = (ND + 3) / 4;   // a wave's tiles of 16 state rows: wv + 4 u
  __shared__ __attribute__((aligned(16))) float Ss[16 * LD];
  __shared__ __attribute__((aligned(16))) float Us[16 * LU];
  const int b = blockIdx.z, h = blockIdx.y, p0 = 16 * blockIdx.x;
  const int n = seg_tokens(cu, b, seg0, seg);
  if (n <= 0) return;
  const int nch = chunks_of(n), base = chunks_before(cu, b, seg0, seg);
  const int lane = threadIdx.x & 63, wv = threadIdx.x >> 6, r16 = lane & 15, g = lane >> 4;
  const int pc = p0 + r16;
  float* Sg = S + (((int64_t)slots[b] * H + h) * d) * dv;           // [d][dv]
  const bool fresh = seg0 == 0 && pos[cu[b]] == 0;
  f32x4 st[NT];
#pragma unroll
  for (int u = 0; u < NT; u++)
#pragma unroll
    for (int i = 0; i < 4; i++) {
      const int r = 16 * (wv + 4 * u) + 4 * g + i;
      st[u][i] = (!fresh && r < d && pc < dv) ? Sg[(int64_t)r * dv + pc] : 0.f;
    }
  f32x4 wf[ND], kf[NT][4], uf, ub[4];                               // the next chunk's operands, requested ahead
  float gf = 0.f;
  f32x4 gv[NT];
  auto request = [&](int c) {
    const int64_t at = (int64_t)(base + c) * H + h;
    if (CHAN) {
#pragma unroll
      for (int u = 0; u < NT; u++)
        if (wv + 4 * u < ND) gv[u] = ld4(sc.gc + at * DP + 16 * (wv + 4 * u) + 4 * g);
    } else {
      gf = sc.gc[at];
    }
    if (DELTA) {
#pragma unroll
      for (int j = 0; j < ND; j++) wf[j] = ld4(sc.w + at * C * DP + (16 * wv + r16) * DP + 16 * j + 4 * g);
      uf = ld4(sc.u + (at * DV + pc) * C + 16 * wv + 4 * g);
    } else {
#pragma unroll
      for (int j = 0; j < 4; j++) ub[j] = ld4(sc.u + (at * DV + pc) * C + 16 * j + 4 * g);
    }
#pragma unroll
    for (int u = 0; u < NT; u++)
      if (wv + 4 * u < ND) {
#pragma unroll
        for (int j = 0; j < 4; j++) kf[u][j] = ld4(sc.kd + at * C * DP + (16 * (wv + 4 * u) + r16) * C + 16 * j + 4 * g);
      }
  };
  request(0);
  for (int c = 0; c < nch; c++) {
    const int64_t at = (int64_t)(base + c) * H + h;
    f32x4 w[ND], kd[NT][4], un = uf, bu[4];
    const float gc = gf;
    f32x4 gr[NT];
#pragma unroll
    for (int u = 0; u < NT; u++) gr[u] = CHAN ? gv[u] : f32x4{gc, gc, gc, gc};
#pragma unroll
    for (int j = 0; j < ND; j++) w[j] = wf[j];
#pragma unroll
    for (int u = 0; u < NT; u++)
#pragma unroll
      for (int j = 0; j < 4; j++) kd[u][j] = kf[u][j];
#pragma unroll
    for (int j = 0; j < 4; j++) bu[j] = ub[j];
    if (c + 1 < nch) request(c + 1);
#pragma unroll
    for (int u = 0; u < NT; u++)
      if (wv + 4 * u < ND) {
        st4(sc.s0 + (at * DV + pc) * DP + 16 * (wv + 4 * u) + 4 * g, st[u]);
        if (DELTA) st4(Ss + r16 * LD + 16 * (wv + 4 * u) + 4 * g, st[u]);
      }
    if (DELTA) {
      __syncthreads();
      f32x4 ws = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int j = 0; j < ND; j++) ws = mfma4(w[j], ld4(Ss + r16 * LD + 16 * j + 4 * g), ws);
#pragma unroll
      for (int i = 0; i < 4; i++) un[i] -= ws[i];
      st4(Us + r16 * LU + 16 * wv + 4 * g, un);
      st4(sc.u + (at * DV + pc) * C + 16 * wv + 4 * g, un);
      __syncthreads();
#pragma unroll
      for (int j = 0; j < 4; j++) bu[j] = ld4(Us + r16 * LU + 16 * j + 4 * g);
    }
#pragma unroll
    for (int u = 0; u < NT; u++)
      if (wv + 4 * u < ND) {
#pragma unroll
        for (int i = 0; i < 4; i++) st[u][i] *= gr[u][i];
#pragma unroll
        for (int j = 0; j < 4; j++) st[u] = mfma4(kd[u][j], bu[j], st[u]);
      }
  }
#pragma unroll
  for (int u = 0; u < NT; u++)
#pragma unroll
    for (int i = 0; i < 4; i++) {
      const int r = 16 * (wv + 4 * u) + 4 * g + i;
      if (r < d && pc < dv) Sg[(int64_t)r * dv + pc] = st[u][i];
    }
}

template <int ND>
__global__ void __launch_bounds__(256) chunk_read_k(const int32_t* __restrict__ cu, int B, int seg0, int seg, Scratch sc,
                                                   float* __restrict__ out, int H, int dv, int DV) {
  constexpr int DP = 16 * ND;
  int b, c;
  if (!find_chunk(cu, B, seg0, seg, blockIdx.x, &b, &c)) return;
  const int h = blockIdx.y, lane = threadIdx.x & 63, wv = threadIdx.x >> 6, r16 = lane & 15, g = lane >> 4;
  const int nt = min(C, seg_tokens(cu, b, seg0, seg) - c * C);
  if (16 * wv >= nt) return;
  const int64_t t0 = (int64_t)cu[b] + seg0 + (int64_t)c * C;
  const int64_t at = (int64_t)blockIdx.x * H + h;
  f32x4 qa[ND], pa[4];
#pragma unroll
  for (int j = 0; j < ND; j++) qa[j] = ld4(sc.gq + at * C * DP + (16 * wv + r16) * DP + 16 * j + 4 * g);
#pragma unroll
  for (int j = 0; j < 4; j++)
    if (j <= wv) pa[j] = ld4(sc.p + at * C * C + (16 * wv + r16) * C + 16 * j + 4 * g);
  for (int n = 0; n < 4; n++) {
    const int pc = 64 * blockIdx.z + 16 * n + r16;
    if (64 * (int)blockIdx.z + 16 * n >= DV) break;
    f32x4 o = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int j = 0; j < ND; j++) o = mfma4(qa[j], ld4(sc.s0 + (at * DV + pc) * DP + 16 * j + 4 * g), o);
#pragma unroll
    for (int j = 0; j < 4; j++)
      if (j <= wv) o = mfma4(pa[j], ld4(sc.u + (at * DV + pc) * C + 16 * j + 4 * g), o);
    if (pc < dv) {
#pragma unroll
      for (int i = 0; i < 4; i++) {
        const int t = 16 * wv + 4 * g + i;
        if (t < nt) out[((t0 + t) * H + h) * dv + pc] = o[i];
      }
    }
  }
}

}  // namespace
}  // namespace sx
}  // namespace illm
