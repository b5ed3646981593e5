// Matrix-state recurrences with one decay per key channel, token by token
// (gfx950, wave64): decoding and short portions.
//
//   delta rule   S <- diag(g) S, u = beta (v - S^T k), S <- S + k u^T, o = S^T q
//   with bonus   o = S^T r + (sum_c u_c k_c r_c) v, S <- diag(g) S + k v^T
//
// The value columns of a state never meet, so a wave owns 16 columns of one
// (sequence, head): lane = (column, one of four row groups), the state rows in
// registers, a row group's keys, queries and decays read from LDS as 16-byte
// pieces; the sums over the rows end with two shuffles.  Tokens go through LDS
// in chunks (unit norms and step sizes, or the bonus, formed while staging).
#include "chanmix.h"
#include "statemix.h"

#include <math.h>

namespace illm {
namespace cx {
namespace {

template <typename E> __device__ __forceinline__ float ldf(const E* p);
template <> __device__ __forceinline__ float ldf<float>(const float* p) { return *p; }
template <> __device__ __forceinline__ float ldf<__bf16>(const __bf16* p) { return (float)*p; }

__device__ __forceinline__ float wave_sum(float v) {
#pragma unroll
  for (int o = 32; o > 0; o >>= 1) v += __shfl_xor(v, o, 64);
  return v;
}

// EQ: type of q / k / v, EB: of the step sizes' inputs.  NC4: 16-row pieces of the state (d <= 16 NC4).  DELTA: q is the
// query; otherwise q is the receptance r and ``bonus`` [H, d] holds u
template <typename EQ, typename EB, int NC4, bool DELTA>
__global__ void __launch_bounds__(256) chan_scan_k(const EQ* __restrict__ q, int64_t q_ld, const EQ* __restrict__ k,
                                                  int64_t k_ld, const EQ* __restrict__ v, int64_t v_ld,
                                                  const float* __restrict__ gd, const float* __restrict__ bonus, DeltaIn di,
                                                  float* __restrict__ S, const int32_t* __restrict__ cu,
                                                  const int32_t* __restrict__ slots, const int64_t* __restrict__ pos,
                                                  float* __restrict__ out, int H, int K, int d, int dv, int TC) {
  extern __shared__ __align__(16) float sm[];
  constexpr int DP = 16 * NC4;
  const int b = blockIdx.x, h = blockIdx.y, p0 = blockIdx.z * 64;
  const int lane = threadIdx.x & 63, wv = threadIdx.x >> 6, NW = blockDim.x >> 6;
  const int col = lane & 15, rg = lane >> 4;
  const int t0 = cu[b], n = cu[b + 1] - t0;
  if (n <= 0) return;
  const int kh = h / (H / K);
  const int pc = p0 + 16 * wv + col;
  float* Ks = sm;                                                   // [TC][DP]
  float* Qs = Ks + (size_t)TC * DP;                                 // [TC][DP]
  float* Gs = Qs + (size_t)TC * DP;                                 // [TC][DP]
  float* vs = Gs + (size_t)TC * DP;                                 // [TC][64]
  float* bs = vs + (size_t)TC * 64;                                 // [TC] step sizes, or the bonus sums
  float st[4 * NC4];                                                // rows 4 (4 j + rg) + i
  float* Sg = S + (((int64_t)slots[b] * H + h) * d) * dv;           // [d][dv]
  const bool fresh = pos[t0] == 0;
#pragma unroll
  for (int j = 0; j < NC4; j++)
#pragma unroll
    for (int i = 0; i < 4; i++) {
      const int r = 4 * (4 * j + rg) + i;
      st[4 * j + i] = (!fresh && r < d && pc < dv) ? Sg[(int64_t)r * dv + pc] : 0.f;
    }
  for (int c0 = 0; c0 < n; c0 += TC) {
    const int nc = min(TC, n - c0);
    __syncthreads();
    // a wave stages whole tokens (their norms and bonus sums need the row)
    for (int tt = wv; tt < nc; tt += NW) {
      const int64_t t = t0 + c0 + tt;
      constexpr int PL = (DP + 63) / 64;
      float kk[PL], qq[PL], gg[PL];
      float sk = 0.f, sq = 0.f;
#pragma unroll
      for (int i = 0; i < PL; i++) {
        const int r = lane + 64 * i;
        kk[i] = qq[i] = 0.f;
        gg[i] = 1.f;
        if (r < d) {
          kk[i] = ldf(k + t * k_ld + (int64_t)kh * d + r);
          qq[i] = ldf(q + t * q_ld + (int64_t)kh * d + r);
          gg[i] = gd[(t * H + h) * d + r];
          if (!DELTA) sk = fmaf(bonus[(int64_t)h * d + r] * kk[i], qq[i], sk);
        }
        if (DELTA) {
          sk = fmaf(kk[i], kk[i], sk);
          sq = fmaf(qq[i], qq[i], sq);
        }
      }
      float fk = 1.f, fq = 1.f;
      sk = wave_sum(sk);
      if (DELTA) {
        fk = 1.0f / sqrtf(sk + di.unit_eps);
        fq = di.q_scale / sqrtf(wave_sum(sq) + di.unit_eps);
      }
      if (lane == 0)
        bs[tt] = DELTA ? 1.0f / (1.0f + expf(-ldf((const EB*)di.b + t * di.b_ld + h))) : sk;
#pragma unroll
      for (int i = 0; i < PL; i++) {
        const int r = lane + 64 * i;
        if (r < DP) {
          Ks[(size_t)tt * DP + r] = kk[i] * fk;
          Qs[(size_t)tt * DP + r] = qq[i] * fq;
          Gs[(size_t)tt * DP + r] = gg[i];
        }
      }
    }
    for (int i = threadIdx.x; i < nc * 64; i += blockDim.x) {
      const int tt = i >> 6, cc = p0 + (i & 63);
      vs[i] = cc < dv ? ldf(v + (int64_t)(t0 + c0 + tt) * v_ld + (int64_t)h * dv + cc) : 0.f;
    }
    __syncthreads();
    for (int tt = 0; tt < nc; tt++) {
      const float4* k4 = (const float4*)(Ks + (size_t)tt * DP);
      const float4* q4 = (const float4*)(Qs + (size_t)tt * DP);
      const float4* g4 = (const float4*)(Gs + (size_t)tt * DP);
      const float vv = vs[tt * 64 + 16 * wv + col], be = bs[tt];
      float u = vv, o0 = 0.f, o1 = 0.f;
      if (DELTA) {
        float a0 = 0.f, a1 = 0.f;
#pragma unroll
        for (int j = 0; j < NC4; j++) {
          const float4 kv = k4[4 * j + rg], gv = g4[4 * j + rg];
          st[4 * j] *= gv.x;
          st[4 * j + 1] *= gv.y;
          st[4 * j + 2] *= gv.z;
          st[4 * j + 3] *= gv.w;
          a0 = fmaf(st[4 * j], kv.x, a0);
          a1 = fmaf(st[4 * j + 1], kv.y, a1);
          a0 = fmaf(st[4 * j + 2], kv.z, a0);
          a1 = fmaf(st[4 * j + 3], kv.w, a1);
        }
        float acc = a0 + a1;
        acc += __shfl_xor(acc, 16, 64);
        acc += __shfl_xor(acc, 32, 64);
        u = be * (vv - acc);
      }
#pragma unroll
      for (int j = 0; j < NC4; j++) {
        const float4 kv = k4[4 * j + rg], qv = q4[4 * j + rg];
        if (DELTA) {
          st[4 * j] = fmaf(kv.x, u, st[4 * j]);
          st[4 * j + 1] = fmaf(kv.y, u, st[4 * j + 1]);
          st[4 * j + 2] = fmaf(kv.z, u, st[4 * j + 2]);
          st[4 * j + 3] = fmaf(kv.w, u, st[4 * j + 3]);
        }
        o0 = fmaf(st[4 * j], qv.x, o0);
        o1 = fmaf(st[4 * j + 1], qv.y, o1);
        o0 = fmaf(st[4 * j + 2], qv.z, o0);
        o1 = fmaf(st[4 * j + 3], qv.w, o1);
        if (!DELTA) {
          const float4 gv = g4[4 * j + rg];
          st[4 * j] = fmaf(kv.x, u, gv.x * st[4 * j]);
          st[4 * j + 1] = fmaf(kv.y, u, gv.y * st[4 * j + 1]);
          st[4 * j + 2] = fmaf(kv.z, u, gv.z * st[4 * j + 2]);
          st[4 * j + 3] = fmaf(kv.w, u, gv.w * st[4 * j + 3]);
        }
      }
      float o = o0 + o1;
      o += __shfl_xor(o, 16, 64);
      o += __shfl_xor(o, 32, 64);
      if (!DELTA) o = fmaf(be, vv, o);
      if (rg == 0 && pc < dv) out[((int64_t)(t0 + c0 + tt) * H + h) * dv + pc] = o;
    }
  }
#pragma unroll
  for (int j = 0; j < NC4; j++)
#pragma unroll
    for (int i = 0; i < 4; i++) {
      const int r = 4 * (4 * j + rg) + i;
      if (r < d && pc < dv) Sg[(int64_t)r * dv + pc] = st[4 * j + i];
    }
}

template <typename EQ, typename EB, bool DELTA>
void launch(const EQ* q, int64_t q_ld, const EQ* k, int64_t k_ld, const EQ* v, int64_t v_ld, const float* gd,
            const float* bonus, DeltaIn di, float* S, const int32_t* cu, const int32_t* slots, const int64_t* pos, float* out,
            int B, int H, int K, int d, int dv, hipStream_t st) {
  if (B <= 0 || d > sx::kScanMaxDim) return;                        // (sizes are refused by the caller beforehand)
  int nc4 = 1;
  while (16 * nc4 < d) nc4 *= 2;
  const int DP = 16 * nc4;
  const size_t per_tok = ((size_t)3 * DP + 64 + 1) * sizeof(float);
  int TC = (int)((40 * 1024) / per_tok);
  TC = TC > 32 ? 32 : (TC < 1 ? 1 : TC);
  const int cols = dv < 64 ? dv : 64;
  const dim3 grid(B, H, (dv + 63) / 64), block(64 * ((cols + 15) / 16));
#define CX_SCAN(N)                                                                                                        \
  chan_scan_k<EQ, EB, N, DELTA><<<grid, block, per_tok * TC, st>>>(q, q_ld, k, k_ld, v, v_ld, gd, bonus, di, S, cu, slots, \
                                                                   pos, out, H, K, d, dv, TC)
  switch (nc4) {
    case 1: CX_SCAN(1); break;
    case 2: CX_SCAN(2); break;
    case 4: CX_SCAN(4); break;
    case 8: CX_SCAN(8); break;
    case 16: CX_SCAN(16); break;
    default: CX_SCAN(32);
  }
#undef CX_SCAN
}

}  // namespace

void delta_scan(bool bf16, const float* q, int64_t q_ld, const float* k, int64_t k_ld, const float* v, int64_t v_ld,
                const float* g, DeltaIn di, float* S, const int32_t* cu, const int32_t* slots, const int64_t* pos,
                float* out, int B, int H, int K, int d, int dv, hipStream_t st) {
  if (bf16)
    launch<float, __bf16, true>(q, q_ld, k, k_ld, v, v_ld, g, nullptr, di, S, cu, slots, pos, out, B, H, K, d, dv, st);
  else
    launch<float, float, true>(q, q_ld, k, k_ld, v, v_ld, g, nullptr, di, S, cu, slots, pos, out, B, H, K, d, dv, st);
}

void bonus_scan(bool bf16, const void* r, int64_t r_ld, const void* k, int64_t k_ld, const void* v, int64_t v_ld,
                const float* g, const float* u, float* S, const int32_t* cu, const int32_t* slots, const int64_t* pos,
                float* out, int B, int H, int d, int dv, hipStream_t st) {
  const DeltaIn none{};
  if (bf16)
    launch<__bf16, __bf16, false>((const __bf16*)r, r_ld, (const __bf16*)k, k_ld, (const __bf16*)v, v_ld, g, u, none, S, cu,
                                  slots, pos, out, B, H, H, d, dv, st);
  else
    launch<float, float, false>((const float*)r, r_ld, (const float*)k, k_ld, (const float*)v, v_ld, g, u, none, S, cu,
                                slots, pos, out, B, H, H, d, dv, st);
}

}  // namespace cx
}  // namespace illm
