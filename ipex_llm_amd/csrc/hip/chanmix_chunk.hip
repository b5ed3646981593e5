// Matrix-state recurrences with one decay per key channel, chunk by chunk of 64
// tokens (gfx950, wave64, 16x16x4 f32 MFMA: the products keep f32 operands).
//
// With D(s, t) the diagonal matrix of the products of the decays of the tokens
// s + 1 .. t and S_0 the state in front of the chunk (tokens counted from 0),
//
//   delta rule   u_t = beta_t (v_t - k_t^T D(-1, t) S_0 - sum_(s < t) (k_t^T D(s, t) k_s) u_s)
//                o_t = q_t^T D(-1, t) S_0 + sum_(s <= t) (q_t^T D(s, t) k_s) u_s
//   with bonus   o_t = r_t^T D(-1, t - 1) S_0 + sum_(s < t) (r_t^T D(s, t - 1) k_s) v_s + (r_t^T diag(u) k_t) v_t
//
// and S_end = D(-1, 63) S_0 + sum_s D(s, 63) k_s u_s^T.  As a decay per channel does
// not leave the scalar products, they are formed with scaled vectors: a chunk is
// four blocks of 16 tokens, and every factor below is a product of decays of
// neighbouring tokens, at most 1 (no logarithms, no differences of sums):
//
//   same block         a wave per block walks its 16 tokens; lane = (s, one of four
//                      groups of channels) carries k_s times the decays since s and
//                      forms the products with the token's key and query.  What is
//                      left at the block's end is k_s D(s, end); the running product
//                      from the block's start scales the token's own key and query
//   block i, block j   (scaled rows of i) (k_s D(s, end of j) B_(j+1) .. B_(i-1))^T on
//                      the matrix cores, B_m a block's whole product
//
// Then, as with one decay per head (statemix_chunk.hip): the unit lower-triangular
// system of the delta rule by forward substitution, the chain over the chunks and
// the read-out (statemix_chunk.cuh).
#include "chanmix.h"
#include "statemix_chunk.cuh"

namespace illm {
namespace cx {
namespace {

using namespace sx;

// DELTA: q is the query; otherwise q is the receptance and ``bonus`` [H, d] holds u
template <typename EQ, typename EB, int ND, bool DELTA>
__global__ void __launch_bounds__(256) chan_prepare_k(const EQ* __restrict__ q, int64_t q_ld, const EQ* __restrict__ k,
                                                     int64_t k_ld, const EQ* __restrict__ v, int64_t v_ld,
                                                     const float* __restrict__ gd, const float* __restrict__ bonus,
                                                     DeltaIn di, const int32_t* __restrict__ cu, int B, int seg0, int seg,
                                                     Scratch sc, int H, int K, int d, int dv, int DV) {
  constexpr int DP = 16 * ND, LD = DP + 4, LA = C + 4;
  extern __shared__ __align__(16) float sm[];
  float* Ks = sm;                                                   // [C][LD] keys, then times the decays from the block's start
  float* Qs = Ks + C * LD;                                          // [C][LD] queries, likewise
  float* Gs = Qs + C * LD;                                          // [C][LD] decays, then keys times the decays to the block's end
  float* Bp = Gs + C * LD;                                          // [4][DP] products of whole blocks
  float* bet = Bp + 4 * DP;                                         // [C]
  float* As = bet + C;                                              // [C][LA] (delta rule only)
  int b, c;
  if (!find_chunk(cu, B, seg0, seg, blockIdx.x, &b, &c)) return;
  const int h = blockIdx.y, kh = h / (H / K);
  const int tid = threadIdx.x, lane = tid & 63, wv = tid >> 6, r16 = lane & 15, g = lane >> 4;
  const int nt = min(C, seg_tokens(cu, b, seg0, seg) - c * C);
  const int64_t t0 = (int64_t)cu[b] + seg0 + (int64_t)c * C;
  const int64_t at = (int64_t)blockIdx.x * H + h;
  float* P = sc.p + at * C * C;
  // keys, queries, decays: a wave per token (tokens past the end: zeros and decays of 1)
  for (int tt = wv; tt < C; tt += 4) {
    constexpr int PL = (DP + 63) / 64;
    float kk[PL], qq[PL], gg[PL];
    float sk = 0.f, sq = 0.f;
#pragma unroll
    for (int i = 0; i < PL; i++) {
      const int r = lane + 64 * i;
      kk[i] = qq[i] = 0.f;
      gg[i] = 1.f;
      if (tt < nt && r < d) {
        kk[i] = ldf(k + (t0 + tt) * k_ld + (int64_t)kh * d + r);
        qq[i] = ldf(q + (t0 + tt) * q_ld + (int64_t)kh * d + r);
        gg[i] = gd[((t0 + tt) * H + h) * d + r];
      }
      if (DELTA) {
        sk = fmaf(kk[i], kk[i], sk);
        sq = fmaf(qq[i], qq[i], sq);
      }
    }
    float fk = 1.f, fq = 1.f;
    if (DELTA) {
      fk = 1.0f / sqrtf(wave_sum(sk) + di.unit_eps);
      fq = di.q_scale / sqrtf(wave_sum(sq) + di.unit_eps);
      if (lane == 0) bet[tt] = tt < nt ? sigmoidf(ldf((const EB*)di.b + (t0 + tt) * di.b_ld + h)) : 0.f;
    }
#pragma unroll
    for (int i = 0; i < PL; i++) {
      const int r = lane + 64 * i;
      if (r < DP) {
        Ks[tt * LD + r] = kk[i] * fk;
        Qs[tt * LD + r] = qq[i] * fq;
        Gs[tt * LD + r] = gg[i];
      }
    }
  }
  __syncthreads();
  // products inside a block: wave = block, lane = (token s, channels 16 j + 4 g + i)
  {
    f32x4 w[ND], run[ND], bo[ND];
#pragma unroll
    for (int j = 0; j < ND; j++) {
      w[j] = f32x4{0.f, 0.f, 0.f, 0.f};
      run[j] = f32x4{1.f, 1.f, 1.f, 1.f};
#pragma unroll
      for (int i = 0; i < 4; i++) {
        const int r = 16 * j + 4 * g + i;
        bo[j][i] = !DELTA && r < d ? bonus[(int64_t)h * d + r] : 0.f;
      }
    }
    for (int tt = 0; tt < 16; tt++) {
      const int t = 16 * wv + tt;
      float* kr = Ks + t * LD + 4 * g;
      float* qr = Qs + t * LD + 4 * g;
      const float* gr = Gs + t * LD + 4 * g;
      float kd = 0.f, qd = 0.f;
      f32x4 kt[ND], qt[ND];
#pragma unroll
      for (int j = 0; j < ND; j++) {
        const f32x4 gt = ld4(gr + 16 * j);
        kt[j] = ld4(kr + 16 * j);
        qt[j] = ld4(qr + 16 * j);
        if (DELTA) {
#pragma unroll
          for (int i = 0; i < 4; i++) {
            w[j][i] *= gt[i];                                       // (zero until token s itself has come)
            kd = fmaf(kt[j][i], w[j][i], kd);
            if (r16 == tt) w[j][i] = kt[j][i];
            qd = fmaf(qt[j][i], w[j][i], qd);
            run[j][i] *= gt[i];
            kt[j][i] *= run[j][i];
            qt[j][i] *= run[j][i];
          }
        } else {
#pragma unroll
          for (int i = 0; i < 4; i++) {
            const bool own = r16 == tt;
            qd = fmaf(qt[j][i], own ? bo[j][i] * kt[j][i] : w[j][i], qd);
            w[j][i] = own ? kt[j][i] : w[j][i] * gt[i];
            qt[j][i] *= run[j][i];
            run[j][i] *= gt[i];
          }
        }
      }
      kd += __shfl_xor(kd, 16, 64);
      kd += __shfl_xor(kd, 32, 64);
      qd += __shfl_xor(qd, 16, 64);
      qd += __shfl_xor(qd, 32, 64);
      if (g == 0) {
        P[t * C + 16 * wv + r16] = r16 <= tt ? qd : 0.f;
        if (DELTA) As[t * LA + 16 * wv + r16] = r16 < tt ? bet[t] * kd : 0.f;
      }
      if (r16 == tt) {                                              // every lane of the wave has read the token's rows
#pragma unroll
        for (int j = 0; j < ND; j++) {
          if (DELTA) st4(kr + 16 * j, kt[j]);
          st4(qr + 16 * j, qt[j]);
        }
      }
    }
#pragma unroll
    for (int j = 0; j < ND; j++) {
      st4(Gs + (16 * wv + r16) * LD + 16 * j + 4 * g, w[j]);
      if (r16 == 0) st4(Bp + wv * DP + 16 * j + 4 * g, run[j]);
    }
  }
  __syncthreads();
  // products between blocks: wave wv owns rows 16 wv .. 16 wv + 15
  {
    f32x4 ka[ND], qa[ND], btw[ND];
#pragma unroll
    for (int j = 0; j < ND; j++) {
      if (DELTA) ka[j] = ld4(Ks + (16 * wv + r16) * LD + 16 * j + 4 * g);
      qa[j] = ld4(Qs + (16 * wv + r16) * LD + 16 * j + 4 * g);
      btw[j] = f32x4{1.f, 1.f, 1.f, 1.f};
    }
    for (int n = wv - 1; n >= 0; n--) {
      f32x4 kk = {0.f, 0.f, 0.f, 0.f}, qk = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int j = 0; j < ND; j++) {
        f32x4 kb = ld4(Gs + (16 * n + r16) * LD + 16 * j + 4 * g);
        const f32x4 bp = ld4(Bp + n * DP + 16 * j + 4 * g);
#pragma unroll
        for (int i = 0; i < 4; i++) {
          kb[i] *= btw[j][i];
          btw[j][i] *= bp[i];
        }
        if (DELTA) kk = mfma4(ka[j], kb, kk);
        qk = mfma4(qa[j], kb, qk);
      }
      const int s = 16 * n + r16;
#pragma unroll
      for (int i = 0; i < 4; i++) {
        const int t = 16 * wv + 4 * g + i;
        P[t * C + s] = qk[i];
        if (DELTA) As[t * LA + s] = bet[t] * kk[i];
      }
    }
  }
  // scaled to the chunk's start (queries, and the rows of W) and to its end (keys)
  for (int i = tid; i < C * DP; i += 256) {
    const int t = i / DP, r = i - t * DP;
    float f = 1.f;
    for (int m = 0; m < t / 16; m++) f *= Bp[m * DP + r];
    sc.gq[at * C * DP + i] = f * Qs[t * LD + r];
  }
  for (int i = tid; i < C * DP; i += 256) {
    const int r = i / C, s = i - r * C;
    float f = 1.f;
    for (int m = 3; m > s / 16; m--) f *= Bp[m * DP + r];
    sc.kd[at * C * DP + i] = f * Gs[s * LD + r];
  }
  for (int r = tid; r < DP; r += 256) sc.gc[at * DP + r] = Bp[r] * Bp[DP + r] * Bp[2 * DP + r] * Bp[3 * DP + r];
  if (DELTA) __syncthreads();
  // columns: W's DP (delta rule only), then U's DV
  const int cw = DELTA ? DP : 0;
  for (int col = tid; col < cw + DV; col += 256) {
    const bool isw = col < cw;
    const int cc = isw ? col : col - cw;
    float x[C];
    float f[4] = {1.f, 1.f, 1.f, 1.f};
    if (isw) {
      f[1] = Bp[cc];
      f[2] = f[1] * Bp[DP + cc];
      f[3] = f[2] * Bp[2 * DP + cc];
    }
#pragma unroll
    for (int t = 0; t < C; t++) {
      if (isw) {
        x[t] = bet[t] * f[t / 16] * Ks[t * LD + cc];
      } else {
        const float val = (t < nt && cc < dv) ? ldf(v + (t0 + t) * v_ld + (int64_t)h * dv + cc) : 0.f;
        x[t] = DELTA ? bet[t] * val : val;
      }
    }
    if (DELTA) solve_unit_lower(As, LA, x);
    if (isw) {
      float* w = sc.w + at * C * DP + cc;
#pragma unroll
      for (int t = 0; t < C; t++) w[t * DP] = x[t];
    } else {
      float* u = sc.u + (at * DV + cc) * C;
#pragma unroll
      for (int t = 0; t < C; t += 4) st4(u + t, f32x4{x[t], x[t + 1], x[t + 2], x[t + 3]});
    }
  }
}

template <typename EQ, typename EB, int ND, bool DELTA>
void run(const EQ* q, int64_t q_ld, const EQ* k, int64_t k_ld, const EQ* v, int64_t v_ld, const float* gd,
         const float* bonus, DeltaIn di, float* S, const int32_t* cu, const int32_t* slots, const int64_t* pos, float* out,
         float* scratch, int B, int nch, int seg0, int seg, int H, int K, int d, int dv, hipStream_t st) {
  constexpr int DP = 16 * ND;
  const int DV = (dv + 15) / 16 * 16;
  const int64_t n = (int64_t)nch * H;
  Scratch sc;
  sc.w = scratch;
  sc.gq = sc.w + (DELTA ? n * C * DP : 0);
  sc.kd = sc.gq + n * C * DP;
  sc.p = sc.kd + n * C * DP;
  sc.u = sc.p + n * C * C;
  sc.s0 = sc.u + n * DV * C;
  sc.gc = sc.s0 + n * DV * DP;
  const size_t lds = ((size_t)3 * C * (DP + 4) + 4 * DP + C + (DELTA ? C * (C + 4) : 0)) * sizeof(float);
  if (lds > 48 * 1024)
    (void)hipFuncSetAttribute((const void*)chan_prepare_k<EQ, EB, ND, DELTA>, hipFuncAttributeMaxDynamicSharedMemorySize,
                              (int)lds);
  chan_prepare_k<EQ, EB, ND, DELTA><<<dim3(nch, H), 256, lds, st>>>(q, q_ld, k, k_ld, v, v_ld, gd, bonus, di, cu, B, seg0,
                                                                    seg, sc, H, K, d, dv, DV);
  chunk_chain_k<ND, DELTA, true><<<dim3(DV / 16, H, B), 256, 0, st>>>(S, cu, slots, pos, seg0, seg, sc, H, d, dv, DV);
  chunk_read_k<ND><<<dim3(nch, H, (DV + 63) / 64), 256, 0, st>>>(cu, B, seg0, seg, sc, out, H, dv, DV);
}

template <typename EQ, typename EB, bool DELTA>
void pick(const EQ* q, int64_t q_ld, const EQ* k, int64_t k_ld, const EQ* v, int64_t v_ld, const float* gd,
          const float* bonus, DeltaIn di, float* S, const int32_t* cu, const int32_t* slots, const int64_t* pos, float* out,
          float* scratch, int B, int nch, int seg0, int seg, int H, int K, int d, int dv, hipStream_t st) {
#define CX_ND(N)                                                                                                         \
  run<EQ, EB, N, DELTA>(q, q_ld, k, k_ld, v, v_ld, gd, bonus, di, S, cu, slots, pos, out, scratch, B, nch, seg0, seg, H, \
                        K, d, dv, st)
  if (d <= 16) CX_ND(1);
  else if (d <= 32) CX_ND(2);
  else if (d <= 64) CX_ND(4);
  else if (d <= kChunkMaxDim) CX_ND(8);                             // (larger ones are refused by the caller beforehand)
#undef CX_ND
}

}  // namespace

int64_t chunk_scratch_floats(bool delta, int64_t nch, int H, int d, int dv) {
  const int64_t DP = d <= 16 ? 16 : (d <= 32 ? 32 : (d <= 64 ? 64 : 128)), DV = (dv + 15) / 16 * 16;
  return nch * H * ((delta ? 3 : 2) * C * DP + C * C + DV * C + DV * DP + DP);
}

void delta_chunks(bool bf16, const float* q, int64_t q_ld, const float* k, int64_t k_ld, const float* v, int64_t v_ld,
                  const float* g, DeltaIn di, float* S, const int32_t* cu, const int32_t* slots, const int64_t* pos,
                  float* out, float* scratch, int B, int nch, int seg0, int seg, int H, int K, int d, int dv,
                  hipStream_t st) {
  if (bf16)
    pick<float, __bf16, true>(q, q_ld, k, k_ld, v, v_ld, g, nullptr, di, S, cu, slots, pos, out, scratch, B, nch, seg0, seg,
                              H, K, d, dv, st);
  else
    pick<float, float, true>(q, q_ld, k, k_ld, v, v_ld, g, nullptr, di, S, cu, slots, pos, out, scratch, B, nch, seg0, seg,
                             H, K, d, dv, st);
}

void bonus_chunks(bool bf16, const void* r, int64_t r_ld, const void* k, int64_t k_ld, const void* v, int64_t v_ld,
                  const float* g, const float* u, float* S, const int32_t* cu, const int32_t* slots, const int64_t* pos,
                  float* out, float* scratch, int B, int nch, int seg0, int seg, int H, int d, int dv, hipStream_t st) {
  const DeltaIn none{};
  if (bf16)
    pick<__bf16, __bf16, false>((const __bf16*)r, r_ld, (const __bf16*)k, k_ld, (const __bf16*)v, v_ld, g, u, none, S, cu,
                                slots, pos, out, scratch, B, nch, seg0, seg, H, H, d, dv, st);
  else
    pick<float, float, false>((const float*)r, r_ld, (const float*)k, k_ld, (const float*)v, v_ld, g, u, none, S, cu, slots,
                              pos, out, scratch, B, nch, seg0, seg, H, H, d, dv, st);
}

}  // namespace cx
}  // namespace illm
