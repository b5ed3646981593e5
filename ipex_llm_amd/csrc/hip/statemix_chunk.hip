// Matrix-state recurrences of long portions, chunk by chunk of 64 tokens
// (gfx950, wave64, 16x16x4 f32 MFMA: the products keep f32 operands).
//
// With G_t = sum_(s <= t) log g_s counted from the chunk's start and S_0 the
// state in front of it,
//
//   S_t = e^(G_t) S_0 + sum_(s <= t) e^(G_t - G_s) k_s u_s^T
//   o_t = e^(G_t) S_0^T q_t + sum_(s <= t) e^(G_t - G_s) (q_t . k_s) u_s
//
// where u_s = v_s for a fixed decay, and for the delta rule
//
//   u_t = beta_t (v_t - e^(G_t) S_0^T k_t - sum_(s < t) e^(G_t - G_s) (k_t . k_s) u_s)
//
// i.e. (I + A) U = diag(beta) V - diag(beta e^G) K S_0 with A strictly lower
// triangular.  Three launches:
//
//   prepare   a workgroup per (chunk, head): unit norms / SiLU, the factors, the
//             two 64 x 64 products, and by forward substitution (a thread per
//             column, its 64 values in registers)  W = (I + A)^-1 diag(beta e^G) K
//             and  U = (I + A)^-1 diag(beta) V
//   chain     a workgroup per (sequence, head, 16 value columns), chunk after
//             chunk: U <- U - W S, S <- e^(G_last) S + (e^(G_last - G) K)^T U; leaves
//             every chunk's start state
//   read out  a workgroup per (chunk, head, 64 value columns): both sums of o
//
// The differences G_t - G_s are formed in f64.  The chain and the read-out are in
// statemix_chunk.cuh.
#include "statemix_chunk.cuh"

namespace illm {
namespace sx {
namespace {

template <typename EQ, typename EA, int ND, bool DELTA>
__global__ void __launch_bounds__(256) chunk_prepare_k(const EQ* __restrict__ q, int64_t q_ld, const EQ* __restrict__ k,
                                                      int64_t k_ld, const EQ* __restrict__ v, int64_t v_ld,
                                                      const float* __restrict__ decay, DeltaArgs da,
                                                      const int32_t* __restrict__ cu, int B, int seg0, int seg, Scratch sc,
                                                      int H, int K, int d, int dv, int DV) {
  constexpr int DP = 16 * ND, LD = DP + 4, LA = C + 4;
  extern __shared__ __align__(16) float sm[];
  float* Ks = sm;                                                   // [C][LD]
  float* Qs = Ks + C * LD;                                          // [C][LD]
  float* As = Qs + C * LD;                                          // [C][LA]
  __shared__ double Gs[C];
  __shared__ float bet[C], gam[C], kf[C], pw[C + 1];
  int b, c;
  if (!find_chunk(cu, B, seg0, seg, blockIdx.x, &b, &c)) return;
  const int h = blockIdx.y, kh = h / (H / K);
  const int tid = threadIdx.x, lane = tid & 63, wv = tid >> 6, r16 = lane & 15, g = lane >> 4;
  const int nt = min(C, seg_tokens(cu, b, seg0, seg) - c * C);
  const int64_t t0 = (int64_t)cu[b] + seg0 + (int64_t)c * C;
  const int64_t at = (int64_t)blockIdx.x * H + h;
  // keys and queries: a wave per token
  for (int tt = wv; tt < C; tt += 4) {
    constexpr int PL = (DP + 63) / 64;
    float kk[PL], qq[PL];
    float sk = 0.f, sq = 0.f;
#pragma unroll
    for (int i = 0; i < PL; i++) {
      const int r = lane + 64 * i;
      kk[i] = qq[i] = 0.f;
      if (tt < nt && r < d) {
        kk[i] = ldf(k + (t0 + tt) * k_ld + (int64_t)kh * d + r);
        qq[i] = ldf(q + (t0 + tt) * q_ld + (int64_t)kh * d + r);
      }
      if (DELTA) {
        sk = fmaf(kk[i], kk[i], sk);
        sq = fmaf(qq[i], qq[i], sq);
      } else {
        kk[i] = silu(kk[i]);
        qq[i] = silu(qq[i]);
      }
    }
    float fk = 1.f, fq = 1.f;
    if (DELTA) {
      fk = 1.0f / sqrtf(wave_sum(sk) + da.unit_eps);
      fq = da.q_scale / sqrtf(wave_sum(sq) + da.unit_eps);
    }
#pragma unroll
    for (int i = 0; i < PL; i++) {
      const int r = lane + 64 * i;
      if (r < DP) {
        Ks[tt * LD + r] = kk[i] * fk;
        Qs[tt * LD + r] = qq[i] * fq;
      }
    }
  }
  if (wv == 0) {                                                    // lane = token: the factors
    if (DELTA) {
      double G = 0.0;
      float be = 0.f;
      if (lane < nt) {
        const int64_t t = t0 + lane;
        G = (double)(-da.rate[h] * softplusf(ldf((const EA*)da.a + t * da.a_ld + h) + da.dt_bias[h]));
        be = sigmoidf(ldf((const EA*)da.b + t * da.b_ld + h));
      }
#pragma unroll
      for (int o = 1; o < 64; o <<= 1) {
        const double up = __shfl_up(G, o, 64);
        if (lane >= o) G += up;
      }
      Gs[lane] = G;
      bet[lane] = be;
      gam[lane] = expf((float)G);
      kf[lane] = expf((float)(__shfl(G, 63, 64) - G));              // padded tokens add nothing to G
    } else {
      const float dec = decay[h];
      pw[lane] = powf(dec, (float)lane);
      if (lane == 0) pw[C] = powf(dec, (float)C);
    }
  }
  __syncthreads();
  if (!DELTA) {
    if (tid < C) {
      gam[tid] = pw[tid + 1];
      kf[tid] = tid < nt ? pw[nt - 1 - tid] : 0.f;
    }
    __syncthreads();
  }
  if (tid == 0) sc.gc[at] = DELTA ? gam[C - 1] : pw[nt];
  // the 64 x 64 products: wave wv owns rows 16 wv .. 16 wv + 15, tiles on and below the diagonal
  {
    f32x4 ka[ND], qa[ND];
#pragma unroll
    for (int j = 0; j < ND; j++) {
      ka[j] = ld4(Ks + (16 * wv + r16) * LD + 16 * j + 4 * g);
      qa[j] = ld4(Qs + (16 * wv + r16) * LD + 16 * j + 4 * g);
    }
    float* P = sc.p + at * C * C;
    for (int n = 0; n <= wv; n++) {
      f32x4 kk = {0.f, 0.f, 0.f, 0.f}, qk = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int j = 0; j < ND; j++) {
        const f32x4 kb = ld4(Ks + (16 * n + r16) * LD + 16 * j + 4 * g);
        if (DELTA) kk = mfma4(ka[j], kb, kk);
        qk = mfma4(qa[j], kb, qk);
      }
      const int s = 16 * n + r16;
#pragma unroll
      for (int i = 0; i < 4; i++) {
        const int t = 16 * wv + 4 * g + i;
        float f = 0.f;
        if (t >= s) f = DELTA ? expf((float)(Gs[t] - Gs[s])) : pw[t - s];
        P[t * C + s] = f * qk[i];
        if (DELTA) As[t * LA + s] = t > s ? bet[t] * f * kk[i] : 0.f;
      }
    }
  }
  for (int i = tid; i < C * DP; i += 256) {
    const int t = i / DP, r = i - t * DP;
    sc.gq[at * C * DP + i] = gam[t] * Qs[t * LD + r];
  }
  for (int i = tid; i < C * DP; i += 256) {
    const int r = i / C, s = i - r * C;
    sc.kd[at * C * DP + i] = kf[s] * Ks[s * LD + r];
  }
  __syncthreads();
  // columns: W's DP (delta rule only), then U's DV
  const int cw = DELTA ? DP : 0;
  for (int col = tid; col < cw + DV; col += 256) {
    const bool isw = col < cw;
    const int cc = isw ? col : col - cw;
    float x[C];
#pragma unroll
    for (int t = 0; t < C; t++) {
      if (isw) {
        x[t] = bet[t] * gam[t] * Ks[t * LD + cc];
      } else {
        float val = (t < nt && cc < dv) ? ldf(v + (t0 + t) * v_ld + (int64_t)h * dv + cc) : 0.f;
        x[t] = DELTA ? bet[t] * val : silu(val);
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

template <typename EQ, typename EA, int ND, bool DELTA>
void run(const EQ* q, int64_t q_ld, const EQ* k, int64_t k_ld, const EQ* v, int64_t v_ld, const float* decay, DeltaArgs da,
         float* S, const int32_t* cu, const int32_t* slots, const int64_t* pos, float* out, float* scratch, int B, int nch,
         int seg0, int seg, int H, int K, int d, int dv, hipStream_t st) {
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
  const size_t lds = ((size_t)2 * C * (DP + 4) + (DELTA ? C * (C + 4) : 0)) * sizeof(float);
  if (lds > 48 * 1024)
    (void)hipFuncSetAttribute((const void*)chunk_prepare_k<EQ, EA, ND, DELTA>, hipFuncAttributeMaxDynamicSharedMemorySize,
                              (int)lds);
  chunk_prepare_k<EQ, EA, ND, DELTA><<<dim3(nch, H), 256, lds, st>>>(q, q_ld, k, k_ld, v, v_ld, decay, da, cu, B, seg0, seg,
                                                                     sc, H, K, d, dv, DV);
  chunk_chain_k<ND, DELTA, false><<<dim3(DV / 16, H, B), 256, 0, st>>>(S, cu, slots, pos, seg0, seg, sc, H, d, dv, DV);
  chunk_read_k<ND><<<dim3(nch, H, (DV + 63) / 64), 256, 0, st>>>(cu, B, seg0, seg, sc, out, H, dv, DV);
}

template <typename EQ, typename EA, bool DELTA>
void pick(const EQ* q, int64_t q_ld, const EQ* k, int64_t k_ld, const EQ* v, int64_t v_ld, const float* decay, DeltaArgs da,
          float* S, const int32_t* cu, const int32_t* slots, const int64_t* pos, float* out, float* scratch, int B, int nch,
          int seg0, int seg, int H, int K, int d, int dv, hipStream_t st) {
#define SX_ND(N) \
  run<EQ, EA, N, DELTA>(q, q_ld, k, k_ld, v, v_ld, decay, da, S, cu, slots, pos, out, scratch, B, nch, seg0, seg, H, K, d, dv, st)
  if (d <= 16) SX_ND(1);
  else if (d <= 32) SX_ND(2);
  else if (d <= 64) SX_ND(4);
  else if (d <= kChunkMaxDim) SX_ND(8);                             // (larger ones are refused by the caller beforehand)
#undef SX_ND
}

}  // namespace

int64_t chunk_scratch_floats(bool delta, int64_t nch, int H, int d, int dv) {
  const int64_t DP = d <= 16 ? 16 : (d <= 32 ? 32 : (d <= 64 ? 64 : 128)), DV = (dv + 15) / 16 * 16;
  return nch * H * ((delta ? 3 : 2) * C * DP + C * C + DV * C + DV * DP + 1);
}

void decay_chunks(bool bf16, const void* q, int64_t q_ld, const void* k, int64_t k_ld, const void* v, int64_t v_ld,
                  const float* decay, float* S, const int32_t* cu, const int32_t* slots, const int64_t* pos, float* out,
                  float* scratch, int B, int nch, int seg0, int seg, int H, int d, int dv, hipStream_t st) {
  const DeltaArgs none{};
  if (bf16)
    pick<__bf16, __bf16, false>((const __bf16*)q, q_ld, (const __bf16*)k, k_ld, (const __bf16*)v, v_ld, decay, none, S, cu,
                                slots, pos, out, scratch, B, nch, seg0, seg, H, H, d, dv, st);
  else
    pick<float, float, false>((const float*)q, q_ld, (const float*)k, k_ld, (const float*)v, v_ld, decay, none, S, cu,
                              slots, pos, out, scratch, B, nch, seg0, seg, H, H, d, dv, st);
}

void delta_chunks(bool bf16, const float* q, int64_t q_ld, const float* k, int64_t k_ld, const float* v, int64_t v_ld,
                  DeltaArgs da, float* S, const int32_t* cu, const int32_t* slots, const int64_t* pos, float* out,
                  float* scratch, int B, int nch, int seg0, int seg, int H, int K, int d, int dv, hipStream_t st) {
  if (bf16)
    pick<float, __bf16, true>(q, q_ld, k, k_ld, v, v_ld, nullptr, da, S, cu, slots, pos, out, scratch, B, nch, seg0, seg, H,
                              K, d, dv, st);
  else
    pick<float, float, true>(q, q_ld, k, k_ld, v, v_ld, nullptr, da, S, cu, slots, pos, out, scratch, B, nch, seg0, seg, H,
                             K, d, dv, st);
}

}  // namespace sx
}  // namespace illm
