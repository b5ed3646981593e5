// Recurrences of the matrix-state and gated-linear mixers (gfx950, wave64).
//
//   matrix-state scan  lightning attention  S' = decay S + k v^T, o = S'^T q and
//                      the gated delta rule S <- g S, S <- S + k u^T with
//                      u = beta (v - S^T k), o = S^T q.  The value columns of a
//                      state never meet, so a wave owns 16 columns of one
//                      (sequence, head): lane = (column, one of four row
//                      groups), the state rows in registers, a row group's keys
//                      and queries read from LDS as 16-byte pieces; the sums over
//                      the rows end with two shuffles.  Tokens go through LDS in
//                      chunks (SiLU, unit norms, decays and step sizes formed
//                      while staging)
//   gates of the LRU   block-diagonal products on the matrix cores; with 16-bit
//                      weights the f32 inputs are split into three 16-bit parts
//                      (hi + mid + lo is the f32 number), so the sums carry f32
//                      precision
//   LRU scan           S' = a S + x per channel: up to 64 pieces of a portion
//                      folded side by side, their carries chained in order, then
//                      run again
//
// Activations are bf16 or f32 (template E); accumulation is always f32.
#include "split_tile.h"
#include "statemix.h"

#include <math.h>

namespace illm {
namespace sx {
namespace {

template <typename E> __device__ __forceinline__ float ldf(const E* p);
template <> __device__ __forceinline__ float ldf<float>(const float* p) { return *p; }
template <> __device__ __forceinline__ float ldf<__bf16>(const __bf16* p) { return (float)*p; }
template <typename E> __device__ __forceinline__ void stf(E* p, float v);
template <> __device__ __forceinline__ void stf<float>(float* p, float v) { *p = v; }
template <> __device__ __forceinline__ void stf<__bf16>(__bf16* p, float v) { *p = (__bf16)v; }

__device__ __forceinline__ float wave_sum(float v) {
#pragma unroll
  for (int o = 32; o > 0; o >>= 1) v += __shfl_xor(v, o, 64);
  return v;
}
__device__ __forceinline__ float sigmoidf(float z) { return 1.0f / (1.0f + expf(-z)); }
__device__ __forceinline__ float silu(float z) { return z / (1.0f + expf(-z)); }
__device__ __forceinline__ float softplusf(float z) { return z > 20.f ? z : log1pf(expf(z)); }

// ------------------------------------------------------------------ matrix-state scan, token by token
// EQ: type of q / k / v, EA: of the delta rule's a / b.  NC4: 16-row pieces of the state (d <= 16 NC4)
template <typename EQ, typename EA, int NC4, bool DELTA>
__global__ void __launch_bounds__(256) state_scan_k(const EQ* __restrict__ q, int64_t q_ld, const EQ* __restrict__ k,
                                                   int64_t k_ld, const EQ* __restrict__ v, int64_t v_ld,
                                                   const float* __restrict__ decay, DeltaArgs da, float* __restrict__ S,
                                                   const int32_t* __restrict__ cu, const int32_t* __restrict__ slots,
                                                   const int64_t* __restrict__ pos, float* __restrict__ out, int H, int K,
                                                   int d, int dv, int TC) {
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
  float* vs = Qs + (size_t)TC * DP;                                 // [TC][64]
  float* gs = vs + (size_t)TC * 64;                                 // [TC] decays, [TC] step sizes
  float* bs = gs + TC;
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
  float g = DELTA ? 1.f : decay[h], beta = 1.f;
  for (int c0 = 0; c0 < n; c0 += TC) {
    const int nc = min(TC, n - c0);
    __syncthreads();
    // a wave stages whole tokens (their unit norms need the row)
    for (int tt = wv; tt < nc; tt += NW) {
      const int64_t t = t0 + c0 + tt;
      constexpr int PL = (DP + 63) / 64;
      float kk[PL], qq[PL];
      float sk = 0.f, sq = 0.f;
#pragma unroll
      for (int i = 0; i < PL; i++) {
        const int r = lane + 64 * i;
        kk[i] = qq[i] = 0.f;
        if (r < d) {
          kk[i] = ldf(k + t * k_ld + (int64_t)kh * d + r);
          qq[i] = ldf(q + t * q_ld + (int64_t)kh * d + r);
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
          Ks[(size_t)tt * DP + r] = kk[i] * fk;
          Qs[(size_t)tt * DP + r] = qq[i] * fq;
        }
      }
    }
    for (int i = threadIdx.x; i < nc * 64; i += blockDim.x) {
      const int tt = i >> 6, cc = p0 + (i & 63);
      float x = cc < dv ? ldf(v + (int64_t)(t0 + c0 + tt) * v_ld + (int64_t)h * dv + cc) : 0.f;
      vs[i] = DELTA ? x : silu(x);
    }
    if (DELTA)
      for (int tt = threadIdx.x; tt < nc; tt += blockDim.x) {
        const int64_t t = t0 + c0 + tt;
        gs[tt] = expf(-da.rate[h] * softplusf(ldf((const EA*)da.a + t * da.a_ld + h) + da.dt_bias[h]));
        bs[tt] = sigmoidf(ldf((const EA*)da.b + t * da.b_ld + h));
      }
    __syncthreads();
    for (int tt = 0; tt < nc; tt++) {
      const float4* k4 = (const float4*)(Ks + (size_t)tt * DP);
      const float4* q4 = (const float4*)(Qs + (size_t)tt * DP);
      const float vv = vs[tt * 64 + 16 * wv + col];
      float u = vv;
      if (DELTA) {
        g = gs[tt];
        beta = bs[tt];
        float a0 = 0.f, a1 = 0.f;
#pragma unroll
        for (int j = 0; j < NC4; j++) {
          const float4 kv = k4[4 * j + rg];
          a0 = fmaf(st[4 * j], kv.x, a0);
          a1 = fmaf(st[4 * j + 1], kv.y, a1);
          a0 = fmaf(st[4 * j + 2], kv.z, a0);
          a1 = fmaf(st[4 * j + 3], kv.w, a1);
        }
        float acc = a0 + a1;
        acc += __shfl_xor(acc, 16, 64);
        acc += __shfl_xor(acc, 32, 64);
        u = beta * (vv - g * acc);
      }
      float o0 = 0.f, o1 = 0.f;
#pragma unroll
      for (int j = 0; j < NC4; j++) {
        const float4 kv = k4[4 * j + rg], qv = q4[4 * j + rg];
        st[4 * j] = fmaf(kv.x, u, g * st[4 * j]);
        st[4 * j + 1] = fmaf(kv.y, u, g * st[4 * j + 1]);
        st[4 * j + 2] = fmaf(kv.z, u, g * st[4 * j + 2]);
        st[4 * j + 3] = fmaf(kv.w, u, g * st[4 * j + 3]);
        o0 = fmaf(st[4 * j], qv.x, o0);
        o1 = fmaf(st[4 * j + 1], qv.y, o1);
        o0 = fmaf(st[4 * j + 2], qv.z, o0);
        o1 = fmaf(st[4 * j + 3], qv.w, o1);
      }
      float o = o0 + o1;
      o += __shfl_xor(o, 16, 64);
      o += __shfl_xor(o, 32, 64);
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

template <typename EQ, typename EA, bool DELTA>
void launch_scan(const EQ* q, int64_t q_ld, const EQ* k, int64_t k_ld, const EQ* v, int64_t v_ld, const float* decay,
                 DeltaArgs da, float* S, const int32_t* cu, const int32_t* slots, const int64_t* pos, float* out, int B,
                 int H, int K, int d, int dv, hipStream_t st) {
  if (B <= 0 || d > kScanMaxDim) return;                            // (sizes are refused by the caller beforehand)
  int nc4 = 1;
  while (16 * nc4 < d) nc4 *= 2;
  const int DP = 16 * nc4;
  const size_t per_tok = ((size_t)2 * DP + 64 + 2) * sizeof(float);
  int TC = (int)((40 * 1024) / per_tok);
  TC = TC > 32 ? 32 : (TC < 1 ? 1 : TC);
  const size_t lds = per_tok * TC;
  const int cols = dv < 64 ? dv : 64;
  const dim3 grid(B, H, (dv + 63) / 64), block(64 * ((cols + 15) / 16));
#define SX_SCAN(N)                                                                                                       \
  state_scan_k<EQ, EA, N, DELTA><<<grid, block, lds, st>>>(q, q_ld, k, k_ld, v, v_ld, decay, da, S, cu, slots, pos, out, \
                                                           H, K, d, dv, TC)
  switch (nc4) {
    case 1: SX_SCAN(1); break;
    case 2: SX_SCAN(2); break;
    case 4: SX_SCAN(4); break;
    case 8: SX_SCAN(8); break;
    case 16: SX_SCAN(16); break;
    default: SX_SCAN(32);
  }
#undef SX_SCAN
}

// ------------------------------------------------------------------ gates of the linear recurrent unit
// a workgroup: TM tokens x 64 output channels of one block, both gates; wave w owns channels 16 w .. 16 w + 15.
// K goes by 64; inside a step of 32 lane group g holds k = 8 g .. 8 g + 7 (tokens' values and weights alike, so the
// f32 products may take them one after another)
template <typename E, int TM>
__global__ void __launch_bounds__(256) rglru_gates_k(const float* __restrict__ u, const E* __restrict__ w_r,
                                                    const float* __restrict__ b_r, const E* __restrict__ w_i,
                                                    const float* __restrict__ b_i, const float* __restrict__ log_base,
                                                    float* __restrict__ a_out, float* __restrict__ x_out, int T, int nb,
                                                    int n) {
  constexpr int NP = Parts<E>::N, KC = 64, LP = KC + (sizeof(E) == 2 ? 8 : 4), MS = TM / 16;
  __shared__ __attribute__((aligned(16))) E us[NP][TM * LP];
  const int nct = (n + 63) / 64;
  const int blk = blockIdx.y / nct, o0 = (blockIdx.y % nct) * 64;
  const int t0 = blockIdx.x * TM;
  const int C = nb * n;
  const int tid = threadIdx.x, wv = tid >> 6, lane = tid & 63, r16 = lane & 15, g = lane >> 4;
  const int oc = o0 + 16 * wv + r16;
  const bool ok = oc < n;
  const E* wr = w_r + ((int64_t)blk * n + (ok ? oc : 0)) * n;
  const E* wi = w_i + ((int64_t)blk * n + (ok ? oc : 0)) * n;
  const bool vec = n % 8 == 0;
  f32x4 ar[MS], ai[MS];
#pragma unroll
  for (int m = 0; m < MS; m++) ar[m] = ai[m] = f32x4{0.f, 0.f, 0.f, 0.f};
  for (int k0 = 0; k0 < n; k0 += KC) {
    Frag<E> br[KC / 32], bi[KC / 32];                               // requested before the tokens' values are staged
#pragma unroll
    for (int ks = 0; ks < KC / 32; ks++) {
      br[ks].load(wr, k0 + 32 * ks + 8 * g, ok ? n : 0, vec);
      bi[ks].load(wi, k0 + 32 * ks + 8 * g, ok ? n : 0, vec);
    }
    __syncthreads();
    if (vec) {                                                      // rows are 16-byte aligned: four values at a time
      for (int i = tid; i < TM * KC / 4; i += 256) {
        const int r = i / (KC / 4), c = 4 * (i - r * (KC / 4));
        float4 v = make_float4(0.f, 0.f, 0.f, 0.f);
        if (t0 + r < T && k0 + c < n) v = *(const float4*)(u + (int64_t)(t0 + r) * C + (int64_t)blk * n + k0 + c);
        stage(us, r * LP + c, v.x);
        stage(us, r * LP + c + 1, v.y);
        stage(us, r * LP + c + 2, v.z);
        stage(us, r * LP + c + 3, v.w);
      }
    } else {
      for (int i = tid; i < TM * KC; i += 256) {
        const int r = i / KC, c = i - r * KC;
        stage(us, r * LP + c,
              (t0 + r < T && k0 + c < n) ? u[(int64_t)(t0 + r) * C + (int64_t)blk * n + k0 + c] : 0.f);
      }
    }
    __syncthreads();
#pragma unroll
    for (int ks = 0; ks < KC / 32; ks++) {
#pragma unroll
      for (int m = 0; m < MS; m++) {
#pragma unroll
        for (int p = NP - 1; p >= 0; p--) {                         // smallest part first
          const E* up = us[p] + (m * 16 + r16) * LP + 32 * ks + 8 * g;
          if constexpr (sizeof(E) == 2) {
            const bf16x8 a = *(const bf16x8*)up;
            ar[m] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, br[ks].v8(), ar[m], 0, 0, 0);
            ai[m] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, bi[ks].v8(), ai[m], 0, 0, 0);
          } else {
#pragma unroll
            for (int j = 0; j < 8; j++) {
              ar[m] = __builtin_amdgcn_mfma_f32_16x16x4f32(up[j], br[ks].v[j], ar[m], 0, 0, 0);
              ai[m] = __builtin_amdgcn_mfma_f32_16x16x4f32(up[j], bi[ks].v[j], ai[m], 0, 0, 0);
            }
          }
        }
      }
    }
  }
  if (!ok) return;
  const int c = blk * n + oc;
  const float cr = b_r[c], ci = b_i[c], lb = log_base[c];
#pragma unroll
  for (int m = 0; m < MS; m++)
#pragma unroll
    for (int i = 0; i < 4; i++) {
      const int t = t0 + m * 16 + 4 * g + i;
      if (t >= T) continue;
      const float la = sigmoidf(ar[m][i] + cr) * lb;
      a_out[(int64_t)t * C + c] = expf(la);
      x_out[(int64_t)t * C + c] = sqrtf(-expm1f(2.0f * la)) * sigmoidf(ai[m][i] + ci) * u[(int64_t)t * C + c];
    }
}

// ------------------------------------------------------------------ scan of the linear recurrent unit
__device__ __forceinline__ float gelu_tanh(float z) {
  return 0.5f * z * (1.0f + tanhf(0.7978845608028654f * (z + 0.044715f * z * z * z)));
}

// a workgroup: CW channels x NC pieces of a portion, thread = (piece, channel).  CW = 16 for long portions (more pieces,
// more workgroups), 64 for decoded tokens
template <typename E, int CW>
__global__ void __launch_bounds__(1024) rglru_scan_k(const float* __restrict__ a, const float* __restrict__ x,
                                                    const E* __restrict__ y, int64_t y_ld, float* __restrict__ state,
                                                    const int32_t* __restrict__ cu, const int32_t* __restrict__ slots,
                                                    const int64_t* __restrict__ pos, E* __restrict__ out, int C) {
  __shared__ float fa[1024], fb[1024];                              // the pieces' factors and results, [NC][CW]
  const int b = blockIdx.y;
  const int ch = threadIdx.x % CW, j = threadIdx.x / CW, NC = blockDim.x / CW;
  const int c = blockIdx.x * CW + ch;
  const int t0 = cu[b], n = cu[b + 1] - t0;
  if (n <= 0) return;
  const bool ok = c < C;
  const int per = (n + NC - 1) / NC;
  const int lo = min(n, j * per), hi = min(n, lo + per);
  const int64_t at = (int64_t)t0 * C + (ok ? c : 0);
  float A = 1.f, Bv = 0.f;                                          // the piece folded: S_out = A S_in + B
  constexpr int UN = 8;                                             // tokens whose inputs are requested together
  if (NC > 1) {
    if (ok)
      for (int tb = lo; tb < hi; tb += UN) {
        float av[UN], xv[UN];
#pragma unroll
        for (int i = 0; i < UN; i++) {
          const int64_t t = min(tb + i, hi - 1);
          av[i] = a[at + t * C];
          xv[i] = x[at + t * C];
        }
#pragma unroll
        for (int i = 0; i < UN; i++) {
          if (tb + i >= hi) break;
          A *= av[i];
          Bv = fmaf(av[i], Bv, xv[i]);
        }
      }
    fa[threadIdx.x] = A;
    fb[threadIdx.x] = Bv;
    __syncthreads();
  }
  float* st = state + (int64_t)slots[b] * C + (ok ? c : 0);
  float S = (ok && pos[t0] != 0) ? *st : 0.f;
  for (int jj = 0; jj < j; jj++) S = fmaf(fa[jj * CW + ch], S, fb[jj * CW + ch]);    // the carries in order
  __syncthreads();                                                  // every piece has read the slot
  if (!ok) return;
  const E* yp = y + (int64_t)t0 * y_ld + c;
  for (int tb = lo; tb < hi; tb += UN) {
    float av[UN], xv[UN], yv[UN];
#pragma unroll
    for (int i = 0; i < UN; i++) {
      const int64_t t = min(tb + i, hi - 1);
      av[i] = a[at + t * C];
      xv[i] = x[at + t * C];
      yv[i] = ldf(yp + t * y_ld);
    }
#pragma unroll
    for (int i = 0; i < UN; i++) {
      if (tb + i >= hi) break;
      S = fmaf(av[i], S, xv[i]);
      stf(out + at + (int64_t)(tb + i) * C, S * gelu_tanh(yv[i]));
    }
  }
  if (hi == n && lo < n) *st = S;                                   // the piece that holds the last token
}

}  // namespace

void decay_scan(bool bf16, const void* q, int64_t q_ld, const void* k, int64_t k_ld, const void* v, int64_t v_ld,
                const float* decay, float* S, const int32_t* cu, const int32_t* slots, const int64_t* pos, float* out,
                int B, int H, int d, int dv, hipStream_t st) {
  const DeltaArgs none{};
  if (bf16)
    launch_scan<__bf16, __bf16, false>((const __bf16*)q, q_ld, (const __bf16*)k, k_ld, (const __bf16*)v, v_ld, decay, none,
                                       S, cu, slots, pos, out, B, H, H, d, dv, st);
  else
    launch_scan<float, float, false>((const float*)q, q_ld, (const float*)k, k_ld, (const float*)v, v_ld, decay, none, S,
                                     cu, slots, pos, out, B, H, H, d, dv, st);
}

void delta_scan(bool bf16, const float* q, int64_t q_ld, const float* k, int64_t k_ld, const float* v, int64_t v_ld,
                DeltaArgs da, float* S, const int32_t* cu, const int32_t* slots, const int64_t* pos, float* out, int B, int H,
                int K, int d, int dv, hipStream_t st) {
  if (bf16)
    launch_scan<float, __bf16, true>(q, q_ld, k, k_ld, v, v_ld, nullptr, da, S, cu, slots, pos, out, B, H, K, d, dv, st);
  else
    launch_scan<float, float, true>(q, q_ld, k, k_ld, v, v_ld, nullptr, da, S, cu, slots, pos, out, B, H, K, d, dv, st);
}

void rglru_gates(bool bf16, const float* u, const void* w_r, const float* b_r, const void* w_i, const float* b_i,
                 const float* log_base, float* a, float* x, int T, int nb, int n, hipStream_t st) {
  if (T <= 0 || n <= 0) return;
  const int ct = nb * ((n + 63) / 64);
#define SX_GATES(E, TM)                                                                                                  \
  rglru_gates_k<E, TM><<<dim3((T + TM - 1) / TM, ct), 256, 0, st>>>(u, (const E*)w_r, b_r, (const E*)w_i, b_i, log_base, \
                                                                    a, x, T, nb, n)
  if (bf16) {
    if (T <= 64) { SX_GATES(__bf16, 16); } else { SX_GATES(__bf16, 64); }
  } else {
    if (T <= 64) { SX_GATES(float, 16); } else { SX_GATES(float, 64); }
  }
#undef SX_GATES
}

void rglru_scan(bool bf16, const float* a, const float* x, const void* y, int64_t y_ld, float* state, const int32_t* cu,
                const int32_t* slots, const int64_t* pos, void* out, int B, int C, int max_n, hipStream_t st) {
  if (B <= 0 || C <= 0) return;
  // pieces per portion: at least 16 tokens a piece, at most 64 of them
  int nc = 1;
  while (nc < 64 && max_n >= 32 * nc) nc *= 2;
#define SX_LRU(E, CW)                                                                                                  \
  rglru_scan_k<E, CW><<<dim3((C + CW - 1) / CW, B), CW * nc, 0, st>>>(a, x, (const E*)y, y_ld, state, cu, slots, pos, \
                                                                      (E*)out, C)
  if (nc >= 4) {
    if (bf16) SX_LRU(__bf16, 16); else SX_LRU(float, 16);
  } else {
    if (bf16) SX_LRU(__bf16, 64); else SX_LRU(float, 64);
  }
#undef SX_LRU
}

}  // namespace sx
}  // namespace illm
