// Element-wise steps and small products of the pre-norm blocks with scaled
// sublayers and of the mixers with per-channel decays (gfx950, wave64).
//
//   residual + norm    x += source, out = x / rms(x) w in one pass, a workgroup
//                      per token; the source is a product's rows, two of them,
//                      or a token's expert rows, each with a scale per coordinate
//   loop input         [x + source | token embedding] as the input rows of the
//                      projection in front of a pass
//   token mixes        several blends of a token's and its predecessor's row
//   low-rank decay     the second product of a low-rank projection on the matrix
//                      cores, its result turned into decays in the epilogue
//   grouped product    decode-size projection whose row groups read different
//                      inputs: one launch for a mixer's whole input projection
//
// Activations are bf16 or f32 (template E); all arithmetic is f32.
#include "chanmix.h"
#include "split_tile.h"

#include <math.h>

namespace illm {
namespace cx {
namespace {

using sx::bf16x8;
using sx::f32x4;

template <typename E> __device__ __forceinline__ float ldf(const E* p);
template <> __device__ __forceinline__ float ldf<float>(const float* p) { return *p; }
template <> __device__ __forceinline__ float ldf<__bf16>(const __bf16* p) { return (float)*p; }
template <typename E> __device__ __forceinline__ void stf(E* p, float v);
template <> __device__ __forceinline__ void stf<float>(float* p, float v) { *p = v; }
template <> __device__ __forceinline__ void stf<__bf16>(__bf16* p, float v) { *p = (__bf16)v; }

// V consecutive values as one access (V = 4: the launcher checks that W is a multiple of 4)
template <typename E, int V> struct Vec;
template <typename E> struct Vec<E, 1> {
  static __device__ __forceinline__ void ld(const E* p, float* v) { v[0] = ldf(p); }
  static __device__ __forceinline__ void st(E* p, const float* v) { stf(p, v[0]); }
};
template <> struct Vec<float, 4> {
  static __device__ __forceinline__ void ld(const float* p, float* v) {
    const float4 a = *(const float4*)p;
    v[0] = a.x, v[1] = a.y, v[2] = a.z, v[3] = a.w;
  }
  static __device__ __forceinline__ void st(float* p, const float* v) { *(float4*)p = make_float4(v[0], v[1], v[2], v[3]); }
};
template <> struct Vec<__bf16, 4> {
  typedef __bf16 B4 __attribute__((ext_vector_type(4)));
  static __device__ __forceinline__ void ld(const __bf16* p, float* v) {
    const B4 a = *(const B4*)p;
    v[0] = (float)a[0], v[1] = (float)a[1], v[2] = (float)a[2], v[3] = (float)a[3];
  }
  static __device__ __forceinline__ void st(__bf16* p, const float* v) {
    *(B4*)p = B4{(__bf16)v[0], (__bf16)v[1], (__bf16)v[2], (__bf16)v[3]};
  }
};

__device__ __forceinline__ float wave_sum(float v) {
#pragma unroll
  for (int o = 32; o > 0; o >>= 1) v += __shfl_xor(v, o, 64);
  return v;
}
__device__ __forceinline__ float block_sum(float v, float* red) {   // red: >= 16 floats of LDS
  v = wave_sum(v);
  const int w = threadIdx.x >> 6, nw = (blockDim.x + 63) >> 6;
  __syncthreads();
  if ((threadIdx.x & 63) == 0) red[w] = v;
  __syncthreads();
  float s = 0.f;
  for (int i = 0; i < nw; i++) s += red[i];
  return s;
}

enum Mode { kNone, kOne, kOneF32, kPair, kRows };

// v += the source's V values of token t at coordinate c
template <typename E, int V, int MODE>
__device__ __forceinline__ void add_source(const Source& y, int64_t t, int c, int W, float* v) {
  if (MODE == kNone) return;
  float s[V], a[V];
  Vec<float, V>::ld(y.sa + c, s);
  if (MODE == kRows) {
    float sum[V];
#pragma unroll
    for (int i = 0; i < V; i++) sum[i] = 0.f;
    for (int k = 0; k < y.top; k++) {
      Vec<float, V>::ld((const float*)y.a + (t * y.top + k) * W + c, a);
#pragma unroll
      for (int i = 0; i < V; i++) sum[i] += a[i];
    }
#pragma unroll
    for (int i = 0; i < V; i++) v[i] = fmaf(s[i], sum[i], v[i]);
    return;
  }
  if (MODE == kOneF32) Vec<float, V>::ld((const float*)y.a + t * W + c, a);
  else Vec<E, V>::ld((const E*)y.a + t * W + c, a);
  if (MODE == kPair) {
    float b[V], sb[V];
    Vec<E, V>::ld((const E*)y.b + t * W + c, b);
    Vec<float, V>::ld(y.sb + c, sb);
#pragma unroll
    for (int i = 0; i < V; i++) v[i] += fmaf(s[i], a[i], sb[i] * b[i]);
  } else {
#pragma unroll
    for (int i = 0; i < V; i++) v[i] = fmaf(s[i], a[i], v[i]);
  }
}

// the row stays in registers between the two passes (KEEP pieces of V values per thread; longer rows read the rest back)
template <typename E, int V, int MODE>
__global__ void __launch_bounds__(1024) add_scaled_norm_k(float* __restrict__ x, Source y, const float* __restrict__ w,
                                                         float eps, E* __restrict__ out, int W) {
  constexpr int KEEP = 4;
  __shared__ float red[16];
  const int64_t t = blockIdx.x;
  float* xr = x + t * W;
  const int step = V * blockDim.x;
  float keep[KEEP][V];
  float q = 0.f;
#pragma unroll
  for (int k = 0; k < KEEP; k++) {
    const int c = V * threadIdx.x + k * step;
    if (c < W) {
      Vec<float, V>::ld(xr + c, keep[k]);
      add_source<E, V, MODE>(y, t, c, W, keep[k]);
      if (MODE != kNone) Vec<float, V>::st(xr + c, keep[k]);
#pragma unroll
      for (int i = 0; i < V; i++) q = fmaf(keep[k][i], keep[k][i], q);
    }
  }
  for (int c = V * threadIdx.x + KEEP * step; c < W; c += step) {
    float v[V];
    Vec<float, V>::ld(xr + c, v);
    add_source<E, V, MODE>(y, t, c, W, v);
    if (MODE != kNone) Vec<float, V>::st(xr + c, v);
#pragma unroll
    for (int i = 0; i < V; i++) q = fmaf(v[i], v[i], q);
  }
  const float rs = 1.0f / sqrtf(block_sum(q, red) / (float)W + eps);
#pragma unroll
  for (int k = 0; k < KEEP; k++) {
    const int c = V * threadIdx.x + k * step;
    if (c < W) {
      float g[V];
      Vec<float, V>::ld(w + c, g);
#pragma unroll
      for (int i = 0; i < V; i++) keep[k][i] = keep[k][i] * rs * g[i];
      Vec<E, V>::st(out + t * W + c, keep[k]);
    }
  }
  for (int c = V * threadIdx.x + KEEP * step; c < W; c += step) {
    float v[V], g[V];
    Vec<float, V>::ld(xr + c, v);
    Vec<float, V>::ld(w + c, g);
#pragma unroll
    for (int i = 0; i < V; i++) v[i] = v[i] * rs * g[i];
    Vec<E, V>::st(out + t * W + c, v);
  }
}

template <typename E, int V, int MODE>
__global__ void __launch_bounds__(256) loop_input_k(const float* __restrict__ x, Source y, const E* __restrict__ embed,
                                                   int64_t vocab, const int64_t* __restrict__ ids, E* __restrict__ out,
                                                   int W) {
  const int c = V * (blockIdx.y * blockDim.x + threadIdx.x);
  if (c >= W) return;
  const int64_t t = blockIdx.x, id = ids[t];
  float v[V], e[V];
  Vec<float, V>::ld(x + t * W + c, v);
  add_source<E, V, MODE>(y, t, c, W, v);
  Vec<E, V>::st(out + t * 2 * W + c, v);
#pragma unroll
  for (int i = 0; i < V; i++) e[i] = 0.f;
  if (id >= 0 && id < vocab) Vec<E, V>::ld(embed + id * W + c, e);
  Vec<E, V>::st(out + t * 2 * W + W + c, e);
}

template <typename E, int V>
__global__ void __launch_bounds__(256) token_mixes_k(const E* __restrict__ h, const float* __restrict__ mu, int NM,
                                                    float* __restrict__ state, const int32_t* __restrict__ cu,
                                                    const int32_t* __restrict__ seq_of, const int32_t* __restrict__ slots,
                                                    const int64_t* __restrict__ pos, E* __restrict__ out, int T, int W,
                                                    int single) {
  const int c = V * (blockIdx.y * blockDim.x + threadIdx.x);
  if (c >= W) return;
  const int64_t t = blockIdx.x;
  const int b = seq_of[t];
  float a[V], p[V], m[V], o[V];
  Vec<E, V>::ld(h + t * W + c, a);
  float* st = state + (int64_t)slots[b] * W + c;
#pragma unroll
  for (int i = 0; i < V; i++) p[i] = 0.f;
  if (t > cu[b]) Vec<E, V>::ld(h + (t - 1) * W + c, p);
  else if (pos[t] > 0) Vec<float, V>::ld(st, p);
#pragma unroll
  for (int i = 0; i < V; i++) p[i] -= a[i];
  for (int j = 0; j < NM; j++) {
    Vec<float, V>::ld(mu + (int64_t)j * W + c, m);
#pragma unroll
    for (int i = 0; i < V; i++) o[i] = fmaf(p[i], m[i], a[i]);
    Vec<E, V>::st(out + ((int64_t)j * T + t) * W + c, o);
  }
  if (single) Vec<float, V>::st(st, a);                             // one token per sequence: the slot's only reader
}

// several tokens per sequence: the slots advance after every first token has read them
template <typename E>
__global__ void __launch_bounds__(256) last_rows_k(const E* __restrict__ h, float* __restrict__ state,
                                                  const int32_t* __restrict__ cu, const int32_t* __restrict__ slots, int W) {
  const int b = blockIdx.x;
  if (cu[b + 1] <= cu[b]) return;
  const E* r = h + (int64_t)(cu[b + 1] - 1) * W;
  for (int c = threadIdx.x; c < W; c += blockDim.x) state[(int64_t)slots[b] * W + c] = ldf(r + c);
}

// ------------------------------------------------------------------ low-rank decay
// softplus(z) = max(z, 0) + log1p(t), t = exp(-|z|); log1p(t) = 2 atanh(s), s = t / (2 + t) <= 1/3, by its power series
__device__ __forceinline__ float softplusf(float z) {
  const float t = __expf(-fabsf(z)), s = t / (2.0f + t), q = s * s;
  float a = 1.0f / 15.0f;
  a = fmaf(a, q, 1.0f / 13.0f);
  a = fmaf(a, q, 1.0f / 11.0f);
  a = fmaf(a, q, 1.0f / 9.0f);
  a = fmaf(a, q, 1.0f / 7.0f);
  a = fmaf(a, q, 1.0f / 5.0f);
  a = fmaf(a, q, 1.0f / 3.0f);
  a = fmaf(a, q, 1.0f);
  return fmaxf(z, 0.f) + 2.0f * s * a;
}

// the parts of an input value: tanh leaves an f32 number (three 16-bit parts), a plain 16-bit input is one part
template <typename E, bool SQ> struct InParts { static constexpr int N = 1; };
template <> struct InParts<__bf16, true> { static constexpr int N = 3; };

// a workgroup: TM tokens x 64 NT outputs, wave w the NT tiles of 16 from 16 NT w on; inside a step of 32 lane group g
// holds k = 8 g .. 8 g + 7 (inputs and weights alike, so the f32 products may take them one after another)
template <typename E, int TM, int NT, bool SQ>
__global__ void __launch_bounds__(256) lowrank_decay_k(const E* __restrict__ in, int64_t ld, const E* __restrict__ w,
                                                      const float* __restrict__ rate, const float* __restrict__ bias,
                                                      int kind, float* __restrict__ out, int T, int N, int R) {
  constexpr int NP = InParts<E, SQ>::N, KC = 64, LP = KC + (sizeof(E) == 2 ? 8 : 4), MS = TM / 16;
  __shared__ __attribute__((aligned(16))) E us[NP][TM * LP];
  const int t0 = blockIdx.x * TM;
  const int tid = threadIdx.x, wv = tid >> 6, lane = tid & 63, r16 = lane & 15, g = lane >> 4;
  const int n0 = (blockIdx.y * 4 + wv) * 16 * NT + r16;
  const bool vec = R % 8 == 0;
  f32x4 acc[NT][MS];
#pragma unroll
  for (int c = 0; c < NT; c++)
#pragma unroll
    for (int m = 0; m < MS; m++) acc[c][m] = f32x4{0.f, 0.f, 0.f, 0.f};
  for (int k0 = 0; k0 < R; k0 += KC) {
    sx::Frag<E> b[NT][KC / 32];
#pragma unroll
    for (int c = 0; c < NT; c++) {
      const int n = n0 + 16 * c;
#pragma unroll
      for (int ks = 0; ks < KC / 32; ks++)
        b[c][ks].load(w + (int64_t)(n < N ? n : 0) * R, k0 + 32 * ks + 8 * g, n < N ? R : 0, vec);
    }
    __syncthreads();
    constexpr int PER = TM * KC / 256;                              // values per thread, all requested together
    float x[PER];
#pragma unroll
    for (int j = 0; j < PER; j++) {
      const int i = tid + 256 * j, r = i / KC, c = i - r * KC;
      x[j] = (t0 + r < T && k0 + c < R) ? ldf(in + (int64_t)(t0 + r) * ld + k0 + c) : 0.f;
    }
#pragma unroll
    for (int j = 0; j < PER; j++) {
      const int i = tid + 256 * j, r = i / KC, c = i - r * KC;
      const float v = SQ ? tanhf(x[j]) : x[j];
      if constexpr (NP == 3) sx::stage(us, r * LP + c, v);
      else us[0][r * LP + c] = (E)v;
    }
    __syncthreads();
#pragma unroll
    for (int ks = 0; ks < KC / 32; ks++) {
      if (k0 + 32 * ks >= R) break;
#pragma unroll
      for (int m = 0; m < MS; m++) {
#pragma unroll
        for (int p = NP - 1; p >= 0; p--) {                         // smallest part first
          const E* up = us[p] + (m * 16 + r16) * LP + 32 * ks + 8 * g;
#pragma unroll
          for (int c = 0; c < NT; c++) {
            if constexpr (sizeof(E) == 2) {
              acc[c][m] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(*(const bf16x8*)up, b[c][ks].v8(), acc[c][m], 0, 0, 0);
            } else {
#pragma unroll
              for (int j = 0; j < 8; j++)
                acc[c][m] = __builtin_amdgcn_mfma_f32_16x16x4f32(up[j], b[c][ks].v[j], acc[c][m], 0, 0, 0);
            }
          }
        }
      }
    }
  }
#pragma unroll
  for (int c = 0; c < NT; c++) {
    const int n = n0 + 16 * c;
    if (n >= N) continue;
    const float bs = bias[n], rt = kind == 0 ? rate[n] : 0.f;
#pragma unroll
    for (int m = 0; m < MS; m++)
#pragma unroll
      for (int i = 0; i < 4; i++) {
        const int t = t0 + m * 16 + 4 * g + i;
        if (t >= T) continue;
        const float z = acc[c][m][i] + bs;
        out[(int64_t)t * N + n] = kind == 0 ? __expf(-rt * softplusf(z)) : __expf(-__expf(z));
      }
  }
}

// ------------------------------------------------------------------ grouped skinny product
// one workgroup per 16-row weight tile, its DW waves over pieces of K: the weight tile is the A operand straight from
// memory, the group's <= 16 input rows the B operand (absent rows zero); the waves' partial tiles are added in wave
// order, so a row's result does not depend on how many rows share the launch
constexpr int DW = 8;

template <typename O>
__global__ void __launch_bounds__(64 * DW) grouped_linear_k(Groups gr, int M, int64_t K, const __bf16* __restrict__ w,
                                                          const __bf16* __restrict__ bias, O* __restrict__ out, int64_t N) {
  __shared__ f32x4 red[DW][64];
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, r = lane & 15, g = lane >> 4;
  const int tile = blockIdx.x;
  const __bf16* x = (const __bf16*)gr.x[0];
  int row0 = gr.row0[0] + 16 * tile, end = gr.row0[1];
#pragma unroll
  for (int j = 1; j < kMaxGroups; j++)
    if (j < gr.n && tile >= gr.tile0[j]) {
      x = (const __bf16*)gr.x[j];
      row0 = gr.row0[j] + 16 * (tile - gr.tile0[j]);
      end = gr.row0[j + 1];
    }
  const int nr = min(row0 + r, end - 1);
  const __bf16* wr = w + (int64_t)nr * K + 8 * g;
  const bool on = r < M;
  const __bf16* xr = x + (int64_t)(on ? r : 0) * K + 8 * g;
  const int64_t steps = K / 64;
  const int64_t s0 = steps * wave / DW, s1 = steps * (wave + 1) / DW;
  auto ld = [](const __bf16* p) { return *(const bf16x8*)p; };
  bf16x8 zero;
#pragma unroll
  for (int i = 0; i < 8; i++) zero[i] = (__bf16)0.f;
  f32x4 acc = {0.f, 0.f, 0.f, 0.f};
  int64_t s = s0;
  for (; s + 1 < s1; s += 2) {
    const int64_t k = s * 64;
    const bf16x8 a0 = ld(wr + k), a1 = ld(wr + k + 32), a2 = ld(wr + k + 64), a3 = ld(wr + k + 96);
    const bf16x8 b0 = on ? ld(xr + k) : zero, b1 = on ? ld(xr + k + 32) : zero;
    const bf16x8 b2 = on ? ld(xr + k + 64) : zero, b3 = on ? ld(xr + k + 96) : zero;
    acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a0, b0, acc, 0, 0, 0);
    acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a1, b1, acc, 0, 0, 0);
    acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a2, b2, acc, 0, 0, 0);
    acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a3, b3, acc, 0, 0, 0);
  }
  if (s < s1) {
    const int64_t k = s * 64;
    const bf16x8 b0 = on ? ld(xr + k) : zero, b1 = on ? ld(xr + k + 32) : zero;
    acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(ld(wr + k), b0, acc, 0, 0, 0);
    acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(ld(wr + k + 32), b1, acc, 0, 0, 0);
  }
  red[wave][lane] = acc;
  __syncthreads();
  if (wave != 0) return;
  f32x4 v = red[0][lane];
#pragma unroll
  for (int i = 1; i < DW; i++) v += red[i][lane];
  if (!on) return;                                                  // lane holds rows row0 + 4 g + i of input row r
#pragma unroll
  for (int i = 0; i < 4; i++) {
    const int n = row0 + 4 * g + i;
    if (n < end) stf(out + (int64_t)r * N + n, v[i] + (bias ? (float)bias[n] : 0.f));
  }
}

int row_threads(int W, int V) {
  const int n = (W + V - 1) / V;
  return n >= 1024 ? 1024 : (n + 63) / 64 * 64;
}
Mode mode_of(const Source& y) {
  return !y.a ? kNone : (y.top > 0 ? kRows : (y.b ? kPair : (y.a_f32 ? kOneF32 : kOne)));
}

}  // namespace

#define CX_V(W, CALL1, CALL4) \
  if ((W) % 4 == 0) {         \
    CALL4;                    \
  } else {                    \
    CALL1;                    \
  }
#define CX_MODES(CALL, E, V)                  \
  switch (mode_of(y)) {                       \
    case kNone: CALL(E, V, kNone); break;     \
    case kOne: CALL(E, V, kOne); break;       \
    case kOneF32: CALL(E, V, kOneF32); break; \
    case kPair: CALL(E, V, kPair); break;     \
    default: CALL(E, V, kRows);               \
  }

void add_scaled_norm(bool bf16, float* x, Source y, const float* w, float eps, void* out, int T, int W, hipStream_t st) {
  if (T <= 0) return;
#define CALL(E, V, M) add_scaled_norm_k<E, V, M><<<T, row_threads(W, V), 0, st>>>(x, y, w, eps, (E*)out, W)
  if (bf16) { CX_V(W, CX_MODES(CALL, __bf16, 1), CX_MODES(CALL, __bf16, 4)) }
  else { CX_V(W, CX_MODES(CALL, float, 1), CX_MODES(CALL, float, 4)) }
#undef CALL
}

void loop_input(bool bf16, const float* x, Source y, const void* embed, int64_t vocab, const int64_t* ids, void* out, int T,
                int W, hipStream_t st) {
  if (T <= 0) return;
#define CALL(E, V, M)                                                                                      \
  loop_input_k<E, V, M><<<dim3(T, ((W + V - 1) / V + 255) / 256), 256, 0, st>>>(x, y, (const E*)embed, vocab, ids, \
                                                                                (E*)out, W)
  if (bf16) { CX_V(W, CX_MODES(CALL, __bf16, 1), CX_MODES(CALL, __bf16, 4)) }
  else { CX_V(W, CX_MODES(CALL, float, 1), CX_MODES(CALL, float, 4)) }
#undef CALL
}

void token_mixes(bool bf16, const void* h, const float* mu, int NM, float* state, const int32_t* cu, const int32_t* seq_of,
                 const int32_t* slots, const int64_t* pos, void* out, int T, int B, int W, bool single, hipStream_t st) {
  if (T <= 0) return;
#define CALL(E, V)                                                                                          \
  token_mixes_k<E, V><<<dim3(T, ((W + V - 1) / V + 255) / 256), 256, 0, st>>>((const E*)h, mu, NM, state, cu, seq_of, \
                                                                              slots, pos, (E*)out, T, W, single ? 1 : 0)
  if (bf16) { CX_V(W, CALL(__bf16, 1), CALL(__bf16, 4)) } else { CX_V(W, CALL(float, 1), CALL(float, 4)) }
#undef CALL
  if (single) return;
  if (bf16) last_rows_k<__bf16><<<B, 256, 0, st>>>((const __bf16*)h, state, cu, slots, W);
  else last_rows_k<float><<<B, 256, 0, st>>>((const float*)h, state, cu, slots, W);
}

void lowrank_decay(bool bf16, const void* in, int64_t ld, const void* w, const float* rate, const float* bias, int kind,
                   bool squash, float* out, int T, int N, int R, hipStream_t st) {
  if (T <= 0 || N <= 0) return;
#define CALL(E, TM, NT, SQ)                                                                                        \
  lowrank_decay_k<E, TM, NT, SQ><<<dim3((T + TM - 1) / TM, (N + 64 * NT - 1) / (64 * NT)), 256, 0, st>>>(            \
      (const E*)in, ld, (const E*)w, rate, bias, kind, out, T, N, R)
#define CALL_T(E, SQ) \
  if (T <= 64) CALL(E, 16, 1, SQ); else CALL(E, 64, 2, SQ)
  if (bf16) { if (squash) { CALL_T(__bf16, true); } else { CALL_T(__bf16, false); } }
  else { if (squash) { CALL_T(float, true); } else { CALL_T(float, false); } }
#undef CALL_T
#undef CALL
}

void grouped_linear(Groups g, int M, int K, const void* w, const void* bias, void* out, bool out_f32, hipStream_t st) {
  const int tiles = g.tile0[g.n], N = g.row0[g.n];
  if (M <= 0 || tiles <= 0) return;
  if (out_f32)
    grouped_linear_k<float><<<tiles, 64 * DW, 0, st>>>(g, M, K, (const __bf16*)w, (const __bf16*)bias, (float*)out, N);
  else
    grouped_linear_k<__bf16><<<tiles, 64 * DW, 0, st>>>(g, M, K, (const __bf16*)w, (const __bf16*)bias, (__bf16*)out, N);
}

}  // namespace cx
}  // namespace illm
