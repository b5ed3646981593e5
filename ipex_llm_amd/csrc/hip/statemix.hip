// Element-wise and routing kernels of the decoders whose sublayers are normed
// before and after (gfx950, wave64).
//
//   tanh norm          tanh(alpha x) w + b: no statistics, so it fuses with
//                      whatever produces x
//   residual + norms   x += post(y), out = pre(x) in one pass.  y is a row of a
//                      product, the mean of two RMS-normed rows (a workgroup
//                      per token forms both sums of squares first), or the sum
//                      of a token's expert rows (identity experts add their
//                      weight times the input)
//   RMS + sigmoid gate over the whole row
//   group routing      one wave per token: softmax over all router outputs (or sigmoids),
//                      corrected scores and the groups' best ones in LDS, the
//                      kept groups by rank, then the winners one after another;
//                      for few tokens the same launch forms the logits
//
// Activations are bf16 or f32 (template E); all arithmetic is f32.
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
__device__ __forceinline__ float wave_max(float v) {
#pragma unroll
  for (int o = 32; o > 0; o >>= 1) v = fmaxf(v, __shfl_xor(v, o, 64));
  return v;
}
// sums of two values over a block of up to 1024 threads; red: >= 32 floats of LDS
__device__ __forceinline__ void block_sum2(float& a, float& b, float* red) {
  a = wave_sum(a);
  b = wave_sum(b);
  const int w = threadIdx.x >> 6, nw = (blockDim.x + 63) >> 6;
  __syncthreads();
  if ((threadIdx.x & 63) == 0) {
    red[2 * w] = a;
    red[2 * w + 1] = b;
  }
  __syncthreads();
  a = b = 0.f;
  for (int i = 0; i < nw; i++) {
    a += red[2 * i];
    b += red[2 * i + 1];
  }
}

template <int V>
__device__ __forceinline__ void norm_v(const Norm& n, float alpha, int c, const float* v, float* o) {
  float w[V], b[V];
  Vec<float, V>::ld(n.w + c, w);
  Vec<float, V>::ld(n.b + c, b);
#pragma unroll
  for (int i = 0; i < V; i++) o[i] = fmaf(tanhf(alpha * v[i]), w[i], b[i]);
}

template <typename E, int V>
__global__ void __launch_bounds__(256) dyn_tanh_k(const float* __restrict__ x, Norm n, E* __restrict__ out, int W) {
  const int c = V * (blockIdx.y * blockDim.x + threadIdx.x);
  if (c >= W) return;
  const int64_t at = (int64_t)blockIdx.x * W + c;
  float v[V], o[V];
  Vec<float, V>::ld(x + at, v);
  norm_v<V>(n, *n.alpha, c, v, o);
  Vec<E, V>::st(out + at, o);
}

// the last part of every fused pass: x += post(y), out = pre(x) for the V values at ``at`` (coordinate c)
template <typename E, int V>
__device__ __forceinline__ void finish(float* __restrict__ x, const float* y, const Norm& post, const Norm& pre,
                                       E* __restrict__ out, int64_t at, int c) {
  float v[V], o[V];
  Vec<float, V>::ld(x + at, v);
  norm_v<V>(post, *post.alpha, c, y, o);
#pragma unroll
  for (int i = 0; i < V; i++) v[i] += o[i];
  Vec<float, V>::st(x + at, v);
  if (pre.alpha) {
    norm_v<V>(pre, *pre.alpha, c, v, o);
    Vec<E, V>::st(out + at, o);
  }
}

template <typename E, typename Y, int V>
__global__ void __launch_bounds__(256) add_normed_k(float* __restrict__ x, const Y* __restrict__ y, Norm post, Norm pre,
                                                   E* __restrict__ out, int W) {
  const int c = V * (blockIdx.y * blockDim.x + threadIdx.x);
  if (c >= W) return;
  const int64_t at = (int64_t)blockIdx.x * W + c;
  float v[V];
  Vec<Y, V>::ld(y + at, v);
  finish<E, V>(x, v, post, pre, out, at, c);
}

template <typename E, int V>
__global__ void __launch_bounds__(1024) add_normed_pair_k(float* __restrict__ x, const E* __restrict__ a,
                                                         const E* __restrict__ b, const E* __restrict__ wa,
                                                         const E* __restrict__ wb, float eps, Norm post, Norm pre,
                                                         E* __restrict__ out, int W) {
  __shared__ float red[32];
  const int64_t r0 = (int64_t)blockIdx.x * W;
  float qa = 0.f, qb = 0.f;
  for (int c = V * threadIdx.x; c < W; c += V * blockDim.x) {
    float va[V], vb[V];
    Vec<E, V>::ld(a + r0 + c, va);
    Vec<E, V>::ld(b + r0 + c, vb);
#pragma unroll
    for (int i = 0; i < V; i++) {
      qa = fmaf(va[i], va[i], qa);
      qb = fmaf(vb[i], vb[i], qb);
    }
  }
  block_sum2(qa, qb, red);
  const float ra = 0.5f / sqrtf(qa / (float)W + eps), rb = 0.5f / sqrtf(qb / (float)W + eps);
  for (int c = V * threadIdx.x; c < W; c += V * blockDim.x) {
    float va[V], vb[V], ga[V], gb[V], y[V];
    Vec<E, V>::ld(a + r0 + c, va);
    Vec<E, V>::ld(b + r0 + c, vb);
    Vec<E, V>::ld(wa + c, ga);
    Vec<E, V>::ld(wb + c, gb);
#pragma unroll
    for (int i = 0; i < V; i++) y[i] = va[i] * ra * ga[i] + vb[i] * rb * gb[i];
    finish<E, V>(x, y, post, pre, out, r0 + c, c);
  }
}

template <typename E, int V>
__global__ void __launch_bounds__(256) add_normed_experts_k(float* __restrict__ x, const float* __restrict__ rows,
                                                           const int32_t* __restrict__ idx, const float* __restrict__ wts,
                                                           const E* __restrict__ h, int top, int experts, Norm post,
                                                           Norm pre, E* __restrict__ out, int W) {
  const int c = V * (blockIdx.y * blockDim.x + threadIdx.x);
  if (c >= W) return;
  const int64_t t = blockIdx.x, at = t * W + c;
  float y[V], hv[V];
  Vec<E, V>::ld(h + at, hv);
#pragma unroll
  for (int i = 0; i < V; i++) y[i] = 0.f;
  for (int k = 0; k < top; k++) {                                   // the chosen experts in order
    const int64_t p = t * top + k;
    if (idx[p] < experts) {
      float v[V];
      Vec<float, V>::ld(rows + p * W + c, v);
#pragma unroll
      for (int i = 0; i < V; i++) y[i] += v[i];
    } else {
      const float w = wts[p];
#pragma unroll
      for (int i = 0; i < V; i++) y[i] = fmaf(w, hv[i], y[i]);
    }
  }
  finish<E, V>(x, y, post, pre, out, at, c);
}

template <typename E>
__global__ void __launch_bounds__(1024) rms_sigmoid_gate_k(const float* __restrict__ o, const E* __restrict__ w,
                                                          const E* __restrict__ gate, int64_t g_ld, E* __restrict__ out,
                                                          int C, float eps) {
  __shared__ float red[32];
  const int64_t t = blockIdx.x;
  float q = 0.f, z = 0.f;
  for (int c = threadIdx.x; c < C; c += blockDim.x) q = fmaf(o[t * C + c], o[t * C + c], q);
  block_sum2(q, z, red);
  const float rs = 1.0f / sqrtf(q / (float)C + eps);
  for (int c = threadIdx.x; c < C; c += blockDim.x)
    stf(out + t * C + c, o[t * C + c] * rs * ldf(w + c) / (1.0f + expf(-ldf(gate + t * g_ld + c))));
}

// ------------------------------------------------------------------ routing
constexpr int kPerLane = 8;                                         // experts <= 512

// one wave routes token t with the logits z[0 .. E - 1]; cs, best: LDS of 64 PER values (E <= 64 PER)
__device__ __forceinline__ void wave_sync() {
  __builtin_amdgcn_fence(__ATOMIC_RELEASE, "wavefront");
  __builtin_amdgcn_wave_barrier();
  __builtin_amdgcn_fence(__ATOMIC_ACQUIRE, "wavefront");
}
template <int PER>
__device__ void route_wave(const float* z, const float* __restrict__ corr, RouteRule rule, int E, int top, int groups,
                           int keep, int32_t* __restrict__ idx, float* __restrict__ w, int64_t t, float* cs, float* best) {
  const int lane = threadIdx.x & 63;
  float s[PER], c[PER];
  float mx = -INFINITY;
#pragma unroll
  for (int i = 0; i < PER; i++) {
    const int e = lane + 64 * i;
    s[i] = e < E ? z[e] : -INFINITY;
    mx = fmaxf(mx, s[i]);
  }
  if (rule.sigmoid) {
#pragma unroll
    for (int i = 0; i < PER; i++) s[i] = lane + 64 * i < E ? 1.0f / (1.0f + expf(-s[i])) : 0.f;
  } else {
    mx = wave_max(mx);
    float sum = 0.f;
#pragma unroll
    for (int i = 0; i < PER; i++) {
      s[i] = lane + 64 * i < E ? expf(s[i] - mx) : 0.f;
      sum += s[i];
    }
    const float inv = 1.0f / wave_sum(sum);
#pragma unroll
    for (int i = 0; i < PER; i++) s[i] *= inv;
  }
#pragma unroll
  for (int i = 0; i < PER; i++) {
    const int e = lane + 64 * i;
    c[i] = e < E ? s[i] + (corr ? corr[e] : 0.f) : -INFINITY;
    if (e < E) cs[e] = c[i];
  }
  if (keep < groups) {
    const int gs = E / groups;
    wave_sync();
    for (int g = lane; g < groups; g += 64) {
      float b = -INFINITY, b2 = -INFINITY;
      for (int j = 0; j < gs; j++) {
        const float v = cs[g * gs + j];
        b2 = fmaxf(b2, fminf(b, v));
        b = fmaxf(b, v);
      }
      best[g] = rule.best_two && gs > 1 ? b + b2 : b;
    }
    wave_sync();
    bool kept[PER];
#pragma unroll
    for (int i = 0; i < PER; i++) {
      const int g = lane + 64 * i;
      int rank = 0;
      if (g < groups) {
        const float b = best[g];
        for (int j = 0; j < groups; j++) rank += best[j] > b || (best[j] == b && j < g);
      }
      kept[i] = g < groups && rank < keep;
    }
    wave_sync();
#pragma unroll
    for (int i = 0; i < PER; i++)
      if (lane + 64 * i < groups) best[lane + 64 * i] = kept[i] ? 1.f : 0.f;
    wave_sync();
#pragma unroll
    for (int i = 0; i < PER; i++) {
      const int e = lane + 64 * i;
      if (e < E && best[e / gs] == 0.f) c[i] = -INFINITY;
    }
  }
  float total = 0.f;
  for (int k = 0; k < top; k++) {
    float bv = -INFINITY;
    int be = 0x7fffffff;
#pragma unroll
    for (int i = 0; i < PER; i++)
      if (c[i] > bv) {                                              // ascending e within a lane: the first of equals stays
        bv = c[i];
        be = lane + 64 * i;
      }
#pragma unroll
    for (int o = 32; o > 0; o >>= 1) {
      const float ov = __shfl_xor(bv, o, 64);
      const int oe = __shfl_xor(be, o, 64);
      if (ov > bv || (ov == bv && oe < be)) {
        bv = ov;
        be = oe;
      }
    }
    const bool none = be == 0x7fffffff;                             // scores that are no numbers: any expert, weight 0
    if (none && lane == 0) {
      idx[t * top + k] = 0;
      w[t * top + k] = 0.f;
    }
#pragma unroll
    for (int i = 0; i < PER; i++)
      if (lane + 64 * i == be) {
        idx[t * top + k] = be;
        if (!rule.renorm) w[t * top + k] = s[i];
        c[i] = -INFINITY;
      }
    if (rule.renorm) {                                              // the winner's score to every lane
      float sv = 0.f;
#pragma unroll
      for (int i = 0; i < PER; i++)
        if (lane + 64 * i == be) sv = s[i];
      if (lane == 0) cs[k] = 0.f;
      wave_sync();
      if (!none && (be & 63) == lane) cs[k] = sv;
      wave_sync();
      total += cs[k];
    }
  }
  if (rule.renorm) {
    const float f = rule.scale / (total + 1e-20f);
    for (int k = lane; k < top; k += 64) w[t * top + k] = cs[k] * f;
  }
}

template <int PER>
__global__ void __launch_bounds__(64) route_groups_k(const float* __restrict__ z, const float* __restrict__ corr,
                                                    RouteRule rule, int E, int top, int groups, int keep, int32_t* __restrict__ idx,
                                                    float* __restrict__ w) {
  __shared__ float cs[64 * PER];                                    // corrected scores
  __shared__ float best[64 * PER];                                  // per group; kept ones become 1, others 0
  const int64_t t = blockIdx.x;
  route_wave<PER>(z + t * E, corr, rule, E, top, groups, keep, idx, w, t, cs, best);
}

// few tokens: the logits as well (f32 products of the router with the token's row, a wave per router output), then the
// first wave routes
template <typename E, int V, int PER>
__global__ void __launch_bounds__(1024) router_k(const E* __restrict__ h, const float* __restrict__ rw,
                                                const float* __restrict__ corr, RouteRule rule, int W, int NE, int top,
                                                int groups, int keep,
                                                int32_t* __restrict__ idx, float* __restrict__ w) {
  __shared__ float cs[64 * PER], best[64 * PER], z[64 * PER];
  const int64_t t = blockIdx.x;
  const int lane = threadIdx.x & 63, wv = threadIdx.x >> 6, NW = blockDim.x >> 6;
  for (int e = wv; e < NE; e += NW) {
    float s = 0.f;
#pragma unroll 4
    for (int c = V * lane; c < W; c += V * 64) {
      float a[V], b[V];
      Vec<E, V>::ld(h + t * W + c, a);
      Vec<float, V>::ld(rw + (int64_t)e * W + c, b);
#pragma unroll
      for (int i = 0; i < V; i++) s = fmaf(a[i], b[i], s);
    }
    s = wave_sum(s);
    if (lane == 0) z[e] = s;
  }
  __syncthreads();
  if (wv == 0) route_wave<PER>(z, corr, rule, NE, top, groups, keep, idx, w, t, cs, best);
}

int row_threads(int W, int V) {
  const int n = (W + V - 1) / V;
  return n >= 1024 ? 1024 : (n + 63) / 64 * 64;
}

}  // namespace

#define SX_V(W, CALL1, CALL4) \
  if ((W) % 4 == 0) {         \
    CALL4;                    \
  } else {                    \
    CALL1;                    \
  }
#define SX_GRID(V) dim3(T, ((W + (V)-1) / (V) + 255) / 256), 256, 0, st

void dyn_tanh(bool bf16, const float* x, Norm n, void* out, int T, int W, hipStream_t st) {
  if (T <= 0) return;
#define CALL(E, V) (dyn_tanh_k<E, V><<<SX_GRID(V)>>>(x, n, (E*)out, W))
  if (bf16) { SX_V(W, CALL(__bf16, 1), CALL(__bf16, 4)) } else { SX_V(W, CALL(float, 1), CALL(float, 4)) }
#undef CALL
}

void add_normed(bool bf16, float* x, const void* y, bool y_f32, Norm post, Norm pre, void* out, int T, int W,
                hipStream_t st) {
  if (T <= 0) return;
#define CALL(E, Y, V) (add_normed_k<E, Y, V><<<SX_GRID(V)>>>(x, (const Y*)y, post, pre, (E*)out, W))
  if (!bf16) { SX_V(W, CALL(float, float, 1), CALL(float, float, 4)) }
  else if (y_f32) { SX_V(W, CALL(__bf16, float, 1), CALL(__bf16, float, 4)) }
  else { SX_V(W, CALL(__bf16, __bf16, 1), CALL(__bf16, __bf16, 4)) }
#undef CALL
}

void add_normed_pair(bool bf16, float* x, const void* a, const void* b, const void* wa, const void* wb, float eps,
                     Norm post, Norm pre, void* out, int T, int W, hipStream_t st) {
  if (T <= 0) return;
#define CALL(E, V)                                                                                                  \
  (add_normed_pair_k<E, V><<<T, row_threads(W, V), 0, st>>>(x, (const E*)a, (const E*)b, (const E*)wa, (const E*)wb, \
                                                            eps, post, pre, (E*)out, W))
  if (bf16) { SX_V(W, CALL(__bf16, 1), CALL(__bf16, 4)) } else { SX_V(W, CALL(float, 1), CALL(float, 4)) }
#undef CALL
}

void add_normed_experts(bool bf16, float* x, const float* rows, const int32_t* idx, const float* wts, const void* h,
                        int top, int experts, Norm post, Norm pre, void* out, int T, int W, hipStream_t st) {
  if (T <= 0) return;
#define CALL(E, V) \
  (add_normed_experts_k<E, V><<<SX_GRID(V)>>>(x, rows, idx, wts, (const E*)h, top, experts, post, pre, (E*)out, W))
  if (bf16) { SX_V(W, CALL(__bf16, 1), CALL(__bf16, 4)) } else { SX_V(W, CALL(float, 1), CALL(float, 4)) }
#undef CALL
}

void rms_sigmoid_gate(bool bf16, const float* o, const void* w, const void* gate, int64_t g_ld, void* out, int T, int C,
                      float eps, hipStream_t st) {
  if (T <= 0) return;
  const int nt = row_threads(C, T > 64 ? 4 : 1);
  if (bf16)
    rms_sigmoid_gate_k<__bf16><<<T, nt, 0, st>>>(o, (const __bf16*)w, (const __bf16*)gate, g_ld, (__bf16*)out, C, eps);
  else
    rms_sigmoid_gate_k<float><<<T, nt, 0, st>>>(o, (const float*)w, (const float*)gate, g_ld, (float*)out, C, eps);
}

void route_groups(const float* z, const float* corr, RouteRule rule, int T, int E, int top, int groups, int keep,
                  int32_t* idx, float* w, hipStream_t st) {
  if (T <= 0) return;
  if (E <= 64) route_groups_k<1><<<T, 64, 0, st>>>(z, corr, rule, E, top, groups, keep, idx, w);
  else route_groups_k<kPerLane><<<T, 64, 0, st>>>(z, corr, rule, E, top, groups, keep, idx, w);
}

void router(bool bf16, const void* h, const float* rw, const float* corr, RouteRule rule, int T, int W, int E, int top,
            int groups, int keep, int32_t* idx, float* w, hipStream_t st) {
  if (T <= 0) return;
  const int nt = 64 * (E < 16 ? E : 16);
#define CALL_P(EL, V, P) \
  (router_k<EL, V, P><<<T, nt, 0, st>>>((const EL*)h, rw, corr, rule, W, E, top, groups, keep, idx, w))
#define CALL(EL, V)        \
  if (E <= 64) {           \
    CALL_P(EL, V, 1);      \
  } else {                 \
    CALL_P(EL, V, kPerLane); \
  }
  if (bf16) { SX_V(W, CALL(__bf16, 1), CALL(__bf16, 4)) } else { SX_V(W, CALL(float, 1), CALL(float, 4)) }
#undef CALL_P
#undef CALL
}

}  // namespace sx
}  // namespace illm
