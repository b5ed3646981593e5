// Masked grouped-query attention over paged [keys | values] rows (gfx950,
// wave64).
//
//   norm + rotary + append   one workgroup per token: the sums of squares of
//                            every head (per-head norm) or of the whole
//                            projection, then every value normed, turned with
//                            its partner and written: queries as f32, keys
//                            and values into the token's cache row
//   attention                one workgroup: one query token x up to HB query
//                            heads of one key head.  Its waves walk the
//                            token's visible key tiles (16 keys, always inside
//                            one cache page) round-robin from the tile that
//                            holds the first visible key; a wave stages keys
//                            and values of the tile in LDS, four lanes share a
//                            key's dot product with every head (f32 queries,
//                            never rounded), the wave does the online-softmax
//                            update per head and every lane accumulates its
//                            value columns.  The waves' partial (max, sum,
//                            out) are merged through LDS; the sink enters the
//                            denominator at the very end (after the merge of
//                            the key splits, if any)
//   chunk softmax            the softmax (sink, causal inside the chunk)
//                            between the batched library products of whole
//                            chunks
//
// Activations are bf16 or f32 (template E); accumulation is always f32.
#include "maskattn.h"

#include <math.h>

namespace illm {
namespace ma {
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
__device__ __forceinline__ float wave_max(float v) {
#pragma unroll
  for (int o = 32; o > 0; o >>= 1) v = fmaxf(v, __shfl_xor(v, o, 64));
  return v;
}
__device__ __forceinline__ void wave_sync() {
  __builtin_amdgcn_fence(__ATOMIC_RELEASE, "wavefront");
  __builtin_amdgcn_wave_barrier();
  __builtin_amdgcn_fence(__ATOMIC_ACQUIRE, "wavefront");
}
__device__ __forceinline__ float block_sum(float v, float* red) {
  v = wave_sum(v);
  const int w = threadIdx.x >> 6, nw = (blockDim.x + 63) >> 6;
  __syncthreads();
  if ((threadIdx.x & 63) == 0) red[w] = v;
  __syncthreads();
  float s = 0.f;
  for (int i = 0; i < nw; i++) s += red[i];
  return s;
}

// ------------------------------------------------------------------ norm + rotary + append
// hs: LDS [H + G] sums of squares per head
template <typename EI, typename E>
__device__ __forceinline__ float normed(const EI* x, int i, int head, int d, const E* nw, bool whole, float rs) {
  float v = ldf(x + i);
  if (nw) v = v * rs * ldf(nw + (whole ? head * d + i : i));
  return v;
}

// EI: element type of the projected q / k / v (f32 when a convolution came first), E: of the norm weights and the rows
template <typename EI, typename E>
__global__ void __launch_bounds__(1024) qkv_store_k(const EI* __restrict__ q, int64_t q_ld, const EI* __restrict__ k,
                                                  int64_t k_ld, const EI* __restrict__ v, int64_t v_ld,
                                                  const E* __restrict__ qn, const E* __restrict__ kn, bool whole,
                                                  float eps, const float* __restrict__ table, int dims, int layout,
                                                  const int64_t* __restrict__ pos, const int64_t* __restrict__ slots,
                                                  E* __restrict__ rows, float* __restrict__ qo,
                                                  const float* __restrict__ temp, int H, int G, int d, int dv) {
  extern __shared__ float hs[];                                     // [H + G] (+ 2 totals)
  const int64_t t = blockIdx.x;
  const int lane = threadIdx.x & 63, wv = threadIdx.x >> 6, NW = blockDim.x >> 6;
  const int NH = H + (k ? G : 0);
  const EI* qr = q + t * q_ld;
  const EI* kr = k ? k + t * k_ld : nullptr;
  for (int hh = wv; hh < NH; hh += NW) {
    const EI* x = hh < H ? qr + hh * d : kr + (hh - H) * d;
    float s = 0.f;
    for (int i = lane; i < d; i += 64) {
      const float a = ldf(x + i);
      s += a * a;
    }
    s = wave_sum(s);
    if (lane == 0) hs[hh] = s;
  }
  __syncthreads();
  if (whole && threadIdx.x == 0) {                                  // fixed order: the same sum whatever the launch
    float a = 0.f, b = 0.f;
    for (int i = 0; i < H; i++) a += hs[i];
    for (int i = H; i < NH; i++) b += hs[i];
    hs[NH] = a;
    hs[NH + 1] = b;
  }
  __syncthreads();
  const int64_t p = pos[t];
  const float* cs = table ? table + p * dims : nullptr;             // [dims / 2][2]
  const int half = dims >> 1;
  E* row = k ? rows + slots[t] * ((int64_t)G * (d + dv)) : nullptr;
  for (int e = threadIdx.x; e < NH * d; e += blockDim.x) {
    const int hh = e / d, i = e - hh * d;
    const bool isq = hh < H;
    const int head = isq ? hh : hh - H;
    const EI* x = isq ? qr + head * d : kr + head * d;
    const E* nw = isq ? qn : kn;
    float rs = 1.f;
    if (nw) rs = whole ? 1.0f / sqrtf(hs[isq ? NH : NH + 1] / (float)((isq ? H : G) * d) + eps)
                       : 1.0f / sqrtf(hs[hh] / (float)d + eps);
    float val = normed(x, i, head, d, nw, whole, rs);
    if (cs && i < dims) {
      int pi, partner;
      bool first;
      if (layout == kHalf) {
        first = i < half;
        pi = first ? i : i - half;
        partner = first ? i + half : i - half;
      } else {
        first = !(i & 1);
        pi = i >> 1;
        partner = i ^ 1;
      }
      const float other = normed(x, partner, head, d, nw, whole, rs);
      const float c = cs[2 * pi], s = cs[2 * pi + 1];
      val = first ? val * c - other * s : val * c + other * s;
    }
    if (isq) qo[(t * H + head) * d + i] = temp ? val * temp[head] : val;
    else stf(row + head * d + i, val);
  }
  if (k)
    for (int e = threadIdx.x; e < G * dv; e += blockDim.x) stf(row + (int64_t)G * d + e, ldf(v + t * v_ld + e));
}

// the same step for per-head norms (or none): eight neighbouring values per lane, LPH lanes per head (a power of two),
// 64 / LPH heads per wave, every value read once (d and dv multiples of 8, d <= 8 LPH).  HALF: half-split pairs (dims a
// multiple of 16: a value's partner sits in the same place of another lane), otherwise neighbouring pairs
template <typename E> struct Eight {
  typedef E V8 __attribute__((ext_vector_type(8)));
  static __device__ __forceinline__ void ld(const E* p, float* v) {
    const V8 a = *(const V8*)p;
#pragma unroll
    for (int i = 0; i < 8; i++) v[i] = (float)a[i];
  }
  static __device__ __forceinline__ void st(E* p, const float* v) {
    V8 a;
#pragma unroll
    for (int i = 0; i < 8; i++) a[i] = (E)v[i];
    *(V8*)p = a;
  }
};

template <typename EI, typename E, int LPH, bool HALF>
__global__ void __launch_bounds__(512) qkv_store_pairs_k(const EI* __restrict__ q, int64_t q_ld, const EI* __restrict__ k,
                                                        int64_t k_ld, const EI* __restrict__ v, int64_t v_ld,
                                                        const E* __restrict__ qn, const E* __restrict__ kn, float eps,
                                                        const float* __restrict__ table, int dims,
                                                        const int64_t* __restrict__ pos, const int64_t* __restrict__ slots,
                                                        E* __restrict__ rows, float* __restrict__ qo,
                                                        const float* __restrict__ temp, int H, int G, int d, int dv) {
  const int64_t t = blockIdx.x;
  const int ln = threadIdx.x & (LPH - 1), i0 = 8 * ln;
  const int NK = H + (k ? G : 0), per = blockDim.x / LPH;           // heads per pass
  E* row = k ? rows + slots[t] * ((int64_t)G * (d + dv)) : nullptr;
  float cs[HALF ? 16 : 8];                                          // this lane's pairs: (cos, sin)
  const bool turn = table && i0 < dims;
  const bool first = i0 < dims / 2;                                 // half-split: the pairs' first values
  const int mate = (threadIdx.x & 63) + (turn ? (first ? dims / 16 : -dims / 16) : 0);
  if (HALF && turn) {
    const float* p = table + pos[t] * dims + 2 * (first ? i0 : i0 - dims / 2);
#pragma unroll
    for (int i = 0; i < 16; i += 4) {
      const float4 r = *(const float4*)(p + i);
      cs[i] = r.x, cs[i + 1] = r.y, cs[i + 2] = r.z, cs[i + 3] = r.w;
    }
  } else if (turn) {
    const float* p = table + pos[t] * dims + i0;
#pragma unroll
    for (int i = 0; i < 8; i += 2) {
      const float2 r = i0 + i < dims ? *(const float2*)(p + i) : make_float2(1.f, 0.f);
      cs[i] = r.x;
      cs[i + 1] = r.y;
    }
  }
  const bool in = i0 < d;
  const bool normed = qn || kn;
  for (int h0 = 0; h0 < NK; h0 += per) {
    const int hh = h0 + threadIdx.x / LPH;
    const bool isq = hh < H, ok = in && hh < NK;
    float a[8];
#pragma unroll
    for (int i = 0; i < 8; i++) a[i] = 0.f;
    float ss = 0.f;
    if (ok) {
      Eight<EI>::ld(isq ? q + t * q_ld + (int64_t)hh * d + i0 : k + t * k_ld + (int64_t)(hh - H) * d + i0, a);
#pragma unroll
      for (int i = 0; i < 8; i++) ss = fmaf(a[i], a[i], ss);
    }
    if (normed) {
#pragma unroll
      for (int o = LPH / 2; o > 0; o >>= 1) ss += __shfl_xor(ss, o, 64);
    }
    const E* nw = isq ? qn : kn;
    if (ok && nw) {
      const float rs = 1.0f / sqrtf(ss / (float)d + eps);
      float w[8];
      Eight<E>::ld(nw + i0, w);
#pragma unroll
      for (int i = 0; i < 8; i++) a[i] = a[i] * rs * w[i];
    }
    if (HALF) {                                                     // (every lane takes part in the exchange)
#pragma unroll
      for (int i = 0; i < 8; i++) {
        const float other = __shfl(a[i], mate, 64);
        if (turn) a[i] = first ? a[i] * cs[2 * i] - other * cs[2 * i + 1] : a[i] * cs[2 * i] + other * cs[2 * i + 1];
      }
    } else if (turn) {
#pragma unroll
      for (int i = 0; i < 8; i += 2) {
        const float n0 = a[i] * cs[i] - a[i + 1] * cs[i + 1];
        a[i + 1] = a[i + 1] * cs[i] + a[i] * cs[i + 1];
        a[i] = n0;
      }
    }
    if (!ok) continue;
    if (isq) {
      if (temp) {
        const float f = temp[hh];
#pragma unroll
        for (int i = 0; i < 8; i++) a[i] *= f;
      }
      Eight<float>::st(qo + (t * H + hh) * d + i0, a);
    } else {
      Eight<E>::st(row + (int64_t)(hh - H) * d + i0, a);
    }
  }
  if (k)
    for (int e = 8 * threadIdx.x; e < G * dv; e += 8 * blockDim.x) {
      float a[8];
      Eight<EI>::ld(v + t * v_ld + e, a);
      Eight<E>::st(row + (int64_t)G * d + e, a);
    }
}

// ------------------------------------------------------------------ attention
constexpr int KT = 16;                                              // keys per tile

__device__ __forceinline__ int64_t first_key(int64_t p, int mask, int size) {
  if (mask == kWindow) return p - size + 1 > 0 ? p - size + 1 : 0;
  if (mask == kChunk) return p - p % size;
  return 0;
}

template <typename E> struct Chunk4;
template <> struct Chunk4<float> { typedef uint4 type; };
template <> struct Chunk4<__bf16> { typedef uint2 type; };

// LDS: qs f32 [HB][DQ] | per wave: tile E [KT][DP] (key d | value dv), weights f32 [HB][KT]
template <typename E, int RC, int HB>
__global__ void __launch_bounds__(256) masked_attn_k(const float* __restrict__ q, const E* __restrict__ rows, int bs,
                                                    const int32_t* __restrict__ bt, int bt_w,
                                                    const int32_t* __restrict__ seq_of, const int64_t* __restrict__ pos,
                                                    float scale, int mask, int size, const float* __restrict__ sink,
                                                    E* __restrict__ out, float* __restrict__ part, int H, int G, int d,
                                                    int dv, int DQ, int DP, float softcap, int keep, int cross) {
  extern __shared__ __align__(16) unsigned char smem[];
  typedef typename Chunk4<E>::type C4;
  const int rep = H / G;
  const int nhb = (rep + HB - 1) / HB;                              // head blocks per key head
  const int nsplit = gridDim.z, zs = blockIdx.z;
  // cross: the heads' weights are applied to the values of EVERY value head (grid y also walks the value heads); the
  // unnormalised partial results leave through ``part`` and the mixing of the heads follows in the combine kernel
  const int by = cross ? blockIdx.y / G : blockIdx.y;
  const int t = blockIdx.x, g = by / nhb, h0 = g * rep + (by % nhb) * HB;
  const int vg = cross ? blockIdx.y % G : g;
  const int nh = min(HB, g * rep + rep - h0);
  const int lane = threadIdx.x & 63, wv = threadIdx.x >> 6, NW = blockDim.x >> 6;
  float* qs = (float*)smem;
  const size_t q_bytes = (size_t)HB * DQ * sizeof(float);
  const size_t tile_bytes = ((size_t)KT * DP * sizeof(E) + 15) & ~(size_t)15;
  const size_t wave_bytes = tile_bytes + (size_t)HB * KT * sizeof(float);
  unsigned char* wbase = smem + q_bytes + wv * wave_bytes;
  E* kt = (E*)wbase;                                                // [KT][DP]
  float* pb = (float*)(wbase + tile_bytes);                         // [HB][KT]
  for (int i = threadIdx.x; i < HB * DQ; i += blockDim.x) {
    const int h = i / DQ, c = i - h * DQ;
    qs[i] = (h < nh && c < d) ? q[((int64_t)t * H + h0 + h) * d + c] : 0.f;
  }
  for (int i = lane; i < KT * DP; i += 64) stf(kt + i, 0.f);        // pad columns and unfilled rows stay finite
  __syncthreads();
  const int64_t p = pos[t];
  const int64_t lo = first_key(p, mask, size);
  const int32_t* tab = bt + (int64_t)seq_of[t] * bt_w;
  const int tile0 = (int)(lo / KT), ntiles = (int)(p / KT) + 1;
  // a window that keeps the sequence's first tokens: their tiles (those before the window's first) are walked first
  const int nkeep = keep > 0 ? min(tile0, (keep + KT - 1) / KT) : 0;
  const int nwalk = nkeep + ntiles - tile0;
  const int64_t RW = (int64_t)G * (d + dv);                         // cache row width
  const int D = d + dv;
  float m[HB], l[HB], o[HB][RC];
#pragma unroll
  for (int h = 0; h < HB; h++) {
    m[h] = -INFINITY;
    l[h] = 0.f;
#pragma unroll
    for (int c = 0; c < RC; c++) o[h][c] = 0.f;
  }
  const int kj = lane & (KT - 1), grp = lane / KT;                  // 4 lanes share a key
  const int d4 = (d + 3) >> 2;                                      // 4-element steps of a key (LDS pad is zero)
  for (int it = zs * NW + wv; it < nwalk; it += NW * nsplit) {
    const int ti = it < nkeep ? it : tile0 + (it - nkeep);
    const int64_t k0 = (int64_t)ti * KT;
    const int nvalid = (int)min((int64_t)KT, p - k0 + 1);
    const int64_t row0 = (int64_t)tab[k0 / bs] * bs + (k0 % bs);
    if (((d | dv) & 3) == 0) {
      // 4-element chunks (the key part, then the value part of every row), four requests in flight per lane
      const int cd = d >> 2, cpr = (d + dv) >> 2, n4 = nvalid * cpr;
      for (int i0 = lane; i0 < n4; i0 += 256) {
        C4 v[4];
        int dst[4];
#pragma unroll
        for (int u = 0; u < 4; u++) {
          const int i = i0 + 64 * u;
          if (i < n4) {
            const int j = i / cpr, c = i - j * cpr;
            const E* src = rows + (row0 + j) * RW +
                           (c < cd ? (int64_t)g * d + 4 * c : (int64_t)G * d + (int64_t)vg * dv + 4 * (c - cd));
            v[u] = *(const C4*)src;
            dst[u] = j * DP + (c < cd ? 4 * c : DQ + 4 * (c - cd));
          }
        }
#pragma unroll
        for (int u = 0; u < 4; u++)
          if (i0 + 64 * u < n4) *(C4*)(kt + dst[u]) = v[u];
      }
    } else {
      for (int i = lane; i < nvalid * D; i += 64) {
        const int j = i / D, c = i - j * D;
        const E* src = rows + (row0 + j) * RW + (c < d ? (int64_t)g * d + c : (int64_t)G * d + (int64_t)vg * dv + (c - d));
        kt[j * DP + (c < d ? c : DQ + (c - d))] = *src;
      }
    }
    wave_sync();
    float s[HB];
#pragma unroll
    for (int h = 0; h < HB; h++) s[h] = 0.f;
    const bool valid = kj < nvalid && (k0 + kj >= lo || k0 + kj < keep);
    if (valid) {
      const E* kr = kt + kj * DP;
      for (int c4 = grp * d4 / 4; c4 < (grp + 1) * d4 / 4; c4++) {
        const int c = c4 * 4;
        const float k0v = ldf(kr + c), k1v = ldf(kr + c + 1), k2v = ldf(kr + c + 2), k3v = ldf(kr + c + 3);
#pragma unroll
        for (int h = 0; h < HB; h++) {
          const float4 qv = *(const float4*)(qs + h * DQ + c);
          s[h] = fmaf(qv.x, k0v, fmaf(qv.y, k1v, fmaf(qv.z, k2v, fmaf(qv.w, k3v, s[h]))));
        }
      }
    }
#pragma unroll
    for (int h = 0; h < HB; h++) {
      s[h] += __shfl_xor(s[h], 16, 64);
      s[h] += __shfl_xor(s[h], 32, 64);
    }
#pragma unroll
    for (int h = 0; h < HB; h++) {
      float sv = s[h] * scale;
      if (softcap > 0.f) sv = softcap * tanhf(sv / softcap);
      if (!valid) sv = -INFINITY;
      const float mn = fmaxf(m[h], wave_max(sv));
      const float alpha = m[h] == -INFINITY ? 0.f : expf(m[h] - mn);
      const float pv = valid ? expf(sv - mn) : 0.f;
      l[h] = l[h] * alpha + wave_sum(lane < KT ? pv : 0.f);
      m[h] = mn;
#pragma unroll
      for (int c = 0; c < RC; c++) o[h][c] *= alpha;
      if (lane < KT) pb[h * KT + lane] = pv;
    }
    wave_sync();
    const int nv4 = (nvalid + 3) & ~3;                              // weights past nvalid are 0, rows finite
    for (int j = 0; j < nv4; j += 4) {
      float vv[4][RC];
#pragma unroll
      for (int jj = 0; jj < 4; jj++)
#pragma unroll
        for (int c = 0; c < RC; c++) {
          const int col = lane + 64 * c;
          vv[jj][c] = col < dv ? ldf(kt + (j + jj) * DP + DQ + col) : 0.f;
        }
#pragma unroll
      for (int h = 0; h < HB; h++) {
        const float4 w4 = *(const float4*)(pb + h * KT + j);
#pragma unroll
        for (int c = 0; c < RC; c++)
          o[h][c] = fmaf(w4.x, vv[0][c], fmaf(w4.y, vv[1][c], fmaf(w4.z, vv[2][c], fmaf(w4.w, vv[3][c], o[h][c]))));
      }
    }
    wave_sync();
  }
  // merge the waves through the (re-used) LDS: every wave leaves (o, m, l) per head
  __syncthreads();
  const int MS = HB * (dv + 2);
  float* mg = (float*)smem + (size_t)wv * MS;
#pragma unroll
  for (int h = 0; h < HB; h++) {
#pragma unroll
    for (int c = 0; c < RC; c++) {
      const int col = lane + 64 * c;
      if (col < dv) mg[h * (dv + 2) + col] = o[h][c];
    }
    if (lane == 0) {
      mg[h * (dv + 2) + dv] = m[h];
      mg[h * (dv + 2) + dv + 1] = l[h];
    }
  }
  __syncthreads();
  const float* m0 = (const float*)smem;
  for (int i = threadIdx.x; i < nh * (dv + 2); i += blockDim.x) {
    const int h = i / (dv + 2), c = i - h * (dv + 2);
    float M = -INFINITY;
    for (int w = 0; w < NW; w++) M = fmaxf(M, m0[(size_t)w * MS + h * (dv + 2) + dv]);
    float L = 0.f, O = 0.f;
    for (int w = 0; w < NW; w++) {
      const float* gp = m0 + (size_t)w * MS + h * (dv + 2);
      const float mw = gp[dv];
      const float f = mw == -INFINITY ? 0.f : expf(mw - M);
      L += gp[dv + 1] * f;
      if (c < dv) O += gp[c] * f;
    }
    if (cross) {
      float* pp = part + ((((int64_t)t * H + h0 + h) * G + vg) * nsplit + zs) * (dv + 2);
      pp[c] = c < dv ? O : (c == dv ? M : L);
    } else if (nsplit > 1) {
      float* pp = part + (((int64_t)t * H + h0 + h) * nsplit + zs) * (dv + 2);
      pp[c] = c < dv ? O : (c == dv ? M : L);
    } else if (c < dv) {
      if (sink) {                                                   // one more term of the denominator
        const float sk = sink[h0 + h];
        const float M2 = fmaxf(M, sk);
        const float f = expf(M - M2);
        O *= f;
        L = L * f + expf(sk - M2);
      }
      stf(out + ((int64_t)t * H + h0 + h) * dv + c, O / L);
    }
  }
}

// merge of the key splits: part [T, H, nsplit, dv + 2] -> out [T, H, dv].  One wave per (token, head): lane z
// holds split z's (max, sum) (nsplit <= 64), the wave reduces them, then every lane sums its value columns
template <typename E>
__global__ void __launch_bounds__(64) masked_attn_combine_k(const float* __restrict__ part, const float* __restrict__ sink,
                                                           E* __restrict__ out, int H, int dv, int nsplit) {
  __shared__ float wz[64];
  const int64_t th = (int64_t)blockIdx.x * H + blockIdx.y;
  const float* pp = part + th * nsplit * (dv + 2);
  const int lane = threadIdx.x;
  const float mz = lane < nsplit ? pp[(size_t)lane * (dv + 2) + dv] : -INFINITY;
  const float lz = lane < nsplit ? pp[(size_t)lane * (dv + 2) + dv + 1] : 0.f;
  const float sk = sink ? sink[blockIdx.y] : -INFINITY;
  const float M = fmaxf(wave_max(mz), sk);
  const float f = mz == -INFINITY ? 0.f : expf(mz - M);
  wz[lane] = f;
  // the splits' sums in index order (a fixed order, whatever the lanes do)
  __syncthreads();
  float L = sink ? expf(sk - M) : 0.f;
  for (int z = 0; z < nsplit; z++) L += __shfl(lz, z, 64) * wz[z];
  const float inv = 1.0f / L;
  for (int c = lane; c < dv; c += 64) {
    float O = 0.f;
    for (int z = 0; z < nsplit; z++) O = fmaf(pp[(size_t)z * (dv + 2) + c], wz[z], O);
    stf(out + th * dv + c, O * inv);
  }
}

// merge of the key splits and mixing of the heads' weights after the softmax:
//   out[t, h] = sum_g talk[h, g] (sum_j w_g(j) value_j[c])   with c = h's value head,
// part [T, H, G, nsplit, dv + 2] holds, for query head g and value head c, the unnormalised sums of every key split.
// One wave per (token, output head); dv <= 512
template <typename E>
__global__ void __launch_bounds__(512) masked_attn_talk_combine_k(const float* __restrict__ part,
                                                                 const float* __restrict__ sink,
                                                                 const float* __restrict__ talk, E* __restrict__ out,
                                                                 int H, int G, int dv, int nsplit) {
  extern __shared__ float cs[];                                     // [NW][64] split factors, then [NW][dv] sums
  const int64_t t = blockIdx.x;
  const int h = blockIdx.y, c = h / (H / G), lane = threadIdx.x & 63, wv = threadIdx.x >> 6, NW = blockDim.x >> 6;
  float* wz = cs + wv * 64;
  float* sums = cs + NW * 64;
  float acc[8];
#pragma unroll
  for (int i = 0; i < 8; i++) acc[i] = 0.f;
  for (int g = wv; g < H; g += NW) {                                // wave w: source heads w, w + NW, ...
    const float* pp = part + ((t * H + g) * G + c) * (int64_t)nsplit * (dv + 2);
    const float mz = lane < nsplit ? pp[(size_t)lane * (dv + 2) + dv] : -INFINITY;
    const float lz = lane < nsplit ? pp[(size_t)lane * (dv + 2) + dv + 1] : 0.f;
    const float sk = sink ? sink[g] : -INFINITY;
    const float M = fmaxf(wave_max(mz), sk);
    const float f = mz == -INFINITY ? 0.f : expf(mz - M);
    wave_sync();
    wz[lane] = f;
    wave_sync();
    float L = sink ? expf(sk - M) : 0.f;
    for (int z = 0; z < nsplit; z++) L += __shfl(lz, z, 64) * wz[z];   // index order, whatever the lanes do
    const float coef = talk[h * H + g] / L;
#pragma unroll
    for (int i = 0; i < 8; i++) {
      const int col = lane + 64 * i;
      if (col < dv) {
        float O = 0.f;
        for (int z = 0; z < nsplit; z++) O = fmaf(pp[(size_t)z * (dv + 2) + col], wz[z], O);
        acc[i] = fmaf(coef, O, acc[i]);
      }
    }
  }
#pragma unroll
  for (int i = 0; i < 8; i++) {
    const int col = lane + 64 * i;
    if (col < dv) sums[wv * dv + col] = acc[i];
  }
  __syncthreads();
  for (int col = threadIdx.x; col < dv; col += blockDim.x) {
    float o = 0.f;
    for (int w = 0; w < NW; w++) o += sums[w * dv + col];           // the waves in order
    stf(out + (t * H + h) * dv + col, o);
  }
}

// mixing of the heads' weights between the chunk products: w f32 [pieces, G, Lq, rep, L] (normalised softmax
// weights) -> mixed weights of the same layout, w'[.., h, ..] = sum_g talk[h, g] w[.., g, ..] with h = key head * rep +
// r; bf16: as pairs hi + lo in hl [R, 2 L] (a row's hi halves, then its lo halves); f32: out32 [R, L].
// A thread per key column, the piece-and-query's H weights of that column staged in LDS
template <typename E>
__global__ void __launch_bounds__(64) talk_mix_k(const float* __restrict__ w, const float* __restrict__ talk, int Lq, int L,
                                                int G, int rep, E* __restrict__ hl, float* __restrict__ out32) {
  extern __shared__ float col[];                                    // [H][64]
  const int H = G * rep;
  const int piece = blockIdx.x / Lq, qi = blockIdx.x % Lq;
  const int j = blockIdx.y * 64 + threadIdx.x;
  if (j >= L) return;
  const int64_t prow = (int64_t)piece * G * Lq * rep;
  for (int g = 0; g < H; g++) {
    const int64_t row = prow + ((int64_t)(g / rep) * Lq + qi) * rep + g % rep;
    col[g * 64 + threadIdx.x] = w[row * L + j];
  }
  for (int h = 0; h < H; h++) {
    float a = 0.f;
    for (int g = 0; g < H; g++) a = fmaf(talk[h * H + g], col[g * 64 + threadIdx.x], a);
    const int64_t row = prow + ((int64_t)(h / rep) * Lq + qi) * rep + h % rep;
    if (hl) {
      const E hv = (E)a;
      hl[row * 2 * L + j] = hv;
      hl[row * 2 * L + L + j] = (E)(a - (float)hv);
    } else {
      out32[row * L + j] = a;
    }
  }
}

// ------------------------------------------------------------------ softmax between the chunk products
// window == 0: a piece of a chunk (query tok sees keys 0 .. L - Lq + tok).  window > 0: a block of queries of a
// sliding window: query tok stands at position q0 + tok; the first nkeep columns are kept first tokens (always
// visible), column nkeep + jj is the key at position k0 + jj, visible when it is not ahead of the query and inside
// the window (or before position ``keep``)
// KEEP > 0: 4-value accesses, the row stays in registers between the passes (L a multiple of 4, at most 1024 KEEP)
template <typename E, int KEEP>
__global__ void __launch_bounds__(256) chunk_softmax_k(float* __restrict__ sc, int Lq, int L, int G, int rep, float scale,
                                                      const float* __restrict__ sink, E* __restrict__ hi, float softcap,
                                                      int window, int keep, int nkeep, int64_t q0, int64_t k0) {
  __shared__ float red[16];
  const int64_t row = blockIdx.x;
  const int tok = (int)((row / rep) % Lq);                          // the piece's queries are its last Lq positions
  const int h = (int)((row / ((int64_t)rep * Lq)) % G) * rep + (int)(row % rep);
  const int64_t p = q0 + tok;
  const int nk = window > 0 ? (int)min((int64_t)L, nkeep + (p - k0) + 1) : L - Lq + tok + 1;
  // the first column of the window's own keys (columns nkeep .. first - 1 are seen only if kept)
  const int first = window > 0 ? nkeep + (int)max((int64_t)0, p - window + 1 - k0) : 0;
  auto vis = [&](int j) -> bool { return window <= 0 || j < nkeep || j >= first || k0 + (j - nkeep) < keep; };
  float* s = sc + row * L;
  const float sk = sink ? sink[h] : -INFINITY;
  float mx = sk;
  constexpr int NK = KEEP > 0 ? KEEP : 1;
  float v[NK][4];
  auto cap = [&](float x) { return softcap > 0.f ? softcap * tanhf(x / softcap) : x; };
  if (KEEP > 0) {
#pragma unroll
    for (int k = 0; k < KEEP; k++) {
      const int j = 4 * (threadIdx.x + 256 * k);
#pragma unroll
      for (int i = 0; i < 4; i++) v[k][i] = -INFINITY;
      if (j < nk) {
        const float4 a = *(const float4*)(s + j);
        const float t[4] = {a.x, a.y, a.z, a.w};
#pragma unroll
        for (int i = 0; i < 4; i++)
          if (j + i < nk && vis(j + i)) {
            v[k][i] = cap(t[i] * scale);
            mx = fmaxf(mx, v[k][i]);
          }
      }
    }
  } else {
    for (int j = threadIdx.x; j < nk; j += blockDim.x) {
      const float x = vis(j) ? cap(s[j] * scale) : -INFINITY;
      s[j] = x;
      mx = fmaxf(mx, x);
    }
  }
  mx = wave_max(mx);
  __syncthreads();
  if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = mx;
  __syncthreads();
  for (int i = 0; i < (int)(blockDim.x >> 6); i++) mx = fmaxf(mx, red[i]);
  float sum = 0.f;
  if (KEEP > 0) {
#pragma unroll
    for (int k = 0; k < KEEP; k++)
#pragma unroll
      for (int i = 0; i < 4; i++) {
        v[k][i] = expf(v[k][i] - mx);                              // a masked column: exp(-inf) = 0
        sum += v[k][i];
      }
  } else {
    for (int j = threadIdx.x; j < nk; j += blockDim.x) {
      const float e = expf(s[j] - mx);
      s[j] = e;
      sum += e;
    }
  }
  const float inv = 1.0f / (block_sum(sum, red) + (sink ? expf(sk - mx) : 0.f));
  if (KEEP > 0) {
#pragma unroll
    for (int k = 0; k < KEEP; k++) {
      const int j = 4 * (threadIdx.x + 256 * k);
      if (j >= L) continue;
#pragma unroll
      for (int i = 0; i < 4; i++) v[k][i] *= inv;
      if (hi) {                                                     // [R, 2 L]: hi halves, then lo halves
        typedef E E4 __attribute__((ext_vector_type(4)));
        E4 h4, l4;
#pragma unroll
        for (int i = 0; i < 4; i++) {
          h4[i] = (E)v[k][i];
          l4[i] = (E)(v[k][i] - (float)h4[i]);
        }
        *(E4*)(hi + row * 2 * L + j) = h4;
        *(E4*)(hi + row * 2 * L + L + j) = l4;
      } else {
        *(float4*)(s + j) = make_float4(v[k][0], v[k][1], v[k][2], v[k][3]);
      }
    }
    return;
  }
  for (int j = threadIdx.x; j < L; j += blockDim.x) {
    const float w = j < nk ? s[j] * inv : 0.f;
    if (hi) {                                                      // [R, 2 L]: hi halves, then lo halves
      const E hv = (E)w;
      hi[row * 2 * L + j] = hv;
      hi[row * 2 * L + L + j] = (E)(w - (float)hv);
    } else {
      s[j] = w;
    }
  }
}

// ------------------------------------------------------------------ operands of the batched products
// a block of queries and the keys it sees as operands of two batched products per key head.  16-bit rows: f32 queries as hi
// and lo halves side by side along the summed axis, so keys (and values, for f32 weights) appear twice
template <typename E>
__global__ void __launch_bounds__(256) pack_queries_k(const float* __restrict__ q, int64_t tok0, int nq, E* __restrict__ q2,
                                                     int H, int G, int d) {
  const int rep = H / G, tok = blockIdx.x;
  constexpr int TW = sizeof(E) == 2 ? 2 : 1;
  for (int i = threadIdx.x; i < H * d; i += blockDim.x) {
    const int h = i / d, c = i - h * d, g = h / rep;
    const float v = q[(tok0 + tok) * H * d + i];
    E* o = q2 + (((int64_t)g * nq + tok) * rep + (h - g * rep)) * TW * d;
    const E hi = (E)v;
    o[c] = hi;
    if (TW == 2) o[d + c] = (E)(v - (float)hi);
  }
}

// column j: position j below nkeep, then k0, k0 + 1, ... (past the last key: that one again).  k2 [G, TW d, nk], v2 [G, TW nk,
// dv]; a workgroup per 64 columns of a key head and 64 channels of its keys (turned through LDS) or of its values.  V values
// per access (4: d, dv and nk are multiples of 4)
template <typename E, int V>
__global__ void __launch_bounds__(256) pack_keys_k(const E* __restrict__ rows, int bs, const int32_t* __restrict__ tab,
                                                  int nkeep, int64_t k0, int nr, int nk, E* __restrict__ k2,
                                                  E* __restrict__ v2, int G, int d, int dv) {
  constexpr int TW = sizeof(E) == 2 ? 2 : 1;
  typedef E EV __attribute__((ext_vector_type(V)));
  __shared__ E tile[64][65];
  __shared__ int64_t at[64];
  const int j0 = blockIdx.x * 64, g = blockIdx.y, nj = min(64, nk - j0), kc = (d + 63) / 64;
  const int64_t ld = (int64_t)G * (d + dv);
  if (threadIdx.x < 64) {
    const int j = min(j0 + (int)threadIdx.x, nk - 1);
    const int64_t p = j < nkeep ? j : k0 + min(j - nkeep, nr - 1);
    at[threadIdx.x] = ((int64_t)tab[p / bs] * bs + p % bs) * ld;
  }
  __syncthreads();
  if ((int)blockIdx.z < kc) {
    const int c0 = 64 * blockIdx.z, nc = min(64, d - c0);
    for (int i = V * threadIdx.x; i < 64 * 64; i += V * 256) {
      const int j = i >> 6, c = i & 63;
      if (j < nj && c < nc) {
        const EV x = *(const EV*)(rows + at[j] + (int64_t)g * d + c0 + c);
#pragma unroll
        for (int e = 0; e < V; e++) tile[j][c + e] = x[e];
      }
    }
    __syncthreads();
    for (int i = V * threadIdx.x; i < 64 * 64; i += V * 256) {
      const int c = i >> 6, j = i & 63;
      if (j < nj && c < nc) {
        EV x;
#pragma unroll
        for (int e = 0; e < V; e++) x[e] = tile[j + e][c];
#pragma unroll
        for (int w = 0; w < TW; w++) *(EV*)(k2 + ((int64_t)g * TW * d + w * d + c0 + c) * nk + j0 + j) = x;
      }
    }
  } else {
    const int c0 = 64 * (blockIdx.z - kc), nc = min(64, dv - c0);
    for (int i = V * threadIdx.x; i < 64 * 64; i += V * 256) {
      const int j = i >> 6, c = i & 63;
      if (j < nj && c < nc) {
        const EV x = *(const EV*)(rows + at[j] + (int64_t)G * d + (int64_t)g * dv + c0 + c);
#pragma unroll
        for (int w = 0; w < TW; w++) *(EV*)(v2 + ((int64_t)g * TW * nk + (int64_t)w * nk + j0 + j) * dv + c0 + c) = x;
      }
    }
  }
}

// o [G, nq, rep, dv] -> out[tok0 + tok] = [heads in order]
template <typename E>
__global__ void __launch_bounds__(256) unpack_k(const float* __restrict__ o, E* __restrict__ out, int64_t tok0, int nq, int H,
                                               int G, int dv) {
  const int rep = H / G, tok = blockIdx.x;
  for (int i = threadIdx.x; i < H * dv; i += blockDim.x) {
    const int h = i / dv, c = i - h * dv, g = h / rep;
    stf(out + (tok0 + tok) * H * dv + i, o[(((int64_t)g * nq + tok) * rep + (h - g * rep)) * dv + c]);
  }
}

// per: consecutive values that share a gate.  V values per thread (V = 8: 16-byte accesses; C, and per unless it is 1,
// are multiples of 8)
template <typename E, int V>
__global__ void __launch_bounds__(256) sigmoid_gate_k(E* __restrict__ o, const E* __restrict__ g, int64_t g_ld, int64_t n,
                                                     int C, int per) {
  typedef E EV __attribute__((ext_vector_type(V)));
  for (int64_t i = V * ((int64_t)blockIdx.x * blockDim.x + threadIdx.x); i < n; i += V * (int64_t)gridDim.x * blockDim.x) {
    const int64_t t = i / C;
    const int c = (int)(i - t * C);
    EV x = *(const EV*)(o + i);
    if (per > 1) {
      const float f = 1.0f / (1.0f + expf(-ldf(g + t * g_ld + c / per)));
#pragma unroll
      for (int j = 0; j < V; j++) x[j] = (E)((float)x[j] * f);
    } else {
      const EV z = *(const EV*)(g + t * g_ld + c);
#pragma unroll
      for (int j = 0; j < V; j++) x[j] = (E)((float)x[j] / (1.0f + expf(-(float)z[j])));
    }
    *(EV*)(o + i) = x;
  }
}

int pad4(int n) { return (n + 3) & ~3; }
// key | value row of a tile: the key part padded to DQ (a multiple of 4, zero filled), the row to 4 (mod 8) elements
int tile_row(int d, int dv) {
  const int n = pad4(d) + pad4(dv);
  return n + ((12 - (n & 7)) & 7);
}

}  // namespace

void qkv_norm_rope_store(bool in_bf16, bool bf16, const void* q, int64_t q_ld, const void* k, int64_t k_ld,
                         const void* v, int64_t v_ld, const void* qn, const void* kn, bool whole, float eps,
                         const float* table, int max_pos, int dims, int layout, const int64_t* pos, const int64_t* slots,
                         void* rows, int64_t num_rows, float* qo, const float* temp, int T, int H, int G, int d, int dv,
                         hipStream_t st) {
  (void)max_pos;
  (void)num_rows;
  if (T <= 0) return;
  const size_t ei = in_bf16 ? 2 : 4, eo = bf16 ? 2 : 4;
  auto wide = [](const void* p, int64_t ld, size_t eb) { return (uintptr_t)p % (8 * eb) == 0 && ld % 8 == 0; };
  const bool half = table && layout == kHalf;
  if (!whole && (!half || dims % 16 == 0) && d % 8 == 0 && d <= 512 && wide(q, q_ld, ei) && wide(qn, 0, eo) &&
      wide(kn, 0, eo) && (!k || (dv % 8 == 0 && wide(k, k_ld, ei) && wide(v, v_ld, ei) && wide(rows, 0, eo)))) {
    int lph = 1;
    while (8 * lph < d) lph *= 2;
    int nt = (H + (k ? G : 0)) * lph;                               // at most two passes over the heads for few tokens
    nt = (nt + 63) / 64 * 64;
    nt = T > 64 ? (nt > 256 ? 256 : nt) : (nt > 512 ? 512 : nt);
#define MA_PAIRS(EI, E, L)                                                                                              \
  if (half) MA_PAIRS_H(EI, E, L, true); else MA_PAIRS_H(EI, E, L, false)
#define MA_PAIRS_H(EI, E, L, HF)                                                                                        \
  qkv_store_pairs_k<EI, E, L, HF><<<T, nt, 0, st>>>((const EI*)q, q_ld, (const EI*)k, k_ld, (const EI*)v, v_ld,             \
                                                (const E*)qn, (const E*)kn, eps, table, dims, pos, slots, (E*)rows, qo, \
                                                temp, H, G, d, dv)
#define MA_L(EI, E)                      \
  switch (lph) {                         \
    case 1: MA_PAIRS(EI, E, 1); break;   \
    case 2: MA_PAIRS(EI, E, 2); break;   \
    case 4: MA_PAIRS(EI, E, 4); break;   \
    case 8: MA_PAIRS(EI, E, 8); break;   \
    case 16: MA_PAIRS(EI, E, 16); break; \
    case 32: MA_PAIRS(EI, E, 32); break; \
    default: MA_PAIRS(EI, E, 64);        \
  }
    if (bf16 && in_bf16) { MA_L(__bf16, __bf16) }
    else if (bf16) { MA_L(float, __bf16) }
    else { MA_L(float, float) }
#undef MA_L
#undef MA_PAIRS
#undef MA_PAIRS_H
    return;
  }
  const size_t lds = (size_t)(H + G + 2) * sizeof(float);
  // few tokens (decode): a thread per value or two, so that no thread walks a chain of dependent loads
  const int64_t vals = (int64_t)(H + G) * d;
  const int nt = T > 64 ? 256 : (vals >= 1024 ? 1024 : (int)((vals + 63) / 64 * 64));
#define MA_STORE(EI, E)                                                                                                 \
  qkv_store_k<EI, E><<<T, nt, lds, st>>>((const EI*)q, q_ld, (const EI*)k, k_ld, (const EI*)v, v_ld, (const E*)qn,      \
                                         (const E*)kn, whole, eps, table, dims, layout, pos, slots, (E*)rows, qo, temp, \
                                         H, G, d, dv)
  if (bf16 && in_bf16) MA_STORE(__bf16, __bf16);
  else if (bf16) MA_STORE(float, __bf16);
  else MA_STORE(float, float);
#undef MA_STORE
}

int masked_attention_plan(bool bf16, int rep, int d, int dv, int* nw, int* hbo) {
  if (d < 1 || dv < 1 || dv > 512) return -1;
  const int hb = rep >= 8 ? 8 : (rep >= 4 ? 4 : (rep >= 2 ? 2 : 1));
  const size_t eb = bf16 ? 2 : 4;
  const size_t q_bytes = (size_t)hb * pad4(d) * 4;
  const size_t wave = (((size_t)KT * tile_row(d, dv) * eb + 15) & ~(size_t)15) + (size_t)hb * KT * 4;
  for (int w = 4; w >= 1; w--) {
    const size_t tiles = q_bytes + (size_t)w * wave;
    const size_t merge = (size_t)w * hb * (dv + 2) * 4;
    const size_t total = tiles > merge ? tiles : merge;
    if (total <= 64 * 1024) {
      *nw = w;
      *hbo = hb;
      return (int)total;
    }
  }
  return -1;
}

int masked_attention_splits(bool bf16, int T, int H, int G, int d, int dv, int max_keys, bool cross) {
  int NW = 0, hb = 0;
  if (masked_attention_plan(bf16, H / G, d, dv, &NW, &hb) < 0) return 1;
  const int64_t blocks = (int64_t)T * G * ((H / G + hb - 1) / hb) * (cross ? G : 1);
  const int tiles = (max_keys + KT - 1) / KT + 1;
  int ns = (int)((1024 + blocks - 1) / blocks);                    // ~4 workgroups per CU
  ns = ns > (tiles + NW - 1) / NW ? (tiles + NW - 1) / NW : ns;
  return ns < 1 ? 1 : (ns > 64 ? 64 : ns);
}

void masked_attention(bool bf16, const float* q, const void* rows, int bs, const int32_t* block_tables, int bt_width,
                      const int32_t* seq_of, const int64_t* pos, float scale, int mask, int size, const float* sink,
                      void* out, float* part, int nsplit, int T, int H, int G, int d, int dv, float softcap, int keep,
                      const float* talk, hipStream_t st) {
  if (T <= 0) return;
  const int cross = talk ? 1 : 0;
  if (mask != kWindow) keep = 0;
  int NW = 0, hb = 0;
  const int rep = H / G;
  const int lds = masked_attention_plan(bf16, rep, d, dv, &NW, &hb);
  if (lds < 0) return;                       // refused by the caller beforehand
  const int DQ = pad4(d), DP = tile_row(d, dv);
  const int rc = (dv + 63) / 64;
  dim3 grid(T, G * ((rep + hb - 1) / hb) * (cross ? G : 1), nsplit), block(64 * NW);
#define MA_LAUNCH(E, RC, HBV)                                                                                          \
  masked_attn_k<E, RC, HBV><<<grid, block, lds, st>>>(q, (const E*)rows, bs, block_tables, bt_width, seq_of, pos, scale, \
                                                      mask, size, sink, (E*)out, part, H, G, d, dv, DQ, DP, softcap,   \
                                                      keep, cross)
#define MA_RC(E, HBV)                                 \
  if (rc <= 1) MA_LAUNCH(E, 1, HBV);                  \
  else if (rc <= 2) MA_LAUNCH(E, 2, HBV);             \
  else if (rc <= 4) MA_LAUNCH(E, 4, HBV);             \
  else MA_LAUNCH(E, 8, HBV)
#define MA_HB(E)                                      \
  if (hb == 8) { MA_RC(E, 8); }                       \
  else if (hb == 4) { MA_RC(E, 4); }                  \
  else if (hb == 2) { MA_RC(E, 2); }                  \
  else { MA_RC(E, 1); }
  if (bf16) { MA_HB(__bf16) } else { MA_HB(float) }
#undef MA_HB
#undef MA_RC
#undef MA_LAUNCH
  if (cross) {
    const int cw = H < 8 ? H : 8;                                   // waves: each merges some of the source heads
    const size_t cl = (size_t)cw * (64 + dv) * sizeof(float);
    if (bf16)
      masked_attn_talk_combine_k<__bf16><<<dim3(T, H), 64 * cw, cl, st>>>(part, sink, talk, (__bf16*)out, H, G, dv, nsplit);
    else
      masked_attn_talk_combine_k<float><<<dim3(T, H), 64 * cw, cl, st>>>(part, sink, talk, (float*)out, H, G, dv, nsplit);
  } else if (nsplit > 1) {
    if (bf16) masked_attn_combine_k<__bf16><<<dim3(T, H), 64, 0, st>>>(part, sink, (__bf16*)out, H, dv, nsplit);
    else masked_attn_combine_k<float><<<dim3(T, H), 64, 0, st>>>(part, sink, (float*)out, H, dv, nsplit);
  }
}

void chunk_softmax(bool bf16, float* sc, int64_t R, int Lq, int L, int G, int rep, float scale, const float* sink,
                   void* hl, float softcap, int window, int keep, int nkeep, int64_t q0, int64_t k0, hipStream_t st) {
  if (R <= 0 || L <= 0) return;
#define MA_SOFT(E, K) \
  chunk_softmax_k<E, K><<<(unsigned)R, 256, 0, st>>>(sc, Lq, L, G, rep, scale, sink, (E*)hl, softcap, window, keep, nkeep, q0, k0)
  if (L % 4 == 0 && L <= 2048) {
    if (bf16) MA_SOFT(__bf16, 2); else MA_SOFT(float, 2);
  } else if (L % 4 == 0 && L <= 4096) {
    if (bf16) MA_SOFT(__bf16, 4); else MA_SOFT(float, 4);
  } else {
    if (bf16) MA_SOFT(__bf16, 0); else MA_SOFT(float, 0);
  }
#undef MA_SOFT
}

void pack_block(bool bf16, const float* q, int64_t tok0, int nq, const void* rows, int bs, const int32_t* tab, int nkeep,
                int64_t k0, int nr, int nk, void* q2, void* k2, void* v2, int H, int G, int d, int dv, hipStream_t st) {
  if (nq <= 0 || nk <= 0) return;
  const dim3 gk((nk + 63) / 64, G, (d + 63) / 64 + (dv + 63) / 64);
  const bool v4 = d % 4 == 0 && dv % 4 == 0 && nk % 4 == 0 && (uintptr_t)rows % 16 == 0;
#define MA_PACK(E)                                                                                                  \
  pack_queries_k<E><<<nq, 256, 0, st>>>(q, tok0, nq, (E*)q2, H, G, d);                                              \
  if (v4) pack_keys_k<E, 4><<<gk, 256, 0, st>>>((const E*)rows, bs, tab, nkeep, k0, nr, nk, (E*)k2, (E*)v2, G, d, dv); \
  else pack_keys_k<E, 1><<<gk, 256, 0, st>>>((const E*)rows, bs, tab, nkeep, k0, nr, nk, (E*)k2, (E*)v2, G, d, dv)
  if (bf16) { MA_PACK(__bf16); } else { MA_PACK(float); }
#undef MA_PACK
}

void unpack_block(bool bf16, const float* o, void* out, int64_t tok0, int nq, int H, int G, int dv, hipStream_t st) {
  if (nq <= 0) return;
  if (bf16) unpack_k<__bf16><<<nq, 256, 0, st>>>(o, (__bf16*)out, tok0, nq, H, G, dv);
  else unpack_k<float><<<nq, 256, 0, st>>>(o, (float*)out, tok0, nq, H, G, dv);
}

void talk_mix(bool bf16, const float* w, const float* talk, int64_t pieces, int Lq, int L, int G, int rep, void* hl,
              float* out32, hipStream_t st) {
  if (pieces <= 0 || L <= 0) return;
  const dim3 grid((unsigned)(pieces * Lq), (L + 63) / 64);
  const size_t lds = (size_t)G * rep * 64 * sizeof(float);
  if (bf16) talk_mix_k<__bf16><<<grid, 64, lds, st>>>(w, talk, Lq, L, G, rep, (__bf16*)hl, nullptr);
  else talk_mix_k<float><<<grid, 64, lds, st>>>(w, talk, Lq, L, G, rep, (float*)nullptr, out32);
}

void sigmoid_gate(bool bf16, void* o, const void* g, int64_t g_ld, int64_t T, int C, int per, hipStream_t st) {
  const int64_t n = T * C;
  if (n <= 0) return;
  const size_t ab = 8 * (bf16 ? 2 : 4);
  const bool v8 = C % 8 == 0 && (uintptr_t)o % ab == 0 &&
                  (per > 1 ? per % 8 == 0 : (g_ld % 8 == 0 && (uintptr_t)g % ab == 0));
  const int64_t nv = v8 ? n / 8 : n;
  const int blocks = (int)((nv + 255) / 256 > 65535 ? 65535 : (nv + 255) / 256);
#define MA_GATE(E, V) sigmoid_gate_k<E, V><<<blocks, 256, 0, st>>>((E*)o, (const E*)g, g_ld, n, C, per)
  if (bf16) { if (v8) MA_GATE(__bf16, 8); else MA_GATE(__bf16, 1); }
  else { if (v8) MA_GATE(float, 8); else MA_GATE(float, 1); }
#undef MA_GATE
}

}  // namespace ma
}  // namespace illm
