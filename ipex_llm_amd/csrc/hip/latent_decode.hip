// Decode-size steps of latent attention (gfx950, wave64), bf16:
//
//   latent_dec_k   one workgroup = (token, up to 16 heads, key split).  Tiles of
//                  64 keys (always inside one page) go through LDS as 16-byte
//                  pieces, the next tile's requested into registers before the
//                  current one is used.  Every wave scores 16 of the keys against
//                  all heads on the matrix cores (bf16 as stored, f32
//                  accumulation); the softmax runs online in f32 over the whole
//                  tile; the weighted sum takes the f32 weights as bf16 hi + lo
//                  halves, every wave owning a quarter of the latent columns of
//                  all heads, so nothing is merged between waves
//   combine_k      merge of the key splits with the sink and the head gate
//   head_linear_k  y[m, h] = x[m, h] W[h]^T for at most 16 rows: the absorbed up-
//                  projections, a wave per 16 outputs of a head
#include "seqmix.h"

#include <math.h>

namespace illm {
namespace sm {
namespace {

typedef __bf16 bf16x8 __attribute__((ext_vector_type(8)));
typedef float f32x4 __attribute__((ext_vector_type(4)));
typedef uint32_t u32x4 __attribute__((ext_vector_type(4)));

constexpr int KT = 64;                                              // keys per tile
constexpr int PF = 18;                                              // 16-byte pieces of a tile per thread (D <= 576)

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
// factor that turns a sum relative to the maximum M (with its weights' sum L) into the softmax's value, the sink included
__device__ __forceinline__ float with_sink(float M, float L, const float* sink, int h) {
  if (!sink) return 1.0f / L;
  const float s = sink[h], m = fmaxf(M, s), f = expf(M - m);
  return f / (L * f + expf(s - m));
}

__host__ __device__ inline int row_of(int D) { return ((D + 31) & ~31) + 8; }

// NT: 16-column tiles per wave (r <= 64 NT)
template <int NT>
__global__ void __launch_bounds__(256) latent_dec_k(const __bf16* __restrict__ q_lat, const __bf16* __restrict__ q_rot,
                                                   int64_t qr_st, int64_t qr_sh, const __bf16* __restrict__ rows, int bs,
                                                   const int32_t* __restrict__ bt, int bt_w,
                                                   const int32_t* __restrict__ seq_of, const int64_t* __restrict__ pos,
                                                   float scale, const __bf16* __restrict__ gate, int64_t g_st,
                                                   const float* __restrict__ sink, __bf16* __restrict__ out,
                                                   float* __restrict__ part, int H, int r, int dr, int window) {
  extern __shared__ __align__(16) unsigned char smem[];
  const int D = r + dr, DP = row_of(D), KS = (D + 31) >> 5, D8 = D >> 3;
  const int nsplit = gridDim.z, zs = blockIdx.z, t = blockIdx.x, h0 = blockIdx.y * 16;
  const int nh = min(16, H - h0);
  const int tid = threadIdx.x, lane = tid & 63, wv = tid >> 6, r16 = lane & 15, g = lane >> 4;
  __bf16* qs = (__bf16*)smem;                                       // [16][DP]
  __bf16* kt = qs + 16 * DP;                                        // [KT][DP]
  float* pb = (float*)(kt + KT * DP);                               // [16][KT + 4] weights
  float* al = pb + 16 * (KT + 4);                                   // [16] rescale factors
  float* mred = al + 16;                                            // [4][16]
  float* lred = mred + 64;                                          // [4][16]
  const int64_t p = pos[t];
  const int32_t* tab = bt + (int64_t)seq_of[t] * bt_w;
  const int ntiles = (int)(p / KT) + 1;
  const int64_t lo = window > 0 ? (p - window + 1 > 0 ? p - window + 1 : 0) : 0;
  u32x4 pf[PF];
  const int krow = tid >> 2, kpc = tid & 3;                         // four threads per key: pieces kpc, kpc + 4, ...
  auto request = [&](int ti) {
    const int64_t k0 = (int64_t)ti * KT;
    const int row = min(krow, (int)min((int64_t)KT, p - k0 + 1) - 1);          // (past the last key: that one again)
    const u32x4* src = (const u32x4*)(rows + ((int64_t)tab[k0 / bs] * bs + (k0 % bs) + row) * D);
#pragma unroll
    for (int u = 0; u < PF; u++) pf[u] = src[min(kpc + 4 * u, D8 - 1)];
  };
  int ti = (int)(lo / KT) + zs;
  if (ti < ntiles) request(ti);
  // queries and the tile buffer: zeros first (pad columns, absent heads, keys a tile does not fill)
  for (int i = tid; i < (16 + KT) * DP / 8; i += 256) ((uint4*)smem)[i] = make_uint4(0u, 0u, 0u, 0u);
  __syncthreads();
  for (int i = tid; i < nh * D8; i += 256) {
    const int h = i / D8, c = 8 * (i - h * D8);
    const __bf16* s = c < r ? q_lat + ((int64_t)t * H + h0 + h) * r + c
                            : q_rot + (int64_t)t * qr_st + (int64_t)(h0 + h) * qr_sh + (c - r);
    *(uint4*)(qs + h * DP + c) = *(const uint4*)s;
  }
  float m_r = -INFINITY, l_r = 0.f;                                 // of head r16, the same in every thread that holds it
  f32x4 o[NT];                                                      // heads 4 g + i, column 16 (wv + 4 n) + r16
#pragma unroll
  for (int n = 0; n < NT; n++) o[n] = f32x4{0.f, 0.f, 0.f, 0.f};
  for (; ti < ntiles; ti += nsplit) {
    const int64_t k0 = (int64_t)ti * KT;
    const int nvalid = (int)min((int64_t)KT, p - k0 + 1);
    if (krow < nvalid) {
#pragma unroll
      for (int u = 0; u < PF; u++)
        if (kpc + 4 * u < D8) *(u32x4*)(kt + krow * DP + 8 * (kpc + 4 * u)) = pf[u];
    }
    __syncthreads();
    if (ti + nsplit < ntiles) request(ti + nsplit);
    f32x4 acc = {0.f, 0.f, 0.f, 0.f};
    const __bf16* ka = kt + (16 * wv + r16) * DP + 8 * g;
    const __bf16* qb = qs + r16 * DP + 8 * g;
    for (int ks = 0; ks < KS; ks++)
      acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(*(const bf16x8*)(ka + 32 * ks), *(const bf16x8*)(qb + 32 * ks), acc, 0, 0, 0);
    // lane: keys 16 wv + 4 g + i of head r16
    float sv[4], ml = -INFINITY;
#pragma unroll
    for (int i = 0; i < 4; i++) {
      const int j = 16 * wv + 4 * g + i;
      sv[i] = j < nvalid && k0 + j >= lo ? acc[i] * scale : -INFINITY;
      ml = fmaxf(ml, sv[i]);
    }
    ml = fmaxf(ml, __shfl_xor(ml, 16, 64));
    ml = fmaxf(ml, __shfl_xor(ml, 32, 64));
    if (g == 0) mred[16 * wv + r16] = ml;
    __syncthreads();
    const float mn = fmaxf(m_r, fmaxf(fmaxf(mred[r16], mred[16 + r16]), fmaxf(mred[32 + r16], mred[48 + r16])));
    const float alpha = m_r == -INFINITY ? 0.f : expf(m_r - mn);
    float pv[4], ls = 0.f;
#pragma unroll
    for (int i = 0; i < 4; i++) {
      pv[i] = sv[i] == -INFINITY ? 0.f : expf(sv[i] - mn);
      ls += pv[i];
    }
    ls += __shfl_xor(ls, 16, 64);
    ls += __shfl_xor(ls, 32, 64);
    m_r = mn;
    *(float4*)(pb + r16 * (KT + 4) + 16 * wv + 4 * g) = make_float4(pv[0], pv[1], pv[2], pv[3]);
    if (g == 0) lred[16 * wv + r16] = ls;
    if (wv == 0 && g == 0) al[r16] = alpha;
    __syncthreads();
    l_r = l_r * alpha + (lred[r16] + lred[16 + r16]) + (lred[32 + r16] + lred[48 + r16]);
    const f32x4 av = *(const f32x4*)(al + 4 * g);
#pragma unroll
    for (int n = 0; n < NT; n++) o[n] *= av;
#pragma unroll
    for (int ks = 0; ks < KT / 32; ks++) {                          // (weights past nvalid are 0, rows finite)
      if (32 * ks >= nvalid) break;
      bf16x8 hi, lo;                                                // head r16, keys 32 ks + 8 g + e
      const float* pw = pb + r16 * (KT + 4) + 32 * ks + 8 * g;
#pragma unroll
      for (int e = 0; e < 8; e += 4) {
        const f32x4 w = *(const f32x4*)(pw + e);
#pragma unroll
        for (int i = 0; i < 4; i++) {
          hi[e + i] = (__bf16)w[i];
          lo[e + i] = (__bf16)(w[i] - (float)hi[e + i]);
        }
      }
#pragma unroll
      for (int n = 0; n < NT; n++) {
        const int c = 16 * (wv + 4 * n);
        if (c >= r) break;
        const __bf16* kr = kt + (32 * ks + 8 * g) * DP + c + r16;    // (columns past r: the rotated part, not kept)
        bf16x8 b;
#pragma unroll
        for (int e = 0; e < 8; e++) b[e] = kr[e * DP];
        o[n] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(lo, b, o[n], 0, 0, 0);
        o[n] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(hi, b, o[n], 0, 0, 0);
      }
    }
    __syncthreads();                                                // the tile and the weights are used again
  }
  if (wv == 0 && g == 0) {                                          // (m, l) of every head for the threads of the columns
    mred[r16] = m_r;
    lred[r16] = l_r;
  }
  __syncthreads();
  for (int h = 0; h < nh; h++) {
    const int64_t th = (int64_t)t * H + h0 + h;
    if (nsplit > 1) {
      float* pp = part + (th * nsplit + zs) * (r + 2);
      if (tid == 0) {
        pp[r] = mred[h];
        pp[r + 1] = lred[h];
      }
    }
  }
#pragma unroll
  for (int i = 0; i < 4; i++) {
    const int h = 4 * g + i;
    if (h >= nh) break;
    const int64_t th = (int64_t)t * H + h0 + h;
    float f = 1.f;
    if (nsplit == 1) {
      f = with_sink(mred[h], lred[h], sink, h0 + h);
      if (gate) f *= 1.0f / (1.0f + expf(-(float)gate[(int64_t)t * g_st + h0 + h]));
    }
#pragma unroll
    for (int n = 0; n < NT; n++) {
      const int c = 16 * (wv + 4 * n) + r16;
      if (c >= r) continue;
      if (nsplit > 1) part[(th * nsplit + zs) * (r + 2) + c] = o[n][i];
      else out[th * r + c] = (__bf16)(o[n][i] * f);
    }
  }
}

// merge of the key splits (nsplit <= 64): part [T, H, nsplit, r + 2] -> out [T, H, r]
__global__ void __launch_bounds__(256) combine_k(const float* __restrict__ part, const __bf16* __restrict__ gate,
                                                int64_t g_st, const float* __restrict__ sink, __bf16* __restrict__ out,
                                                int H, int r, int nsplit) {
  __shared__ float wz[64];
  const int64_t t = blockIdx.x;
  const int h = blockIdx.y;
  const float* pp = part + ((t * H + h) * nsplit) * (int64_t)(r + 2);
  const int c = blockIdx.z * 256 + threadIdx.x;
  if (threadIdx.x < 64) {
    const int z = threadIdx.x;
    const float mz = z < nsplit ? pp[(int64_t)z * (r + 2) + r] : -INFINITY;
    const float M = wave_max(mz);
    const float e = mz == -INFINITY ? 0.f : expf(mz - M);
    const float L = wave_sum(z < nsplit ? pp[(int64_t)z * (r + 2) + r + 1] * e : 0.f);
    const float g = gate ? 1.0f / (1.0f + expf(-(float)gate[t * g_st + h])) : 1.0f;
    wz[z] = e * with_sink(M, L, sink, h) * g;
  }
  __syncthreads();
  if (c >= r) return;
  float O = 0.f;
  int z = 0;
  for (; z + 8 <= nsplit; z += 8) {
    float v[8];
#pragma unroll
    for (int i = 0; i < 8; i++) v[i] = pp[(int64_t)(z + i) * (r + 2) + c];
#pragma unroll
    for (int i = 0; i < 8; i++) O = fmaf(v[i], wz[z + i], O);
  }
  for (; z < nsplit; z++) O = fmaf(pp[(int64_t)z * (r + 2) + c], wz[z], O);
  out[(t * H + h) * r + c] = (__bf16)O;
}

__global__ void __launch_bounds__(256) head_linear_k(const __bf16* __restrict__ x, int64_t st_m, int64_t st_h, int M, int K,
                                                    const __bf16* __restrict__ w, int N, __bf16* __restrict__ out, int H) {
  const int h = blockIdx.y, lane = threadIdx.x & 63, r16 = lane & 15, g = lane >> 4;
  const int n0 = 16 * (4 * blockIdx.x + (threadIdx.x >> 6));
  if (n0 >= N) return;
  const bool on = r16 < M;
  const __bf16* xr = x + (on ? r16 : 0) * st_m + h * st_h + 8 * g;
  const __bf16* wr = w + ((int64_t)h * N + min(n0 + r16, N - 1)) * K + 8 * g;
  bf16x8 zero;
#pragma unroll
  for (int i = 0; i < 8; i++) zero[i] = (__bf16)0.f;
  f32x4 acc = {0.f, 0.f, 0.f, 0.f};
  int k = 0;
  for (; k + 128 <= K; k += 128) {
    bf16x8 a[4], b[4];
#pragma unroll
    for (int i = 0; i < 4; i++) {
      a[i] = *(const bf16x8*)(wr + k + 32 * i);
      b[i] = on ? *(const bf16x8*)(xr + k + 32 * i) : zero;
    }
#pragma unroll
    for (int i = 0; i < 4; i++) acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a[i], b[i], acc, 0, 0, 0);
  }
  for (; k < K; k += 32)
    acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(*(const bf16x8*)(wr + k), on ? *(const bf16x8*)(xr + k) : zero, acc, 0, 0, 0);
  if (!on) return;
  __bf16* y = out + ((int64_t)r16 * H + h) * N + n0 + 4 * g;        // lane: outputs n0 + 4 g + i of row r16
#pragma unroll
  for (int i = 0; i < 4; i++)
    if (n0 + 4 * g + i < N) y[i] = (__bf16)acc[i];
}

int lds_bytes(int D) { return (16 + KT) * row_of(D) * 2 + (16 * (KT + 4) + 16 + 128) * 4; }

}  // namespace

bool latent_decode_fits(int r, int dr) {
  const int D = r + dr;
  return r >= 1 && r <= 512 && r % 8 == 0 && dr % 8 == 0 && D <= 8 * 4 * PF && lds_bytes(D) <= 160 * 1024;
}

int latent_decode_splits(int T, int H, int max_keys) {
  const int64_t blocks = (int64_t)T * ((H + 15) / 16);
  const int tiles = (max_keys + KT - 1) / KT + 1;
  // one workgroup per CU at a time: as many splits as give every CU one, equal numbers of tiles in each
  int ns = (int)(256 / blocks);
  ns = ns < 1 ? 1 : (ns > 64 ? 64 : ns);
  const int per = (tiles + ns - 1) / ns;
  return (tiles + per - 1) / per;
}

void latent_decode(const void* q_lat, const void* q_rot, int64_t qr_st, int64_t qr_sh, const void* rows, int bs,
                   const int32_t* block_tables, int bt_width, const int32_t* seq_of, const int64_t* pos, float scale,
                   const void* gate, int64_t g_st, const float* sink, void* out, float* part, int nsplit, int T, int H, int r,
                   int dr, int window, hipStream_t st) {
  if (T <= 0 || !latent_decode_fits(r, dr)) return;                 // (refused by the caller beforehand)
  const int lds = lds_bytes(r + dr);
  const dim3 grid(T, (H + 15) / 16, nsplit);
#define SM_DEC(NT)                                                                                                    \
  {                                                                                                                   \
    (void)hipFuncSetAttribute((const void*)latent_dec_k<NT>, hipFuncAttributeMaxDynamicSharedMemorySize, lds);        \
    latent_dec_k<NT><<<grid, 256, lds, st>>>((const __bf16*)q_lat, (const __bf16*)q_rot, qr_st, qr_sh,                \
                                             (const __bf16*)rows, bs, block_tables, bt_width, seq_of, pos, scale,     \
                                             (const __bf16*)gate, g_st, sink, (__bf16*)out, part, H, r, dr, window);  \
  }
  if (r > 256) SM_DEC(8)
  else if (r > 128) SM_DEC(4)
  else SM_DEC(2)
#undef SM_DEC
  if (nsplit > 1)
    combine_k<<<dim3(T, H, (r + 255) / 256), 256, 0, st>>>(part, (const __bf16*)gate, g_st, sink, (__bf16*)out, H, r, nsplit);
}

void head_linear(const void* x, int64_t st_m, int64_t st_h, int M, int H, int K, const void* w, int N, void* out,
                 hipStream_t st) {
  if (M <= 0 || N <= 0 || H <= 0) return;
  head_linear_k<<<dim3((N + 63) / 64, H), 256, 0, st>>>((const __bf16*)x, st_m, st_h, M, K, (const __bf16*)w, N,
                                                        (__bf16*)out, H);
}

}  // namespace sm
}  // namespace illm
