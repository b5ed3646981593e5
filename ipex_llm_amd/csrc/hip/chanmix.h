// Launchers of the kernels of the mixers whose decay has one number per key
// channel (chanmix.hip, chanmix_scan.hip, chanmix_chunk.hip) and of the pre-norm
// blocks with scaled sublayers around them.  ``bf16`` selects the activation
// element type (bf16 when true, f32 when false); everything the kernels
// accumulate is f32 either way.
#pragma once
#include <hip/hip_runtime.h>
#include <stdint.h>

namespace illm {
namespace cx {

// ---- element-wise steps and small products (chanmix.hip)
// a sublayer's result still to be added to the residual stream: sa a + sb b (b null: one term; a, b in the activation
// type or, a_f32, a in f32), or sa times the sum of a token's ``top`` f32 rows (top > 0: a is [T, top, W]); a null: nothing
struct Source {
  const void* a;
  const float* sa;
  const void* b;
  const float* sb;
  int top;
  bool a_f32;
};
// x += source, out = x / sqrt(mean(x^2) + eps) w; w f32 [W]
void add_scaled_norm(bool bf16, float* x, Source y, const float* w, float eps, void* out, int T, int W, hipStream_t st);
// out [T, 2 W] = [x + source | embed[id]] (x itself is left as it is); an id outside the table reads as zeros
void loop_input(bool bf16, const float* x, Source y, const void* embed, int64_t vocab, const int64_t* ids, void* out, int T,
                int W, hipStream_t st);
// out[m] = h + (previous token's h - h) mu[m], m = 0 .. NM - 1 (out [NM, T, W], mu f32 [NM, W]); the token before a
// portion's first one comes from state f32 [slots, W] (zeros at position 0), every portion leaves its last h there
void token_mixes(bool bf16, const void* h, const float* mu, int NM, float* state, const int32_t* cu, const int32_t* seq_of,
                 const int32_t* slots, const int64_t* pos, void* out, int T, int B, int W, bool single, hipStream_t st);
// z = in W^T + bias over rows in [T, R] (row stride ld; squash: tanh(in)), W [N, R] in the activation type;
// kind 0: exp(-rate[n] softplus(z)), kind 1: exp(-exp(z)); out f32 [T, N]
void lowrank_decay(bool bf16, const void* in, int64_t ld, const void* w, const float* rate, const float* bias, int kind,
                   bool squash, float* out, int T, int N, int R, hipStream_t st);
// decode-size projections whose row groups read different inputs, one launch: out[m, n] = w[n] . x[group of n][m] (+ bias),
// M <= 16 rows, K a multiple of 64, 16-bit; group g holds the weight rows row0[g] .. row0[g + 1] - 1
constexpr int kMaxGroups = 8;
struct Groups {
  const void* x[kMaxGroups];
  int row0[kMaxGroups + 1];
  int tile0[kMaxGroups + 1];                                        // 16-row tiles in front of the group
  int n;
};
void grouped_linear(Groups g, int M, int K, const void* w, const void* bias, void* out, bool out_f32, hipStream_t st);

// ---- recurrences with one decay per key channel; g f32 [T, H d] (heads contiguous in a row)
// channel-decay delta rule: q, k f32 rows [T, K d] (made unit vectors, q times q_scale), v f32 [T, H dv], b [T, H] in the
// activation type: S <- diag(g) S, u = sigmoid(b) (v - S^T k), S <- S + k u^T, o = S^T q
struct DeltaIn {
  const void* b;
  int64_t b_ld;
  float q_scale, unit_eps;
};
void delta_scan(bool bf16, const float* q, int64_t q_ld, const float* k, int64_t k_ld, const float* v, int64_t v_ld,
                const float* g, DeltaIn di, float* S, const int32_t* cu, const int32_t* slots, const int64_t* pos,
                float* out, int B, int H, int K, int d, int dv, hipStream_t st);
void delta_chunks(bool bf16, const float* q, int64_t q_ld, const float* k, int64_t k_ld, const float* v, int64_t v_ld,
                  const float* g, DeltaIn di, float* S, const int32_t* cu, const int32_t* slots, const int64_t* pos,
                  float* out, float* scratch, int B, int nch, int seg0, int seg, int H, int K, int d, int dv,
                  hipStream_t st);
// read-out before the write, with a bonus for the current token: r, k [T, H d], v [T, H dv] in the activation type, u f32
// [H, d]: o = S^T r + (sum_c u_c k_c r_c) v, S <- diag(g) S + k v^T
void bonus_scan(bool bf16, const void* r, int64_t r_ld, const void* k, int64_t k_ld, const void* v, int64_t v_ld,
                const float* g, const float* u, float* S, const int32_t* cu, const int32_t* slots, const int64_t* pos,
                float* out, int B, int H, int d, int dv, hipStream_t st);
void bonus_chunks(bool bf16, const void* r, int64_t r_ld, const void* k, int64_t k_ld, const void* v, int64_t v_ld,
                  const float* g, const float* u, float* S, const int32_t* cu, const int32_t* slots, const int64_t* pos,
                  float* out, float* scratch, int B, int nch, int seg0, int seg, int H, int d, int dv, hipStream_t st);
int64_t chunk_scratch_floats(bool delta, int64_t nch, int H, int d, int dv);

}  // namespace cx
}  // namespace illm
