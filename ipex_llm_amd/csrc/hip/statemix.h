// Launchers of the kernels of the decoders whose sublayers are normed before
// and after (statemix.hip) and of their recurrent mixers (statemix_scan.hip).
// ``bf16`` selects the activation element type (bf16 when true, f32 when
// false); everything the kernels accumulate is f32 either way.
#pragma once
#include <hip/hip_runtime.h>
#include <stdint.h>

namespace illm {
namespace sx {

// ---- element-wise and routing (statemix.hip)
// tanh(alpha x) w + b; alpha f32 [1], w / b f32 [W]; all null: no norm
struct Norm {
  const float* alpha;
  const float* w;
  const float* b;
};
void dyn_tanh(bool bf16, const float* x, Norm n, void* out, int T, int W, hipStream_t st);
// x += post(y), then out = pre(x) in the activation type (pre.alpha null: no second norm, out unused)
void add_normed(bool bf16, float* x, const void* y, bool y_f32, Norm post, Norm pre, void* out, int T, int W,
                hipStream_t st);
// y = (rms_norm(a) wa + rms_norm(b) wb) / 2; a, b, wa, wb in the activation type
void add_normed_pair(bool bf16, float* x, const void* a, const void* b, const void* wa, const void* wb, float eps,
                     Norm post, Norm pre, void* out, int T, int W, hipStream_t st);
// y = sum_k (idx < experts ? rows[t, k] : wts h[t]); rows f32 [T, top, W]
void add_normed_experts(bool bf16, float* x, const float* rows, const int32_t* idx, const float* wts, const void* h,
                        int top, int experts, Norm post, Norm pre, void* out, int T, int W, hipStream_t st);
// out = o / rms(o) w sigmoid(gate), o f32 [T, C]
void rms_sigmoid_gate(bool bf16, const float* o, const void* w, const void* gate, int64_t g_ld, void* out, int T, int C,
                      float eps, hipStream_t st);
// E <= 512 scores s (softmax over all, or sigmoid); choice by s + corr inside the best ``keep`` of ``groups`` groups; a
// group's score: its largest corrected score, or the sum of its two largest; weights s, or scale s / (their sum + 1e-20)
struct RouteRule {
  bool sigmoid, best_two, renorm;
  float scale;
};
void route_groups(const float* z, const float* corr, RouteRule rule, int T, int E, int top, int groups, int keep,
                  int32_t* idx, float* w, hipStream_t st);
// the same from the router's input rows h [T, W] (activation type) and weights rw f32 [E, W]
void router(bool bf16, const void* h, const float* rw, const float* corr, RouteRule rule, int T, int W, int E, int top,
            int groups, int keep, int32_t* idx, float* w, hipStream_t st);

// ---- recurrences (statemix_scan.hip)
constexpr int kScanMaxDim = 512;
// S' = decay S + silu(k) silu(v)^T, o = S'^T silu(q); q, k rows [T, H d], v [T, H dv] in the activation type
void decay_scan(bool bf16, const void* q, int64_t q_ld, const void* k, int64_t k_ld, const void* v, int64_t v_ld,
                const float* decay, float* S, const int32_t* cu, const int32_t* slots, const int64_t* pos, float* out,
                int B, int H, int d, int dv, hipStream_t st);
// gated delta rule; q, k f32 rows [T, K d], v f32 [T, H dv]; a, b [T, H] in the activation type
struct DeltaArgs {
  const void* a;
  int64_t a_ld;
  const void* b;
  int64_t b_ld;
  const float* rate;
  const float* dt_bias;
  float q_scale, unit_eps;
};
void delta_scan(bool bf16, const float* q, int64_t q_ld, const float* k, int64_t k_ld, const float* v, int64_t v_ld,
                DeltaArgs da, float* S, const int32_t* cu, const int32_t* slots, const int64_t* pos, float* out, int B, int H,
                int K, int d, int dv, hipStream_t st);
// the same two recurrences for long portions, in chunks of kChunk tokens on the matrix cores (statemix_chunk.hip): the
// tokens [seg0, seg0 + seg) of every portion, nch chunks in all (a portion's last one may be short); the state is read
// from and left in the slots.  Key sizes up to kChunkMaxDim
constexpr int kChunk = 64;
constexpr int kChunkMaxDim = 128;
int64_t chunk_scratch_floats(bool delta, int64_t nch, int H, int d, int dv);
void decay_chunks(bool bf16, const void* q, int64_t q_ld, const void* k, int64_t k_ld, const void* v, int64_t v_ld,
                  const float* decay, float* S, const int32_t* cu, const int32_t* slots, const int64_t* pos, float* out,
                  float* scratch, int B, int nch, int seg0, int seg, int H, int d, int dv, hipStream_t st);
void delta_chunks(bool bf16, const float* q, int64_t q_ld, const float* k, int64_t k_ld, const float* v, int64_t v_ld,
                  DeltaArgs da, float* S, const int32_t* cu, const int32_t* slots, const int64_t* pos, float* out,
                  float* scratch, int B, int nch, int seg0, int seg, int H, int K, int d, int dv, hipStream_t st);
// block-diagonal gates: w_r, w_i [nb, n, n] in the activation type; u, a, x f32 [T, nb n]
void rglru_gates(bool bf16, const float* u, const void* w_r, const float* b_r, const void* w_i, const float* b_i,
                 const float* log_base, float* a, float* x, int T, int nb, int n, hipStream_t st);
// S' = a S + x, out = S' gelu_tanh(y)
void rglru_scan(bool bf16, const float* a, const float* x, const void* y, int64_t y_ld, float* state, const int32_t* cu,
                const int32_t* slots, const int64_t* pos, void* out, int B, int C, int max_n, hipStream_t st);

}  // namespace sx
}  // namespace illm
