// torch.ops.ipex_llm_amd.sx_*: the kernels of the decoders whose sublayers are
// normed before and after and of their recurrent mixers (csrc/hip/statemix.hip,
// statemix_scan.hip).  Every entry checks on the host that the operand shapes,
// dtypes and strides are what its kernel and grid assume.
#include <ATen/ATen.h>
#include <ATen/hip/HIPContext.h>
#include <c10/core/DeviceGuard.h>
#include <torch/library.h>

#include <algorithm>
#include <tuple>

#include "../hip/statemix.h"

using at::Tensor;
using OptT = c10::optional<Tensor>;
using illm::sx::Norm;

namespace {

hipStream_t stream() { return at::hip::getCurrentHIPStream().stream(); }
bool is_act(const Tensor& t) { return t.scalar_type() == at::kBFloat16 || t.scalar_type() == at::kFloat; }
bool bf(const Tensor& t) { return t.scalar_type() == at::kBFloat16; }
bool has(const OptT& t) { return t.has_value() && t->defined(); }
at::ScalarType act_type(bool act_f32) { return act_f32 ? at::kFloat : at::kBFloat16; }

bool vec(const Tensor& t, at::ScalarType ty, int64_t n) {
  return t.is_cuda() && t.scalar_type() == ty && t.is_contiguous() && t.numel() == n;
}
bool rows(const Tensor& t, at::ScalarType ty, int64_t T, int64_t W) {
  return t.is_cuda() && t.dim() == 2 && t.scalar_type() == ty && t.is_contiguous() && t.size(0) == T && t.size(1) == W;
}
// [T, n] view of a projection's rows (unit inner stride)
bool strided(const Tensor& t, at::ScalarType ty, int64_t T, int64_t n) {
  return t.is_cuda() && t.dim() == 2 && t.scalar_type() == ty && t.size(0) == T && t.size(1) == n &&
         (n == 1 || t.stride(1) == 1);
}
// [T, heads, n] view of a projection's rows: heads contiguous inside a row
bool head_rows(const Tensor& t, at::ScalarType ty) {
  return t.is_cuda() && t.dim() == 3 && t.scalar_type() == ty && t.stride(2) == 1 && t.stride(1) == t.size(2) &&
         t.stride(0) >= t.size(1) * t.size(2);
}
void check_step(const Tensor& cu, const Tensor& slots, const Tensor& pos, int64_t T, const char* what) {
  TORCH_CHECK(cu.is_cuda() && cu.scalar_type() == at::kInt && cu.is_contiguous() && cu.numel() >= 2 &&
                  slots.is_cuda() && slots.scalar_type() == at::kInt && slots.is_contiguous() &&
                  slots.numel() >= cu.numel() - 1 && pos.is_cuda() && pos.scalar_type() == at::kLong &&
                  pos.is_contiguous() && pos.numel() >= T && cu.numel() - 1 <= 65535,
              what, ": cu int32 [B + 1], slots int32 [B], pos int64 [T]");
}
Norm norm_of(const Tensor& alpha, const Tensor& w, const Tensor& b, int64_t W, const char* what) {
  TORCH_CHECK(vec(alpha, at::kFloat, 1) && vec(w, at::kFloat, W) && vec(b, at::kFloat, W), what,
              ": norm (alpha [1], w [W], b [W]) in f32");
  return {alpha.data_ptr<float>(), w.data_ptr<float>(), b.data_ptr<float>()};
}
Norm norm_of(const OptT& alpha, const OptT& w, const OptT& b, int64_t W, const char* what) {
  if (!has(alpha)) return {nullptr, nullptr, nullptr};
  TORCH_CHECK(has(w) && has(b), what, ": a norm has alpha, w and b");
  return norm_of(*alpha, *w, *b, W, what);
}
void check_x(const Tensor& x, const char* what) {
  TORCH_CHECK(x.is_cuda() && x.dim() == 2 && x.scalar_type() == at::kFloat && x.is_contiguous() && x.size(1) >= 1 &&
                  x.size(1) <= 1 << 24,
              what, ": x f32 [T, W] contiguous");
}
Tensor result(const Tensor& x, const Norm& pre, bool act_f32) {
  return pre.alpha ? at::empty(x.sizes(), x.options().dtype(act_type(act_f32)))
                   : at::empty({0}, x.options().dtype(act_type(act_f32)));
}

Tensor sx_dyn_tanh(const Tensor& x, const Tensor& alpha, const Tensor& w, const Tensor& b, bool act_f32) {
  c10::DeviceGuard g(x.device());
  check_x(x, "sx_dyn_tanh");
  const Norm n = norm_of(alpha, w, b, x.size(1), "sx_dyn_tanh");
  Tensor out = result(x, n, act_f32);
  illm::sx::dyn_tanh(!act_f32, x.data_ptr<float>(), n, out.data_ptr(), (int)x.size(0), (int)x.size(1), stream());
  return out;
}

Tensor sx_add_normed(Tensor& x, const Tensor& y, const Tensor& pa, const Tensor& pw, const Tensor& pb, const OptT& qa,
                     const OptT& qw, const OptT& qb, bool act_f32) {
  c10::DeviceGuard g(x.device());
  check_x(x, "sx_add_normed");
  const int64_t T = x.size(0), W = x.size(1);
  const auto ty = y.scalar_type();
  TORCH_CHECK((ty == at::kFloat || ty == act_type(act_f32)) && rows(y, ty, T, W),
              "sx_add_normed: y [T, W] contiguous, f32 or the activation dtype");
  const Norm post = norm_of(pa, pw, pb, W, "sx_add_normed"), pre = norm_of(qa, qw, qb, W, "sx_add_normed");
  Tensor out = result(x, pre, act_f32);
  illm::sx::add_normed(!act_f32, x.data_ptr<float>(), y.data_ptr(), ty == at::kFloat, post, pre, out.data_ptr(), (int)T,
                       (int)W, stream());
  return out;
}

Tensor sx_add_normed_pair(Tensor& x, const Tensor& a, const Tensor& b, const Tensor& wa, const Tensor& wb, double eps,
                          const Tensor& pa, const Tensor& pw, const Tensor& pb, const OptT& qa, const OptT& qw,
                          const OptT& qb, bool act_f32) {
  c10::DeviceGuard g(x.device());
  check_x(x, "sx_add_normed_pair");
  const int64_t T = x.size(0), W = x.size(1);
  const auto ty = act_type(act_f32);
  TORCH_CHECK(rows(a, ty, T, W) && rows(b, ty, T, W) && vec(wa, ty, W) && vec(wb, ty, W),
              "sx_add_normed_pair: a, b [T, W] contiguous and weights [W] in the activation dtype");
  const Norm post = norm_of(pa, pw, pb, W, "sx_add_normed_pair"), pre = norm_of(qa, qw, qb, W, "sx_add_normed_pair");
  Tensor out = result(x, pre, act_f32);
  illm::sx::add_normed_pair(!act_f32, x.data_ptr<float>(), a.data_ptr(), b.data_ptr(), wa.data_ptr(), wb.data_ptr(),
                            (float)eps, post, pre, out.data_ptr(), (int)T, (int)W, stream());
  return out;
}

Tensor sx_add_normed_experts(Tensor& x, const Tensor& er, const Tensor& idx, const Tensor& wts, const Tensor& h,
                             int64_t experts, const Tensor& pa, const Tensor& pw, const Tensor& pb, const OptT& qa,
                             const OptT& qw, const OptT& qb, bool act_f32) {
  c10::DeviceGuard g(x.device());
  check_x(x, "sx_add_normed_experts");
  const int64_t T = x.size(0), W = x.size(1);
  TORCH_CHECK(idx.is_cuda() && idx.dim() == 2 && idx.scalar_type() == at::kInt && idx.is_contiguous() && idx.size(0) == T &&
                  idx.size(1) >= 1 && vec(wts, at::kFloat, idx.numel()) && experts >= 0,
              "sx_add_normed_experts: idx int32 [T, top], weights f32 [T, top]");
  TORCH_CHECK(vec(er, at::kFloat, T * idx.size(1) * W), "sx_add_normed_experts: rows f32 [T, top, W]");
  TORCH_CHECK(rows(h, act_type(act_f32), T, W), "sx_add_normed_experts: h [T, W] in the activation dtype");
  const Norm post = norm_of(pa, pw, pb, W, "sx_add_normed_experts"),
             pre = norm_of(qa, qw, qb, W, "sx_add_normed_experts");
  Tensor out = result(x, pre, act_f32);
  illm::sx::add_normed_experts(!act_f32, x.data_ptr<float>(), er.data_ptr<float>(), idx.data_ptr<int32_t>(),
                               wts.data_ptr<float>(), h.data_ptr(), (int)idx.size(1), (int)experts, post, pre,
                               out.data_ptr(), (int)T, (int)W, stream());
  return out;
}

Tensor sx_rms_sigmoid_gate(const Tensor& o, const Tensor& w, const Tensor& gate, double eps, bool act_f32) {
  c10::DeviceGuard g(o.device());
  check_x(o, "sx_rms_sigmoid_gate");
  const int64_t T = o.size(0), C = o.size(1);
  const auto ty = act_type(act_f32);
  TORCH_CHECK(vec(w, ty, C) && strided(gate, ty, T, C),
              "sx_rms_sigmoid_gate: weight [C] and gate [T, C] in the activation dtype");
  Tensor out = at::empty({T, C}, o.options().dtype(ty));
  illm::sx::rms_sigmoid_gate(!act_f32, o.data_ptr<float>(), w.data_ptr(), gate.data_ptr(), gate.stride(0), out.data_ptr(),
                             (int)T, (int)C, (float)eps, stream());
  return out;
}

std::tuple<Tensor, Tensor> sx_route_groups(const Tensor& z, const OptT& corr, int64_t top, int64_t groups, int64_t keep,
                                           bool sigmoid, bool best_two, bool renorm, double scale) {
  c10::DeviceGuard g(z.device());
  TORCH_CHECK(z.is_cuda() && z.dim() == 2 && z.scalar_type() == at::kFloat && z.is_contiguous(),
              "sx_route_groups: logits f32 [T, E] contiguous");
  const int64_t T = z.size(0), E = z.size(1);
  TORCH_CHECK(E >= 1 && E <= 512 && groups >= 1 && E % groups == 0 && keep >= 1 && keep <= groups && top >= 1 &&
                  top <= keep * (E / groups),
              "sx_route_groups: E <= 512, equal groups, 1 <= top <= outputs of the kept groups");
  TORCH_CHECK(!has(corr) || vec(*corr, at::kFloat, E), "sx_route_groups: correction f32 [E]");
  Tensor idx = at::empty({T, top}, z.options().dtype(at::kInt)), w = at::empty({T, top}, z.options());
  illm::sx::route_groups(z.data_ptr<float>(), has(corr) ? corr->data_ptr<float>() : nullptr,
                         {sigmoid, best_two, renorm, (float)scale}, (int)T, (int)E, (int)top, (int)groups,
                         (int)keep, idx.data_ptr<int32_t>(), w.data_ptr<float>(), stream());
  return {idx, w};
}

std::tuple<Tensor, Tensor> sx_router(const Tensor& h, const Tensor& rw, const OptT& corr, int64_t top, int64_t groups,
                                     int64_t keep, bool sigmoid, bool best_two, bool renorm, double scale) {
  c10::DeviceGuard g(h.device());
  TORCH_CHECK(h.is_cuda() && h.dim() == 2 && is_act(h) && h.is_contiguous(), "sx_router: h [T, W] contiguous");
  const int64_t T = h.size(0), W = h.size(1), E = rw.dim() == 2 ? rw.size(0) : 0;
  TORCH_CHECK(rows(rw, at::kFloat, E, W), "sx_router: router f32 [E, W]");
  TORCH_CHECK(E >= 1 && E <= 512 && groups >= 1 && E % groups == 0 && keep >= 1 && keep <= groups && top >= 1 &&
                  top <= keep * (E / groups),
              "sx_router: E <= 512, equal groups, 1 <= top <= outputs of the kept groups");
  TORCH_CHECK(!has(corr) || vec(*corr, at::kFloat, E), "sx_router: correction f32 [E]");
  auto f = h.options().dtype(at::kFloat);
  Tensor idx = at::empty({T, top}, f.dtype(at::kInt)), w = at::empty({T, top}, f);
  illm::sx::router(bf(h), h.data_ptr(), rw.data_ptr<float>(), has(corr) ? corr->data_ptr<float>() : nullptr,
                   {sigmoid, best_two, renorm, (float)scale}, (int)T, (int)W, (int)E,
                   (int)top, (int)groups, (int)keep, idx.data_ptr<int32_t>(), w.data_ptr<float>(), stream());
  return {idx, w};
}

void check_state(const Tensor& S, int64_t H, int64_t d, int64_t dv, const char* what) {
  TORCH_CHECK(S.is_cuda() && S.scalar_type() == at::kFloat && S.is_contiguous() && S.dim() == 4 && S.size(1) == H &&
                  S.size(2) == d && S.size(3) == dv,
              what, ": state f32 [slots, H, d, dv]");
  TORCH_CHECK(d >= 1 && d <= illm::sx::kScanMaxDim && dv >= 1 && H <= 65535 && (dv + 63) / 64 <= 65535, what,
              ": key size 1..", illm::sx::kScanMaxDim);
}

// portions of at least ``chunk_min`` tokens (0: never) run in chunks; long ones segment by segment, so that the scratch
// memory stays bounded.  f(chunks, first token, tokens) launches one segment
constexpr int64_t kSegment = 8192;
bool by_chunks(c10::IntArrayRef lens, int64_t chunk_min, int64_t d) {
  int64_t n = 0;
  for (auto v : lens) n = std::max(n, v);
  return chunk_min > 0 && n >= chunk_min && d <= illm::sx::kChunkMaxDim;
}
template <typename F> void segments(c10::IntArrayRef lens, F f) {
  int64_t longest = 0;
  for (auto v : lens) longest = std::max(longest, v);
  for (int64_t s0 = 0; s0 < longest; s0 += kSegment) {
    int64_t nch = 0;
    for (auto v : lens) {
      const int64_t n = std::min(kSegment, v - s0);
      if (n > 0) nch += (n + illm::sx::kChunk - 1) / illm::sx::kChunk;
    }
    f((int)nch, (int)s0, (int)kSegment);
  }
}
void check_lens(c10::IntArrayRef lens, const Tensor& cu, int64_t T, const char* what) {
  int64_t sum = 0;
  for (auto v : lens) {
    TORCH_CHECK(v >= 0, what, ": negative portion");
    sum += v;
  }
  TORCH_CHECK((int64_t)lens.size() == cu.numel() - 1 && sum == T, what, ": one length per sequence, T in all");
}

Tensor sx_decay_scan(const Tensor& q, const Tensor& k, const Tensor& v, const Tensor& decay, Tensor& S, const Tensor& cu,
                     const Tensor& slots, const Tensor& pos, c10::IntArrayRef lens, int64_t chunk_min) {
  c10::DeviceGuard g(q.device());
  const auto ty = q.scalar_type();
  TORCH_CHECK(is_act(q) && head_rows(q, ty) && head_rows(k, ty) && k.sizes() == q.sizes(),
              "sx_decay_scan: q, k [T, H, d] (heads contiguous in a row)");
  const int64_t T = q.size(0), H = q.size(1), d = q.size(2);
  TORCH_CHECK(head_rows(v, ty) && v.size(0) == T && v.size(1) == H, "sx_decay_scan: v [T, H, dv]");
  const int64_t dv = v.size(2);
  TORCH_CHECK(vec(decay, at::kFloat, H), "sx_decay_scan: decay f32 [H]");
  check_state(S, H, d, dv, "sx_decay_scan");
  check_step(cu, slots, pos, T, "sx_decay_scan");
  Tensor out = at::empty({T, H, dv}, q.options().dtype(at::kFloat));
  if (T == 0) return out;
  check_lens(lens, cu, T, "sx_decay_scan");
  if (by_chunks(lens, chunk_min, d)) {
    segments(lens, [&](int nch, int s0, int seg) {
      Tensor scratch = at::empty({illm::sx::chunk_scratch_floats(false, nch, (int)H, (int)d, (int)dv)}, out.options());
      illm::sx::decay_chunks(bf(q), q.data_ptr(), q.stride(0), k.data_ptr(), k.stride(0), v.data_ptr(), v.stride(0),
                             decay.data_ptr<float>(), S.data_ptr<float>(), cu.data_ptr<int32_t>(), slots.data_ptr<int32_t>(),
                             pos.data_ptr<int64_t>(), out.data_ptr<float>(), scratch.data_ptr<float>(), (int)cu.numel() - 1,
                             nch, s0, seg, (int)H, (int)d, (int)dv, stream());
    });
    return out;
  }
  illm::sx::decay_scan(bf(q), q.data_ptr(), q.stride(0), k.data_ptr(), k.stride(0), v.data_ptr(), v.stride(0),
                       decay.data_ptr<float>(), S.data_ptr<float>(), cu.data_ptr<int32_t>(), slots.data_ptr<int32_t>(),
                       pos.data_ptr<int64_t>(), out.data_ptr<float>(), (int)cu.numel() - 1, (int)H, (int)d, (int)dv,
                       stream());
  return out;
}

Tensor sx_delta_scan(const Tensor& q, const Tensor& k, const Tensor& v, const Tensor& a, const Tensor& b,
                     const Tensor& rate, const Tensor& dt_bias, double q_scale, double unit_eps, Tensor& S,
                     const Tensor& cu, const Tensor& slots, const Tensor& pos, c10::IntArrayRef lens, int64_t chunk_min) {
  c10::DeviceGuard g(q.device());
  TORCH_CHECK(head_rows(q, at::kFloat) && head_rows(k, at::kFloat) && k.sizes() == q.sizes(),
              "sx_delta_scan: q, k f32 [T, K, d] (heads contiguous in a row)");
  const int64_t T = q.size(0), K = q.size(1), d = q.size(2);
  TORCH_CHECK(head_rows(v, at::kFloat) && v.size(0) == T && K >= 1 && v.size(1) % K == 0,
              "sx_delta_scan: v f32 [T, H, dv], H a multiple of K");
  const int64_t H = v.size(1), dv = v.size(2);
  TORCH_CHECK(is_act(a) && strided(a, a.scalar_type(), T, H) && strided(b, a.scalar_type(), T, H),
              "sx_delta_scan: a, b [T, H] (unit inner stride)");
  TORCH_CHECK(vec(rate, at::kFloat, H) && vec(dt_bias, at::kFloat, H), "sx_delta_scan: rate, dt_bias f32 [H]");
  check_state(S, H, d, dv, "sx_delta_scan");
  check_step(cu, slots, pos, T, "sx_delta_scan");
  Tensor out = at::empty({T, H, dv}, q.options());
  if (T == 0) return out;
  check_lens(lens, cu, T, "sx_delta_scan");
  const illm::sx::DeltaArgs da{a.data_ptr(), a.stride(0), b.data_ptr(), b.stride(0), rate.data_ptr<float>(),
                               dt_bias.data_ptr<float>(), (float)q_scale, (float)unit_eps};
  if (by_chunks(lens, chunk_min, d)) {
    segments(lens, [&](int nch, int s0, int seg) {
      Tensor scratch = at::empty({illm::sx::chunk_scratch_floats(true, nch, (int)H, (int)d, (int)dv)}, out.options());
      illm::sx::delta_chunks(bf(a), q.data_ptr<float>(), q.stride(0), k.data_ptr<float>(), k.stride(0), v.data_ptr<float>(),
                             v.stride(0), da, S.data_ptr<float>(), cu.data_ptr<int32_t>(), slots.data_ptr<int32_t>(),
                             pos.data_ptr<int64_t>(), out.data_ptr<float>(), scratch.data_ptr<float>(), (int)cu.numel() - 1,
                             nch, s0, seg, (int)H, (int)K, (int)d, (int)dv, stream());
    });
    return out;
  }
  illm::sx::delta_scan(bf(a), q.data_ptr<float>(), q.stride(0), k.data_ptr<float>(), k.stride(0), v.data_ptr<float>(),
                       v.stride(0), da, S.data_ptr<float>(), cu.data_ptr<int32_t>(), slots.data_ptr<int32_t>(),
                       pos.data_ptr<int64_t>(), out.data_ptr<float>(), (int)cu.numel() - 1, (int)H, (int)K, (int)d, (int)dv,
                       stream());
  return out;
}

std::tuple<Tensor, Tensor> sx_rglru_gates(const Tensor& u, const Tensor& w_r, const Tensor& b_r, const Tensor& w_i,
                                          const Tensor& b_i, const Tensor& log_base) {
  c10::DeviceGuard g(u.device());
  check_x(u, "sx_rglru_gates");
  const int64_t T = u.size(0), C = u.size(1);
  TORCH_CHECK(w_r.is_cuda() && w_r.dim() == 3 && is_act(w_r) && w_r.is_contiguous() && w_r.size(1) == w_r.size(2) &&
                  w_r.size(0) * w_r.size(1) == C && w_i.is_cuda() && w_i.sizes() == w_r.sizes() &&
                  w_i.scalar_type() == w_r.scalar_type() && w_i.is_contiguous(),
              "sx_rglru_gates: gate matrices [blocks, n, n] with blocks n = C");
  TORCH_CHECK(vec(b_r, at::kFloat, C) && vec(b_i, at::kFloat, C) && vec(log_base, at::kFloat, C),
              "sx_rglru_gates: biases and log_base f32 [C]");
  const int64_t nb = w_r.size(0), n = w_r.size(1);
  TORCH_CHECK(nb * ((n + 63) / 64) <= 65535, "sx_rglru_gates: too many blocks for one launch");
  Tensor a = at::empty({T, C}, u.options()), x = at::empty({T, C}, u.options());
  illm::sx::rglru_gates(bf(w_r), u.data_ptr<float>(), w_r.data_ptr(), b_r.data_ptr<float>(), w_i.data_ptr(),
                        b_i.data_ptr<float>(), log_base.data_ptr<float>(), a.data_ptr<float>(), x.data_ptr<float>(), (int)T,
                        (int)nb, (int)n, stream());
  return {a, x};
}

Tensor sx_rglru_scan(const Tensor& a, const Tensor& x, const Tensor& y, Tensor& state, const Tensor& cu,
                     const Tensor& slots, const Tensor& pos, int64_t max_n) {
  c10::DeviceGuard g(a.device());
  check_x(a, "sx_rglru_scan");
  const int64_t T = a.size(0), C = a.size(1);
  TORCH_CHECK(rows(x, at::kFloat, T, C) && is_act(y) && strided(y, y.scalar_type(), T, C),
              "sx_rglru_scan: a, x f32 [T, C], y [T, C]");
  TORCH_CHECK(state.is_cuda() && state.scalar_type() == at::kFloat && state.is_contiguous() && state.dim() == 2 &&
                  state.size(1) == C,
              "sx_rglru_scan: state f32 [slots, C]");
  check_step(cu, slots, pos, T, "sx_rglru_scan");
  Tensor out = at::empty({T, C}, y.options());
  if (T == 0) return out;
  illm::sx::rglru_scan(bf(y), a.data_ptr<float>(), x.data_ptr<float>(), y.data_ptr(), y.stride(0), state.data_ptr<float>(),
                       cu.data_ptr<int32_t>(), slots.data_ptr<int32_t>(), pos.data_ptr<int64_t>(), out.data_ptr(),
                       (int)cu.numel() - 1, (int)C, (int)max_n, stream());
  return out;
}

}  // namespace

TORCH_LIBRARY_FRAGMENT(ipex_llm_amd, m) {
  m.def("sx_dyn_tanh(Tensor x, Tensor alpha, Tensor w, Tensor b, bool act_f32) -> Tensor");
  m.def("sx_add_normed(Tensor(a!) x, Tensor y, Tensor pa, Tensor pw, Tensor pb, Tensor? qa, Tensor? qw, Tensor? qb, "
        "bool act_f32) -> Tensor");
  m.def("sx_add_normed_pair(Tensor(a!) x, Tensor a, Tensor b, Tensor wa, Tensor wb, float eps, Tensor pa, Tensor pw, "
        "Tensor pb, Tensor? qa, Tensor? qw, Tensor? qb, bool act_f32) -> Tensor");
  m.def("sx_add_normed_experts(Tensor(a!) x, Tensor rows, Tensor idx, Tensor wts, Tensor h, int experts, Tensor pa, "
        "Tensor pw, Tensor pb, Tensor? qa, Tensor? qw, Tensor? qb, bool act_f32) -> Tensor");
  m.def("sx_rms_sigmoid_gate(Tensor o, Tensor w, Tensor gate, float eps, bool act_f32) -> Tensor");
  m.def("sx_route_groups(Tensor z, Tensor? corr, int top, int groups, int keep, bool sigmoid=False, bool best_two=False, "
        "bool renorm=False, float scale=1.0) -> (Tensor, Tensor)");
  m.def("sx_router(Tensor h, Tensor rw, Tensor? corr, int top, int groups, int keep, bool sigmoid=False, bool best_two=False, "
        "bool renorm=False, float scale=1.0) -> (Tensor, Tensor)");
  m.def("sx_decay_scan(Tensor q, Tensor k, Tensor v, Tensor decay, Tensor(a!) S, Tensor cu, Tensor slots, Tensor pos, "
        "int[] lens, int chunk_min) -> Tensor");
  m.def("sx_delta_scan(Tensor q, Tensor k, Tensor v, Tensor a, Tensor b, Tensor rate, Tensor dt_bias, float q_scale, "
        "float unit_eps, Tensor(a!) S, Tensor cu, Tensor slots, Tensor pos, int[] lens, int chunk_min) -> Tensor");
  m.def("sx_rglru_gates(Tensor u, Tensor w_r, Tensor b_r, Tensor w_i, Tensor b_i, Tensor log_base) -> (Tensor, Tensor)");
  m.def("sx_rglru_scan(Tensor a, Tensor x, Tensor y, Tensor(a!) state, Tensor cu, Tensor slots, Tensor pos, int max_n) "
        "-> Tensor");
}

TORCH_LIBRARY_IMPL(ipex_llm_amd, CUDA, m) {
  m.impl("sx_dyn_tanh", &sx_dyn_tanh);
  m.impl("sx_add_normed", &sx_add_normed);
  m.impl("sx_add_normed_pair", &sx_add_normed_pair);
  m.impl("sx_add_normed_experts", &sx_add_normed_experts);
  m.impl("sx_rms_sigmoid_gate", &sx_rms_sigmoid_gate);
  m.impl("sx_route_groups", &sx_route_groups);
  m.impl("sx_router", &sx_router);
  m.impl("sx_decay_scan", &sx_decay_scan);
  m.impl("sx_delta_scan", &sx_delta_scan);
  m.impl("sx_rglru_gates", &sx_rglru_gates);
  m.impl("sx_rglru_scan", &sx_rglru_scan);
}
