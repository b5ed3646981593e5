// torch.ops.ipex_llm_amd.cx_*: the kernels of the mixers with per-channel decays
// and of the pre-norm blocks with scaled sublayers (csrc/hip/chanmix*.hip).  Every
// entry checks on the host that the operand shapes, dtypes and strides are what
// its kernel and grid assume.
#include <ATen/ATen.h>
#include <ATen/hip/HIPContext.h>
#include <c10/core/DeviceGuard.h>
#include <torch/library.h>

#include <algorithm>

#include "../hip/chanmix.h"
#include "../hip/statemix.h"

using at::Tensor;
using OptT = c10::optional<Tensor>;
using illm::cx::Source;

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
void check_x(const Tensor& x, const char* what) {
  TORCH_CHECK(x.is_cuda() && x.dim() == 2 && x.scalar_type() == at::kFloat && x.is_contiguous() && x.size(1) >= 1 &&
                  x.size(1) <= 1 << 22,
              what, ": x f32 [T, W] contiguous");
}

// a [T, W] (activation type or f32) or expert rows f32 [T, top, W], sa f32 [W]; b like a with sb, or none
Source source(const OptT& a, const OptT& sa, const OptT& b, const OptT& sb, int64_t T, int64_t W, bool act_f32,
              const char* what) {
  Source y{nullptr, nullptr, nullptr, nullptr, 0, false};
  if (!has(a)) return y;
  TORCH_CHECK(has(sa) && vec(*sa, at::kFloat, W), what, ": scale f32 [W]");
  y.a = a->data_ptr();
  y.sa = sa->data_ptr<float>();
  if (a->dim() == 3) {
    TORCH_CHECK(a->size(0) == T && a->size(1) >= 1 && a->size(2) == W && vec(*a, at::kFloat, a->numel()) && !has(b), what,
                ": expert rows f32 [T, top, W]");
    y.top = (int)a->size(1);
    return y;
  }
  const auto ty = act_type(act_f32);
  y.a_f32 = a->scalar_type() == at::kFloat && !act_f32;
  TORCH_CHECK(rows(*a, y.a_f32 ? at::kFloat : ty, T, W), what, ": result [T, W] contiguous");
  if (has(b)) {
    TORCH_CHECK(!y.a_f32 && rows(*b, ty, T, W) && has(sb) && vec(*sb, at::kFloat, W), what,
                ": two results [T, W] in the activation dtype, scales f32 [W]");
    y.b = b->data_ptr();
    y.sb = sb->data_ptr<float>();
  }
  return y;
}

Tensor cx_add_scaled_norm(Tensor& x, const OptT& a, const OptT& sa, const OptT& b, const OptT& sb, const Tensor& w,
                          double eps, bool act_f32) {
  c10::DeviceGuard g(x.device());
  check_x(x, "cx_add_scaled_norm");
  const int64_t T = x.size(0), W = x.size(1);
  TORCH_CHECK(vec(w, at::kFloat, W), "cx_add_scaled_norm: weight f32 [W]");
  const Source y = source(a, sa, b, sb, T, W, act_f32, "cx_add_scaled_norm");
  Tensor out = at::empty({T, W}, x.options().dtype(act_type(act_f32)));
  illm::cx::add_scaled_norm(!act_f32, x.data_ptr<float>(), y, w.data_ptr<float>(), (float)eps, out.data_ptr(), (int)T,
                            (int)W, stream());
  return out;
}

Tensor cx_loop_input(const Tensor& x, const OptT& a, const OptT& sa, const OptT& b, const OptT& sb, const Tensor& embed,
                     const Tensor& ids) {
  c10::DeviceGuard g(x.device());
  check_x(x, "cx_loop_input");
  const int64_t T = x.size(0), W = x.size(1);
  TORCH_CHECK(embed.is_cuda() && embed.dim() == 2 && is_act(embed) && embed.is_contiguous() && embed.size(1) == W,
              "cx_loop_input: embedding table [vocab, W] contiguous");
  TORCH_CHECK(vec(ids, at::kLong, T), "cx_loop_input: ids int64 [T]");
  const bool act_f32 = embed.scalar_type() == at::kFloat;
  const Source y = source(a, sa, b, sb, T, W, act_f32, "cx_loop_input");
  Tensor out = at::empty({T, 2 * W}, embed.options());
  illm::cx::loop_input(!act_f32, x.data_ptr<float>(), y, embed.data_ptr(), embed.size(0), ids.data_ptr<int64_t>(),
                       out.data_ptr(), (int)T, (int)W, stream());
  return out;
}

Tensor cx_token_mixes(const Tensor& h, const Tensor& mu, Tensor& state, const Tensor& cu, const Tensor& seq_of,
                      const Tensor& slots, const Tensor& pos, bool single) {
  c10::DeviceGuard g(h.device());
  TORCH_CHECK(h.is_cuda() && h.dim() == 2 && is_act(h) && h.is_contiguous(), "cx_token_mixes: h [T, W] contiguous");
  const int64_t T = h.size(0), W = h.size(1);
  TORCH_CHECK(mu.dim() == 2 && rows(mu, at::kFloat, mu.size(0), W), "cx_token_mixes: mu f32 [mixes, W]");
  TORCH_CHECK(state.is_cuda() && state.scalar_type() == at::kFloat && state.is_contiguous() && state.dim() == 2 &&
                  state.size(1) == W,
              "cx_token_mixes: state f32 [slots, W]");
  check_step(cu, slots, pos, T, "cx_token_mixes");
  TORCH_CHECK(seq_of.is_cuda() && seq_of.scalar_type() == at::kInt && seq_of.is_contiguous() && seq_of.numel() >= T,
              "cx_token_mixes: seq_of int32 [T]");
  TORCH_CHECK(!single || cu.numel() - 1 == T, "cx_token_mixes: one token per sequence");
  Tensor out = at::empty({mu.size(0), T, W}, h.options());
  illm::cx::token_mixes(bf(h), h.data_ptr(), mu.data_ptr<float>(), (int)mu.size(0), state.data_ptr<float>(),
                        cu.data_ptr<int32_t>(), seq_of.data_ptr<int32_t>(), slots.data_ptr<int32_t>(),
                        pos.data_ptr<int64_t>(), out.data_ptr(), (int)T, (int)cu.numel() - 1, (int)W, single, stream());
  return out;
}

Tensor cx_lowrank_decay(const Tensor& in, const Tensor& w, const OptT& rate, const Tensor& bias, int64_t kind, bool squash) {
  c10::DeviceGuard g(in.device());
  TORCH_CHECK(w.is_cuda() && w.dim() == 2 && is_act(w) && w.is_contiguous(), "cx_lowrank_decay: w [N, R] contiguous");
  const int64_t N = w.size(0), R = w.size(1), T = in.size(0);
  TORCH_CHECK(R >= 1 && strided(in, w.scalar_type(), T, R), "cx_lowrank_decay: input [T, R] of w's dtype (unit inner stride)");
  TORCH_CHECK(kind == 0 || kind == 1, "cx_lowrank_decay: kind 0 (softplus) or 1 (exp)");
  TORCH_CHECK(vec(bias, at::kFloat, N) && (kind == 1 || (has(rate) && vec(*rate, at::kFloat, N))),
              "cx_lowrank_decay: bias and rate f32 [N]");
  TORCH_CHECK((N + 63) / 64 <= 65535, "cx_lowrank_decay: too many outputs for one launch");
  Tensor out = at::empty({T, N}, in.options().dtype(at::kFloat));
  illm::cx::lowrank_decay(bf(w), in.data_ptr(), in.stride(0), w.data_ptr(), kind == 0 ? rate->data_ptr<float>() : nullptr,
                          bias.data_ptr<float>(), (int)kind, squash, out.data_ptr<float>(), (int)T, (int)N, (int)R, stream());
  return out;
}

// xs: one input [M, K] per row group, sizes: the groups' weight rows, w [sum of sizes, K], bias [N] or none
Tensor cx_grouped_linear(at::TensorList xs, c10::IntArrayRef sizes, const Tensor& w, const OptT& bias, bool out_f32) {
  TORCH_CHECK(!xs.empty() && xs.size() == sizes.size() && xs.size() <= (size_t)illm::cx::kMaxGroups,
              "cx_grouped_linear: one input per row group, at most ", illm::cx::kMaxGroups, " groups");
  c10::DeviceGuard g(w.device());
  const int64_t K = w.size(1), M = xs[0].size(0);
  TORCH_CHECK(w.is_cuda() && w.dim() == 2 && bf(w) && w.is_contiguous() && K % 64 == 0 && M <= 16,
              "cx_grouped_linear: 16-bit w [N, K], K a multiple of 64, at most 16 rows");
  illm::cx::Groups gr{};
  gr.n = (int)xs.size();
  int64_t row = 0, tile = 0;
  for (int i = 0; i < gr.n; i++) {
    TORCH_CHECK(rows(xs[i], at::kBFloat16, M, K) && (uintptr_t)xs[i].data_ptr() % 16 == 0 && sizes[i] >= 1,
                "cx_grouped_linear: inputs [M, K] contiguous, no empty group");
    gr.x[i] = xs[i].data_ptr();
    gr.row0[i] = (int)row;
    gr.tile0[i] = (int)tile;
    row += sizes[i];
    tile += (sizes[i] + 15) / 16;
  }
  gr.row0[gr.n] = (int)row;
  gr.tile0[gr.n] = (int)tile;
  TORCH_CHECK(row == w.size(0) && row < (int64_t)1 << 30, "cx_grouped_linear: the groups' rows must be w's");
  TORCH_CHECK(!has(bias) || vec(*bias, at::kBFloat16, row), "cx_grouped_linear: bias [N]");
  Tensor out = at::empty({M, row}, w.options().dtype(out_f32 ? at::kFloat : at::kBFloat16));
  illm::cx::grouped_linear(gr, (int)M, (int)K, w.data_ptr(), has(bias) ? bias->data_ptr() : nullptr, out.data_ptr(), out_f32,
                           stream());
  return out;
}

// ------------------------------------------------------------------ recurrences
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

Tensor cx_delta_scan(const Tensor& q, const Tensor& k, const Tensor& v, const Tensor& gd, const Tensor& b, double q_scale,
                     double unit_eps, Tensor& S, const Tensor& cu, const Tensor& slots, const Tensor& pos,
                     c10::IntArrayRef lens, int64_t chunk_min) {
  c10::DeviceGuard g(q.device());
  TORCH_CHECK(head_rows(q, at::kFloat) && head_rows(k, at::kFloat) && k.sizes() == q.sizes(),
              "cx_delta_scan: q, k f32 [T, K, d] (heads contiguous in a row)");
  const int64_t T = q.size(0), K = q.size(1), d = q.size(2);
  TORCH_CHECK(head_rows(v, at::kFloat) && v.size(0) == T && K >= 1 && v.size(1) % K == 0,
              "cx_delta_scan: v f32 [T, H, dv], H a multiple of K");
  const int64_t H = v.size(1), dv = v.size(2);
  TORCH_CHECK(is_act(b) && strided(b, b.scalar_type(), T, H), "cx_delta_scan: b [T, H] (unit inner stride)");
  TORCH_CHECK(vec(gd, at::kFloat, T * H * d), "cx_delta_scan: decays f32 [T, H, d]");
  check_state(S, H, d, dv, "cx_delta_scan");
  check_step(cu, slots, pos, T, "cx_delta_scan");
  Tensor out = at::empty({T, H, dv}, q.options());
  if (T == 0) return out;
  check_lens(lens, cu, T, "cx_delta_scan");
  const illm::cx::DeltaIn di{b.data_ptr(), b.stride(0), (float)q_scale, (float)unit_eps};
  const int B = (int)cu.numel() - 1;
  if (by_chunks(lens, chunk_min, d)) {
    segments(lens, [&](int nch, int s0, int seg) {
      Tensor scratch = at::empty({illm::cx::chunk_scratch_floats(true, nch, (int)H, (int)d, (int)dv)}, out.options());
      illm::cx::delta_chunks(bf(b), q.data_ptr<float>(), q.stride(0), k.data_ptr<float>(), k.stride(0), v.data_ptr<float>(),
                             v.stride(0), gd.data_ptr<float>(), di, S.data_ptr<float>(), cu.data_ptr<int32_t>(),
                             slots.data_ptr<int32_t>(), pos.data_ptr<int64_t>(), out.data_ptr<float>(),
                             scratch.data_ptr<float>(), B, nch, s0, seg, (int)H, (int)K, (int)d, (int)dv, stream());
    });
    return out;
  }
  illm::cx::delta_scan(bf(b), q.data_ptr<float>(), q.stride(0), k.data_ptr<float>(), k.stride(0), v.data_ptr<float>(),
                       v.stride(0), gd.data_ptr<float>(), di, S.data_ptr<float>(), cu.data_ptr<int32_t>(),
                       slots.data_ptr<int32_t>(), pos.data_ptr<int64_t>(), out.data_ptr<float>(), B, (int)H, (int)K, (int)d,
                       (int)dv, stream());
  return out;
}

Tensor cx_bonus_scan(const Tensor& r, const Tensor& k, const Tensor& v, const Tensor& gd, const Tensor& u, Tensor& S,
                     const Tensor& cu, const Tensor& slots, const Tensor& pos, c10::IntArrayRef lens, int64_t chunk_min) {
  c10::DeviceGuard g(r.device());
  const auto ty = r.scalar_type();
  TORCH_CHECK(is_act(r) && head_rows(r, ty) && head_rows(k, ty) && k.sizes() == r.sizes(),
              "cx_bonus_scan: r, k [T, H, d] (heads contiguous in a row)");
  const int64_t T = r.size(0), H = r.size(1), d = r.size(2);
  TORCH_CHECK(head_rows(v, ty) && v.size(0) == T && v.size(1) == H, "cx_bonus_scan: v [T, H, dv]");
  const int64_t dv = v.size(2);
  TORCH_CHECK(vec(gd, at::kFloat, T * H * d) && vec(u, at::kFloat, H * d),
              "cx_bonus_scan: decays f32 [T, H, d], bonus f32 [H, d]");
  check_state(S, H, d, dv, "cx_bonus_scan");
  check_step(cu, slots, pos, T, "cx_bonus_scan");
  Tensor out = at::empty({T, H, dv}, r.options().dtype(at::kFloat));
  if (T == 0) return out;
  check_lens(lens, cu, T, "cx_bonus_scan");
  const int B = (int)cu.numel() - 1;
  if (by_chunks(lens, chunk_min, d)) {
    segments(lens, [&](int nch, int s0, int seg) {
      Tensor scratch = at::empty({illm::cx::chunk_scratch_floats(false, nch, (int)H, (int)d, (int)dv)}, out.options());
      illm::cx::bonus_chunks(bf(r), r.data_ptr(), r.stride(0), k.data_ptr(), k.stride(0), v.data_ptr(), v.stride(0),
                             gd.data_ptr<float>(), u.data_ptr<float>(), S.data_ptr<float>(), cu.data_ptr<int32_t>(),
                             slots.data_ptr<int32_t>(), pos.data_ptr<int64_t>(), out.data_ptr<float>(),
                             scratch.data_ptr<float>(), B, nch, s0, seg, (int)H, (int)d, (int)dv, stream());
    });
    return out;
  }
  illm::cx::bonus_scan(bf(r), r.data_ptr(), r.stride(0), k.data_ptr(), k.stride(0), v.data_ptr(), v.stride(0),
                       gd.data_ptr<float>(), u.data_ptr<float>(), S.data_ptr<float>(), cu.data_ptr<int32_t>(),
                       slots.data_ptr<int32_t>(), pos.data_ptr<int64_t>(), out.data_ptr<float>(), B, (int)H, (int)d, (int)dv,
                       stream());
  return out;
}

}  // namespace

TORCH_LIBRARY_FRAGMENT(ipex_llm_amd, m) {
  m.def("cx_add_scaled_norm(Tensor(a!) x, Tensor? a, Tensor? sa, Tensor? b, Tensor? sb, Tensor w, float eps, bool act_f32) "
        "-> Tensor");
  m.def("cx_loop_input(Tensor x, Tensor? a, Tensor? sa, Tensor? b, Tensor? sb, Tensor embed, Tensor ids) -> Tensor");
  m.def("cx_token_mixes(Tensor h, Tensor mu, Tensor(a!) state, Tensor cu, Tensor seq_of, Tensor slots, Tensor pos, "
        "bool single) -> Tensor");
  m.def("cx_lowrank_decay(Tensor inp, Tensor w, Tensor? rate, Tensor bias, int kind, bool squash) -> Tensor");
  m.def("cx_grouped_linear(Tensor[] xs, int[] sizes, Tensor w, Tensor? bias, bool out_f32=False) -> Tensor");
  m.def("cx_delta_scan(Tensor q, Tensor k, Tensor v, Tensor g, Tensor b, float q_scale, float unit_eps, Tensor(a!) S, "
        "Tensor cu, Tensor slots, Tensor pos, int[] lens, int chunk_min) -> Tensor");
  m.def("cx_bonus_scan(Tensor r, Tensor k, Tensor v, Tensor g, Tensor u, Tensor(a!) S, Tensor cu, Tensor slots, "
        "Tensor pos, int[] lens, int chunk_min) -> Tensor");
}

TORCH_LIBRARY_IMPL(ipex_llm_amd, CUDA, m) {
  m.impl("cx_add_scaled_norm", &cx_add_scaled_norm);
  m.impl("cx_loop_input", &cx_loop_input);
  m.impl("cx_token_mixes", &cx_token_mixes);
  m.impl("cx_lowrank_decay", &cx_lowrank_decay);
  m.impl("cx_grouped_linear", &cx_grouped_linear);
  m.impl("cx_delta_scan", &cx_delta_scan);
  m.impl("cx_bonus_scan", &cx_bonus_scan);
}
