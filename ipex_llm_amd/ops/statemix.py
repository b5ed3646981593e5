"""Ops of the decoders whose sublayers are normed before and after
(models/hybrid.py ``SandwichLayer``) and of their recurrent mixers: the
statistics-free tanh norm fused with the residual sum, linear attention with a
fixed decay per head (lightning attention), the gated delta rule, the
real-gated linear recurrent unit with block-diagonal gates, and the routing of
experts in groups with a choice correction and identity experts.

Every op takes a *ragged step* like ``ops/seqmix.py``.  GPU tensors run the
HIP kernels of ``csrc/hip/statemix*.hip``; CPU tensors run the torch forms
below, which are also what the kernels are tested against.

Precision (both paths): norms, the residual sum, router scores and weights,
decays with their logarithms, step sizes, gates, unit norms, states and the
recurrences' sums are f32 whatever the activation dtype is.
"""
from __future__ import annotations

import math
import os
from dataclasses import dataclass
from typing import List, Optional, Tuple, Union

import torch
import torch.nn.functional as F

from .seqmix import native

__all__ = ["PairMean", "ExpertSum", "dyn_tanh", "add_normed_", "decay_scan", "delta_scan", "rms_sigmoid_gate",
           "rglru_gates", "rglru_scan", "RouteRule", "route_groups", "route", "SCAN_MAX_DIM"]

SCAN_MAX_DIM = 512             # largest key size per head the scan kernels hold (4 lanes x 128 state rows)

# GPU: a step with a portion of at least CHUNK_MIN tokens (0: never) runs the matrix-state recurrences in chunks of 64
# tokens on the matrix cores, other steps (decoding, short portions) token by token
CHUNK_MIN = int(os.environ.get("ILLM_STATE_CHUNK_MIN", "64"))


def _ops():
    return torch.ops.ipex_llm_amd


# ------------------------------------------------------------------ norm + residual
@dataclass
class PairMean:
    """A sublayer's result that is not formed yet: ``(rms_norm(a) wa + rms_norm(b) wb) / 2`` over rows [T, W]."""
    a: torch.Tensor
    b: torch.Tensor
    wa: torch.Tensor
    wb: torch.Tensor
    eps: float

    def value(self) -> torch.Tensor:
        a, b = self.a.float(), self.b.float()
        ya = a * torch.rsqrt((a * a).mean(-1, keepdim=True) + self.eps) * self.wa.float()
        yb = b * torch.rsqrt((b * b).mean(-1, keepdim=True) + self.eps) * self.wb.float()
        return 0.5 * (ya + yb)


@dataclass
class ExpertSum:
    """A sublayer's result that is not formed yet: the sum over a token's chosen experts of ``rows`` f32
    [T, top, W] (already weighted; the rows of identity experts hold nothing), where an index ``idx`` of
    ``experts`` or more is an identity expert: ``wts`` times the input ``h`` [T, W] itself."""
    rows: torch.Tensor
    idx: torch.Tensor
    wts: torch.Tensor
    h: torch.Tensor
    experts: int

    def value(self) -> torch.Tensor:
        same = (self.idx >= self.experts)[..., None]
        part = torch.where(same, self.wts[..., None] * self.h.float()[:, None], self.rows)
        return part.sum(1)


Source = Union[torch.Tensor, PairMean, ExpertSum]
Norm = Tuple[torch.Tensor, torch.Tensor, torch.Tensor]                  # alpha [1], w [W], b [W], all f32


def _dt(x: torch.Tensor, n: Norm) -> torch.Tensor:
    return torch.tanh(n[0] * x) * n[1] + n[2]


def dyn_tanh(x: torch.Tensor, n: Norm, act_dtype: torch.dtype) -> torch.Tensor:
    """``tanh(alpha x) w + b`` for f32 rows ``x`` [T, W] (one number alpha, vectors w and b); result in ``act_dtype``"""
    if native(x):
        return _ops().sx_dyn_tanh(x.contiguous(), *n, act_dtype == torch.float32)
    return _dt(x, n).to(act_dtype)


def add_normed_(x: torch.Tensor, y: Source, post: Norm, pre: Optional[Norm],
                act_dtype: torch.dtype) -> Optional[torch.Tensor]:
    """``x += post(y)`` on the f32 residual rows in place, then ``pre(x)`` in ``act_dtype`` (``pre`` None: no second
    norm, returns None): a sublayer's result normed and added, and the norm in front of the next sublayer, in one
    pass.  ``y`` is f32 or the activation dtype, or a ``PairMean`` / ``ExpertSum`` that the same pass forms."""
    if native(x):
        f32 = act_dtype == torch.float32
        p = (None, None, None) if pre is None else pre
        if isinstance(y, PairMean):
            h = _ops().sx_add_normed_pair(x, y.a.contiguous(), y.b.contiguous(), y.wa, y.wb, y.eps, *post, *p, f32)
        elif isinstance(y, ExpertSum):
            h = _ops().sx_add_normed_experts(x, y.rows, y.idx, y.wts, y.h.contiguous(), y.experts, *post, *p, f32)
        else:
            h = _ops().sx_add_normed(x, y.contiguous(), *post, *p, f32)
        return h if pre is not None else None
    v = y.float() if isinstance(y, torch.Tensor) else y.value()
    x.add_(_dt(v, post))
    return _dt(x, pre).to(act_dtype) if pre is not None else None


def rms_sigmoid_gate(o: torch.Tensor, w: torch.Tensor, gate_pre: torch.Tensor, eps: float,
                     out_dtype: torch.dtype) -> torch.Tensor:
    """``o`` f32 [T, C] divided by its root mean square (over the whole row), times ``w`` [C], times
    ``sigmoid(gate_pre)`` (``gate_pre`` [T, C], strided view allowed).  Returns [T, C] in ``out_dtype``."""
    if native(o):
        return _ops().sx_rms_sigmoid_gate(o.contiguous(), w, gate_pre, eps, out_dtype == torch.float32)
    n = o * torch.rsqrt((o * o).mean(-1, keepdim=True) + eps) * w.float()
    return (n * torch.sigmoid(gate_pre.float())).to(out_dtype)


# ------------------------------------------------------------------ matrix-state recurrences
def _sequences(q_lens: List[int], state_slots: torch.Tensor, pos: torch.Tensor):
    """(first token, tokens, slot, starts at position 0) of every sequence that brings tokens"""
    slots, first = state_slots.tolist(), pos.tolist()
    t0 = 0
    for s, n in enumerate(q_lens):
        if n:
            yield t0, n, slots[s], first[t0] == 0
        t0 += n


def decay_scan(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, decay: torch.Tensor, state: torch.Tensor,
               cu: torch.Tensor, state_slots: torch.Tensor, pos: torch.Tensor, q_lens: List[int]) -> torch.Tensor:
    """Linear attention with a fixed decay per head, token by token, per sequence and head.

    ``q`` / ``k`` [T, H, d], ``v`` [T, H, dv] as projected, in the activation
    dtype (strided views allowed); SiLU is applied to all three first.
    ``decay`` f32 [H]:

        S' = decay S + k v^T        [d, dv]
        o  = S'^T q                 [dv]

    ``state`` f32 [slots, H, d, dv] is read at ``state_slots[s]`` (a sequence
    whose first new token is at position 0 starts from zero instead) and written
    back after the last token.  Returns o f32 [T, H, dv]."""
    T, H, d = q.shape
    if native(q):
        if d > SCAN_MAX_DIM:
            raise ValueError(f"decay_scan: key size {d} is above the kernel's {SCAN_MAX_DIM}")
        return _ops().sx_decay_scan(q, k, v, decay, state, cu, state_slots, pos, q_lens, CHUNK_MIN)
    out = torch.empty(T, H, v.shape[2], dtype=torch.float32, device=q.device)
    qf, kf, vf = F.silu(q.float()), F.silu(k.float()), F.silu(v.float())
    dec = decay.float()[:, None, None]
    for t0, n, slot, fresh in _sequences(q_lens, state_slots, pos):
        S = torch.zeros_like(state[slot]) if fresh else state[slot].clone()
        for t in range(t0, t0 + n):
            S = dec * S + kf[t][:, :, None] * vf[t][:, None, :]
            out[t] = (S * qf[t][:, :, None]).sum(1)
        state[slot] = S
    return out


UNIT_EPS = 1e-6


def delta_scan(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, a_pre: torch.Tensor, b_pre: torch.Tensor,
               rate: torch.Tensor, dt_bias: torch.Tensor, q_scale: float, state: torch.Tensor, cu: torch.Tensor,
               state_slots: torch.Tensor, pos: torch.Tensor, q_lens: List[int]) -> torch.Tensor:
    """The gated delta rule, token by token, per sequence and head.

    ``q`` / ``k`` f32 [T, K, d] (head h reads key head h // (H / K)), ``v`` f32
    [T, H, dv] (strided views allowed); ``a_pre`` / ``b_pre`` [T, H] in the
    activation dtype (strided views), ``rate`` / ``dt_bias`` f32 [H].  q and k
    are first made unit vectors per head, x / sqrt(sum x^2 + 1e-6), and q is
    multiplied by ``q_scale``.  With beta = sigmoid(b_pre) and
    g = exp(-rate softplus(a_pre + dt_bias)):

        S <- g S;   u = beta (v - S^T k);   S <- S + k u^T;   o = S^T q

    ``state`` f32 [slots, H, d, dv] as in ``decay_scan``.  Returns o f32
    [T, H, dv]."""
    T, K, d = q.shape
    H, dv = v.shape[1], v.shape[2]
    if native(q):
        if d > SCAN_MAX_DIM:
            raise ValueError(f"delta_scan: key size {d} is above the kernel's {SCAN_MAX_DIM}")
        return _ops().sx_delta_scan(q, k, v, a_pre, b_pre, rate, dt_bias, q_scale, UNIT_EPS, state, cu, state_slots,
                                    pos, q_lens, CHUNK_MIN)
    rep = H // K
    out = torch.empty(T, H, dv, dtype=torch.float32, device=q.device)

    def unit(x):
        x = x.float()
        return (x / torch.sqrt((x * x).sum(-1, keepdim=True) + UNIT_EPS)).repeat_interleave(rep, 1)
    qf, kf, vf = unit(q) * q_scale, unit(k), v.float()
    beta = torch.sigmoid(b_pre.float())
    g = torch.exp(-rate.float() * F.softplus(a_pre.float() + dt_bias.float(), threshold=30.0))
    for t0, n, slot, fresh in _sequences(q_lens, state_slots, pos):
        S = torch.zeros_like(state[slot]) if fresh else state[slot].clone()
        for t in range(t0, t0 + n):
            S = g[t][:, None, None] * S
            u = beta[t][:, None] * (vf[t] - (S * kf[t][:, :, None]).sum(1))
            S = S + kf[t][:, :, None] * u[:, None, :]
            out[t] = (S * qf[t][:, :, None]).sum(1)
        state[slot] = S
    return out


# ------------------------------------------------------------------ real-gated linear recurrent unit
def rglru_gates(u: torch.Tensor, w_r: torch.Tensor, b_r: torch.Tensor, w_i: torch.Tensor, b_i: torch.Tensor,
                log_base: torch.Tensor) -> Tuple[torch.Tensor, torch.Tensor]:
    """Gates of the recurrence for rows ``u`` f32 [T, C], split into ``blocks``
    equal parts: per part b

        r = sigmoid(w_r[b] u_b + b_r[b]),   i = sigmoid(w_i[b] u_b + b_i[b])

    (``w_r`` / ``w_i`` [blocks, n, n] as [out, in], biases f32 [C]), and with
    log a = r * log_base (``log_base`` f32 [C], negative):

        a = exp(log a),   x = sqrt(1 - a^2) i u

    Returns ``a`` and ``x`` f32 [T, C]."""
    if native(u):
        return _ops().sx_rglru_gates(u, w_r, b_r, w_i, b_i, log_base)
    T, C = u.shape
    nb, n, _ = w_r.shape
    ub = u.float().view(T, nb, n).transpose(0, 1)                        # [nb, T, n]
    zr = torch.bmm(ub, w_r.float().transpose(1, 2)).transpose(0, 1).reshape(T, C) + b_r
    zi = torch.bmm(ub, w_i.float().transpose(1, 2)).transpose(0, 1).reshape(T, C) + b_i
    la = torch.sigmoid(zr) * log_base
    return torch.exp(la), torch.sqrt(-torch.expm1(2.0 * la)) * torch.sigmoid(zi) * u.float()


def rglru_scan(a: torch.Tensor, x: torch.Tensor, y_pre: torch.Tensor, state: torch.Tensor, cu: torch.Tensor,
               state_slots: torch.Tensor, pos: torch.Tensor, q_lens: List[int]) -> torch.Tensor:
    """``S_t = a_t S_(t-1) + x_t`` element by element (``a`` / ``x`` f32 [T, C]),
    out_t = S_t gelu_tanh(y_pre_t) (``y_pre`` [T, C] in the activation dtype,
    strided view allowed).  ``state`` f32 [slots, C] as in ``decay_scan``.
    Returns [T, C] in y_pre's dtype."""
    if native(a):
        return _ops().sx_rglru_scan(a, x, y_pre, state, cu, state_slots, pos, max(q_lens))
    out = torch.empty_like(a)
    yf = y_pre.float()
    g = 0.5 * yf * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (yf + 0.044715 * yf * yf * yf)))
    for t0, n, slot, fresh in _sequences(q_lens, state_slots, pos):
        S = torch.zeros_like(state[slot]) if fresh else state[slot].clone()
        for t in range(t0, t0 + n):
            S = a[t] * S + x[t]
            out[t] = S * g[t]
        state[slot] = S
    return out.to(y_pre.dtype)


# ------------------------------------------------------------------ routing
@dataclass
class RouteRule:
    """How router logits become scores and weights.  ``score``: "softmax" over all router outputs, or "sigmoid";
    ``group``: a group's score is its "max" corrected score, or the sum of its two largest ("top2"); ``renorm``: the
    winners' scores are divided by their sum (+ 1e-20) and multiplied by ``scale``."""
    score: str = "softmax"
    group: str = "max"
    renorm: bool = False
    scale: float = 1.0

    def __post_init__(self):
        if self.score not in ("softmax", "sigmoid") or self.group not in ("max", "top2"):
            raise ValueError(f"unknown routing rule {self}")
        if not self.renorm and self.scale != 1.0:
            raise ValueError("a routing scale belongs to renormalised weights")

    def args(self):
        return self.score == "sigmoid", self.group == "top2", self.renorm, float(self.scale)


SOFTMAX_RULE = RouteRule()


def route_groups(z: torch.Tensor, correction: Optional[torch.Tensor], top: int, groups: int, keep: int,
                 rule: RouteRule = SOFTMAX_RULE) -> Tuple[torch.Tensor, torch.Tensor]:
    """Router logits ``z`` f32 [T, E] -> the chosen experts (int32 [T, top]) and
    their weights (f32 [T, top]).  Scores s = softmax(z) over all E (or sigmoids,
    ``rule``); the choice goes by c = s + ``correction`` (f32 [E] or None).  The E
    experts form ``groups`` equal groups of neighbours; the ``keep`` groups with
    the largest best c (or sum of the two best) stay, the others' experts cannot
    be chosen.  The ``top`` largest c win (lowest index first among equals, groups
    alike); the weights are their s, as they are or renormalised."""
    T, E = z.shape
    if native(z) and E <= 512:
        return _ops().sx_route_groups(z.contiguous(), correction, top, groups, keep, *rule.args())
    s = torch.sigmoid(z.float()) if rule.score == "sigmoid" else torch.softmax(z.float(), -1)
    c = s + correction.float() if correction is not None else s
    if keep < groups:
        n = min(2 if rule.group == "top2" else 1, E // groups)
        best = c.view(T, groups, E // groups).topk(n, -1).values.sum(-1)
        kept = torch.sort(best, dim=-1, descending=True, stable=True).indices[:, :keep]
        ok = torch.zeros(T, groups, dtype=torch.bool, device=z.device).scatter_(1, kept, True)
        c = c.masked_fill(~ok.repeat_interleave(E // groups, 1), float("-inf"))
    idx = torch.sort(c, dim=-1, descending=True, stable=True).indices[:, :top]
    w = s.gather(1, idx)
    if rule.renorm:
        w = w * (rule.scale / (w.sum(-1, keepdim=True) + 1e-20))
    return idx.to(torch.int32).contiguous(), w.contiguous()


ROUTER_MAX_T = 64              # GPU: up to this many tokens the logits and the routing are one launch


def route(h: torch.Tensor, router: torch.Tensor, correction: Optional[torch.Tensor], top: int, groups: int,
          keep: int, rule: RouteRule = SOFTMAX_RULE) -> Tuple[torch.Tensor, torch.Tensor]:
    """``route_groups`` of the logits ``h router^T`` (f32 products; ``h`` [T, W] in the activation dtype, ``router``
    f32 [E, W])"""
    if native(h) and h.shape[0] <= ROUTER_MAX_T and router.shape[0] <= 512:
        return _ops().sx_router(h.contiguous(), router, correction, top, groups, keep, *rule.args())
    return route_groups(F.linear(h.float(), router), correction, top, groups, keep, rule)
