"""Ops of the mixers whose decay has one number per key channel and of the
pre-norm blocks with scaled sublayers around them (models/hybrid.py
``ChannelDelta``, ``TimeMix``, ``ScaledSum``, ``PreNormLayer``): the scaled
residual sum fused with the next norm, the input rows of the projection in front
of a loop's pass, the blends of a token's and its predecessor's row, low-rank
decays, projections whose row groups read different inputs, and the two
recurrences (delta rule, and read-out before the write with a bonus).

Every op takes a *ragged step* like ``ops/seqmix.py``.  GPU tensors run the
HIP kernels of ``csrc/hip/chanmix*.hip``; CPU tensors run the torch forms
below, which are also what the kernels are tested against.

Precision (both paths): norms, the residual sum, decays with their logarithms,
softplus and exponentials, step sizes, unit norms, states and the recurrences'
sums are f32 whatever the activation dtype is.
"""
from __future__ import annotations

import os
from dataclasses import dataclass
from typing import List, Optional, Sequence

import torch
import torch.nn.functional as F

from .seqmix import _mm_f32, native
from .statemix import SCAN_MAX_DIM, UNIT_EPS, _sequences

__all__ = ["Pending", "add_scaled_norm_", "loop_input", "linear_f32", "token_mixes", "lowrank_decay", "grouped_linear",
           "grouped_fits", "channel_delta_scan", "bonus_scan"]

# GPU: a step with a portion of at least CHUNK_MIN tokens (0: never) runs the recurrences in chunks of 64 tokens on the
# matrix cores, other steps (decoding, short portions) token by token
CHUNK_MIN = int(os.environ.get("ILLM_CHANNEL_CHUNK_MIN", "64"))


def _ops():
    return torch.ops.ipex_llm_amd


def _single(q_lens: List[int], T: int) -> bool:
    return len(q_lens) == T and all(n == 1 for n in q_lens)


# ------------------------------------------------------------------ residual stream
@dataclass
class Pending:
    """A sublayer's result that is not in the residual stream yet: ``sa a + sb b`` row by row (``b`` may be None), with
    scales f32 [W]; ``a`` [T, W] in the activation dtype or f32, or f32 [T, top, W] (a token's weighted expert rows,
    summed first)."""
    a: torch.Tensor
    sa: torch.Tensor
    b: Optional[torch.Tensor] = None
    sb: Optional[torch.Tensor] = None

    def value(self) -> torch.Tensor:
        v = self.sa * (self.a.float() if self.a.dim() == 2 else self.a.sum(1))
        return v if self.b is None else v + self.sb * self.b.float()

    def select(self, idx: torch.Tensor) -> "Pending":
        return Pending(self.a.index_select(0, idx), self.sa, None if self.b is None else self.b.index_select(0, idx), self.sb)

    def args(self):
        return self.a.contiguous(), self.sa, None if self.b is None else self.b.contiguous(), self.sb


_NOTHING = (None, None, None, None)


def add_scaled_norm_(x: torch.Tensor, y: Optional[Pending], w: torch.Tensor, eps: float,
                     act_dtype: torch.dtype) -> torch.Tensor:
    """``x += y`` on the f32 residual rows in place, then ``x / sqrt(mean(x^2) + eps) * w`` (``w`` f32 [W]) in
    ``act_dtype``: one sublayer's scaled residual sum and the norm in front of the next in one pass."""
    if native(x):
        return _ops().cx_add_scaled_norm(x, *(y.args() if y is not None else _NOTHING), w, eps, act_dtype == torch.float32)
    if y is not None:
        x.add_(y.value())
    return (x * torch.rsqrt((x * x).mean(-1, keepdim=True) + eps) * w).to(act_dtype)


def loop_input(x: torch.Tensor, y: Optional[Pending], embed: torch.Tensor, ids: torch.Tensor) -> torch.Tensor:
    """``[x + y | embed[ids]]`` [T, 2 W] in the table's dtype (``x`` f32 is left as it is)."""
    if native(x):
        return _ops().cx_loop_input(x, *(y.args() if y is not None else _NOTHING), embed, ids.contiguous())
    v = x if y is None else x + y.value()
    return torch.cat([v.to(embed.dtype), embed[ids.long()]], -1)


def grouped_fits(M: int, w: torch.Tensor) -> bool:
    """decode-size steps that ``grouped_linear`` serves on the GPU (16-bit weights, at most 16 rows)"""
    return w.is_cuda and w.dtype == torch.bfloat16 and M <= 16 and w.shape[1] % 64 == 0


def grouped_linear(xs: Sequence[torch.Tensor], sizes: Sequence[int], w: torch.Tensor, b: Optional[torch.Tensor] = None,
                   f32: bool = False) -> torch.Tensor:
    """A projection whose row groups read different inputs: the first ``sizes[0]`` rows of ``w`` [N, K] (and of ``b``)
    times ``xs[0]`` [M, K], the next ``sizes[1]`` times ``xs[1]``, ...; one launch (see ``grouped_fits``).  Returns
    [M, N] in w's dtype, or f32."""
    if native(w):
        return _ops().cx_grouped_linear(list(xs), list(sizes), w, b, f32)
    out, lo = [], 0
    for x, n in zip(xs, sizes):
        y = x.float() @ w[lo:lo + n].float().t()
        out.append(y if b is None else y + b[lo:lo + n].float())
        lo += n
    y = torch.cat(out, -1)
    return y if f32 else y.to(w.dtype)


def linear_f32(x: torch.Tensor, w: torch.Tensor) -> torch.Tensor:
    """``x W^T`` with an f32 result (16-bit operands: f32 accumulation, the result is not rounded)"""
    if grouped_fits(x.shape[0], w):
        return grouped_linear([x], [w.shape[0]], w, None, True)
    return _mm_f32(x, w.t())


# ------------------------------------------------------------------ inputs of the recurrences
def token_mixes(h: torch.Tensor, mu: torch.Tensor, state: torch.Tensor, cu: torch.Tensor, seq_of: torch.Tensor,
                state_slots: torch.Tensor, pos: torch.Tensor, q_lens: List[int]) -> torch.Tensor:
    """``h_t + (h_(t-1) - h_t) mu[m]`` for every row of ``mu`` f32 [mixes, W]; ``h`` [T, W] in the activation dtype.

    ``h_(t-1)`` is zero at position 0; before a portion's first token it is what ``state`` f32 [slots, W] holds for the
    sequence, and every portion leaves its last row there.  Returns [mixes, T, W] in h's dtype."""
    T = h.shape[0]
    if native(h):
        return _ops().cx_token_mixes(h.contiguous(), mu, state, cu, seq_of, state_slots, pos, _single(q_lens, T))
    hf = h.float()
    prev = torch.zeros_like(hf)
    for t0, n, slot, fresh in _sequences(q_lens, state_slots, pos):
        prev[t0 + 1:t0 + n] = hf[t0:t0 + n - 1]
        if not fresh:
            prev[t0] = state[slot]
        state[slot] = hf[t0 + n - 1]
    return (hf[None] + (prev - hf)[None] * mu[:, None]).to(h.dtype)


DECAYS = {"softplus": 0, "exp": 1}


def lowrank_decay(a: torch.Tensor, w: torch.Tensor, rate: Optional[torch.Tensor], bias: torch.Tensor, kind: str,
                  squash: bool = False) -> torch.Tensor:
    """The second product of a low-rank projection turned into decays: z = a W^T + bias (``a`` [T, R] in the
    activation dtype, a strided view is allowed; ``squash``: tanh(a) instead of a; ``w`` [N, R]; f32 sums), then

        kind "softplus":  exp(-rate softplus(z))        kind "exp":  exp(-exp(z))

    ``rate`` / ``bias`` f32 [N].  Returns f32 [T, N]."""
    if native(a):
        return _ops().cx_lowrank_decay(a, w, rate, bias, DECAYS[kind], squash)
    af = torch.tanh(a.float()) if squash else a.float()
    z = af @ w.float().t() + bias
    if kind == "softplus":
        return torch.exp(-rate * F.softplus(z, threshold=30.0))
    return torch.exp(-torch.exp(z))


# ------------------------------------------------------------------ recurrences
def channel_delta_scan(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, g: torch.Tensor, b_pre: torch.Tensor,
                       q_scale: float, state: torch.Tensor, cu: torch.Tensor, state_slots: torch.Tensor,
                       pos: torch.Tensor, q_lens: List[int]) -> torch.Tensor:
    """The delta rule with one decay per key channel, token by token, per sequence and head.

    ``q`` / ``k`` f32 [T, K, d] (head h reads key head h // (H / K)), ``v`` f32 [T, H, dv] (strided views allowed),
    ``g`` f32 [T, H, d] the decays, ``b_pre`` [T, H] in the activation dtype (strided view).  q and k are first made
    unit vectors per head, x / sqrt(sum x^2 + 1e-6), and q is multiplied by ``q_scale``.  With beta = sigmoid(b_pre):

        S <- diag(g) S;   u = beta (v - S^T k);   S <- S + k u^T;   o = S^T q

    ``state`` f32 [slots, H, d, dv] is read at ``state_slots[s]`` (a sequence whose first new token is at position 0
    starts from zero instead) and written back after the last token.  Returns o f32 [T, H, dv]."""
    T, K, d = q.shape
    H, dv = v.shape[1], v.shape[2]
    if native(q):
        if d > SCAN_MAX_DIM:
            raise ValueError(f"channel_delta_scan: key size {d} is above the kernel's {SCAN_MAX_DIM}")
        return _ops().cx_delta_scan(q, k, v, g.contiguous(), b_pre, q_scale, UNIT_EPS, state, cu, state_slots, pos, q_lens,
                                    CHUNK_MIN)
    rep = H // K
    out = torch.empty(T, H, dv, dtype=torch.float32, device=q.device)

    def unit(x):
        x = x.float()
        return (x / torch.sqrt((x * x).sum(-1, keepdim=True) + UNIT_EPS)).repeat_interleave(rep, 1)
    qf, kf, vf = unit(q) * q_scale, unit(k), v.float()
    beta = torch.sigmoid(b_pre.float())
    for t0, n, slot, fresh in _sequences(q_lens, state_slots, pos):
        S = torch.zeros_like(state[slot]) if fresh else state[slot].clone()
        for t in range(t0, t0 + n):
            S = g[t][:, :, None] * S
            u = beta[t][:, None] * (vf[t] - (S * kf[t][:, :, None]).sum(1))
            S = S + kf[t][:, :, None] * u[:, None, :]
            out[t] = (S * qf[t][:, :, None]).sum(1)
        state[slot] = S
    return out


def bonus_scan(r: torch.Tensor, k: torch.Tensor, v: torch.Tensor, g: torch.Tensor, u: torch.Tensor, state: torch.Tensor,
               cu: torch.Tensor, state_slots: torch.Tensor, pos: torch.Tensor, q_lens: List[int]) -> torch.Tensor:
    """A matrix state read before it is written, with a bonus for the current token, per sequence and head.

    ``r`` / ``k`` [T, H, d], ``v`` [T, H, dv] in the activation dtype (strided views allowed), ``g`` f32 [T, H, d] the
    decays per key channel, ``u`` f32 [H, d]:

        o = (S + diag(u) k v^T)^T r;   S <- diag(g) S + k v^T

    ``state`` f32 [slots, H, d, dv] as in ``channel_delta_scan``.  Returns o f32 [T, H, dv]."""
    T, H, d = r.shape
    if native(r):
        if d > SCAN_MAX_DIM:
            raise ValueError(f"bonus_scan: key size {d} is above the kernel's {SCAN_MAX_DIM}")
        return _ops().cx_bonus_scan(r, k, v, g.contiguous(), u, state, cu, state_slots, pos, q_lens, CHUNK_MIN)
    out = torch.empty(T, H, v.shape[2], dtype=torch.float32, device=r.device)
    rf, kf, vf = r.float(), k.float(), v.float()
    bonus = (u[None] * kf * rf).sum(-1)
    for t0, n, slot, fresh in _sequences(q_lens, state_slots, pos):
        S = torch.zeros_like(state[slot]) if fresh else state[slot].clone()
        for t in range(t0, t0 + n):
            out[t] = (S * rf[t][:, :, None]).sum(1) + bonus[t][:, None] * vf[t]
            S = g[t][:, :, None] * S + kf[t][:, :, None] * vf[t][:, None, :]
        state[slot] = S
    return out
