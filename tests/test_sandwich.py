"""Decoders whose sublayers are normed before and after (Sudosun layout): the
framework -- checkpoint reader, paged rows and state slots, scheduler, ragged
engine steps, kernels -- against the plain float64 forms of
tests/sandwich_oracle.py.

Every test runs on the CPU (torch forms of ops/statemix.py, ops/maskattn.py,
...) and, marked ``gpu``, on the HIP kernels.  Models are small random ones
made here.
"""
import json
import math
import os
import subprocess
import sys

import pytest
import torch

from . import sandwich_oracle as O

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
DEVS = ["cpu", pytest.param("cuda", marks=pytest.mark.gpu)]
F64 = torch.float64
TOL = {torch.float32: 2e-4, torch.bfloat16: 0.12}


@pytest.fixture(params=DEVS)
def dev(request):
    if request.param == "cuda":
        if not torch.cuda.is_available():
            pytest.skip("no GPU")
        import ipex_llm_amd.ops as ops
        ops.require_seqmix()
    return torch.device(request.param)


def std_cfg():
    """all three mixers, dense and routed feed-forwards and a layer without one; windows shorter than a page and one
    that straddles pages; value sizes that differ from key sizes"""
    return O.config([O.pair_layer(heads=4, kv_heads=2, dim=12, vdim=10, window=9, dims=8, width=24, blocks=3, taps=2,
                                  mlp=O.dense_ff(20, 0.8)),
                     O.delta_layer(heads=4, kv_heads=2, dim=12, vdim=10, taps=3, mlp=O.moe(5, 1, 2, 12, (3, 2))),
                     O.lightning_layer(heads=3, dim=6, vdim=10, mlp=O.moe(4, 2, 3, 8, (2, 1))),
                     O.pair_layer(heads=2, kv_heads=1, dim=16, vdim=24, window=70, dims=16, scaling=None, width=70, blocks=2,
                                  taps=4),
                     O.delta_layer(heads=3, kv_heads=3, dim=20, vdim=70, taps=1, mlp=O.dense_ff(24, 2.0))], width=40)


def build(cfg, W, dev, dtype=torch.float32):
    from ipex_llm_amd.models import sudosun as S
    return S.build(S.spec_from_config(cfg), W, dtype, dev)


def engine(cfg, W, dev, dtype=torch.float32, max_batch=4, num_blocks=16, prefill=1 << 30, graph=False):
    from ipex_llm_amd.serving.engine import LLMEngine
    return LLMEngine(build(cfg, W, dev, dtype), max_batch=max_batch, block_size=64, num_blocks=num_blocks,
                     max_model_len=num_blocks * 64, max_prefill_tokens=prefill, use_graph=graph,
                     enable_prefix_caching=False)


def replay(eng, prompts, schedule, keep_open=()):
    """schedule: steps of [(name, count)]; every token's logits are asked for.
    Returns name -> [T, V] (f64, on the CPU) of what was run."""
    at, rid, got = {}, {}, {}
    for step in schedule:
        entries = []
        for name, n in step:
            lo = at.get(name, 0)
            if name not in rid:
                rid[name] = eng.open_stream()
            entries.append((rid[name], prompts[name][lo:lo + n], list(range(n))))
            at[name] = lo + n
        lg = eng.feed(entries).double().cpu()
        o = 0
        for name, n in step:
            got.setdefault(name, []).append(lg[o:o + n])
            o += n
            if at[name] == len(prompts[name]) and name not in keep_open:
                eng.close_stream(rid.pop(name))
    return {k: torch.cat(v) for k, v in got.items()}


def rel_err(got, want):
    """largest row error: rms over the vocabulary of the centred difference, over the logits' spread"""
    d = got - want
    d = d - d.mean(-1, keepdim=True)
    return float((d.pow(2).mean(-1).sqrt() / want.std()).max())


def ragged(lens, starts, dev, slots=None):
    """cu, seq_of, state slots, positions of a step whose sequence s brings lens[s] tokens from position starts[s]"""
    cu = torch.tensor([0] + list(torch.tensor(lens).cumsum(0)), dtype=torch.int32, device=dev)
    seq_of = torch.cat([torch.full((n,), s, dtype=torch.int32) for s, n in enumerate(lens)]).to(dev)
    pos = torch.cat([torch.arange(a, a + n) for a, n in zip(starts, lens)]).to(dev)
    slots = slots if slots is not None else range(1, 1 + len(lens))
    return cu, seq_of, torch.tensor(list(slots), dtype=torch.int32, device=dev), pos


def in_portions(f, seqs, cuts, dev):
    """run ``f(rows of the step, lens, cu, seq_of, slots, pos)`` over ``seqs`` (a list of [n_s, ...] inputs) cut into
    the steps ``cuts`` (per step the tokens every sequence brings, 0: it sits the step out); returns per sequence
    the concatenated results"""
    at = [0] * len(seqs)
    outs = [[] for _ in seqs]
    for step in cuts:
        who = [s for s, n in enumerate(step) if n]
        lens = [step[s] for s in who]
        cu, seq_of, slots, pos = ragged(lens, [at[s] for s in who], dev, [s + 1 for s in who])
        rows = torch.cat([seqs[s][at[s]:at[s] + step[s]] for s in who]).to(dev)
        res = f(rows, lens, cu, seq_of, slots, pos)
        o = 0
        for s, n in zip(who, lens):
            outs[s].append(res[o:o + n].double().cpu())
            o += n
            at[s] += n
    return [torch.cat(o) for o in outs]


CUTS = [[5, 1, 0], [1, 1, 70], [2, 60, 1], [64, 2, 1], [1, 0, 3]]     # three sequences, 73 / 64 / 75 tokens


# ------------------------------------------------------------------ mechanisms alone (ops)
def rand_norm(Wd, g):
    return torch.tensor([0.7]), 1 + 0.3 * torch.randn(Wd, generator=g), 0.3 * torch.randn(Wd, generator=g)


@pytest.mark.parametrize("act", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("Wd", [5, 37, 40, 1100, 4160])
def test_residual_and_norms(dev, act, Wd):
    """the first norm alone; a sublayer's result normed, added and normed again, for each of the three sources"""
    from ipex_llm_amd.ops import statemix as SX
    g = torch.Generator().manual_seed(Wd)
    T, top, E = 7, 3, 4
    tol = 2e-5 if act == torch.float32 else 3e-2
    x0 = torch.randn(T, Wd, generator=g) * 2
    post, pre = rand_norm(Wd, g), rand_norm(Wd, g)

    def dt(n, v):
        return O.dyn_tanh(v, *(t.double() for t in n))

    def on(n):
        return tuple(t.to(dev) for t in n)
    got = SX.dyn_tanh(x0.to(dev), on(pre), act)
    assert got.dtype == act and (got.double().cpu() - dt(pre, x0.double())).abs().max() < tol
    y = (torch.randn(T, Wd, generator=g) * 2).to(act)
    y32 = torch.randn(T, Wd, generator=g)
    a, b = (torch.randn(T, Wd, generator=g) * 3).to(act), torch.randn(T, Wd, generator=g).to(act)
    wa, wb = (1 + 0.2 * torch.randn(Wd, generator=g)).to(act), (1 + 0.2 * torch.randn(Wd, generator=g)).to(act)
    rows = torch.randn(T, top, Wd, generator=g)
    idx = torch.randint(0, E + 2, (T, top), generator=g).to(torch.int32)
    wts = torch.rand(T, top, generator=g)
    h = torch.randn(T, Wd, generator=g).to(act)
    esum = torch.zeros(T, Wd, dtype=F64)
    for t in range(T):
        for k in range(top):
            esum[t] += rows[t, k].double() if idx[t, k] < E else wts[t, k].double() * h[t].double()
    pair = 0.5 * (O.unit_rms(a.double(), 1e-5) * wa.double() + O.unit_rms(b.double(), 1e-5) * wb.double())
    for src, want in ((y.to(dev), y.double()), (y32.to(dev), y32.double()),
                      (SX.PairMean(a.to(dev), b.to(dev), wa.to(dev), wb.to(dev), 1e-5), pair),
                      (SX.ExpertSum(rows.to(dev), idx.to(dev), wts.to(dev), h.to(dev), E), esum)):
        for second in (pre, None):
            x = x0.clone().to(dev)
            got = SX.add_normed_(x, src, on(post), on(second) if second else None, act)
            xn = x0.double() + dt(post, want)
            assert (x.double().cpu() - xn).abs().max() < 2e-5
            if second is None:
                assert got is None
            else:
                assert got.dtype == act and (got.double().cpu() - dt(pre, xn)).abs().max() < tol


@pytest.mark.parametrize("act", [torch.float32, torch.bfloat16])
def test_row_norm_with_sigmoid_gate(dev, act):
    from ipex_llm_amd.ops import statemix as SX
    g = torch.Generator().manual_seed(1)
    tol = 2e-5 if act == torch.float32 else 5e-2
    for T, C in ((6, 30), (3, 1030), (70, 4100), (2, 1)):
        o = torch.randn(T, C, generator=g) * 3
        w = (1 + 0.2 * torch.randn(C, generator=g)).to(act)
        gate = torch.randn(T, C + 9, generator=g).to(act)
        got = SX.rms_sigmoid_gate(o.to(dev), w.to(dev), gate.to(dev)[:, 4:4 + C], 1e-5, act)
        want = O.unit_rms(o.double(), 1e-5) * w.double() * O.sigmoid(gate[:, 4:4 + C].double())
        assert got.dtype == act and (got.double().cpu() - want).abs().max() < tol


SCAN_SIZES = [(3, 6, 10), (2, 48, 64), (1, 70, 70), (2, 130, 8), (1, 1, 1), (1, 300, 20), (4, 64, 128), (2, 16, 17)]


@pytest.mark.parametrize("chunk_min", [0, 2])
@pytest.mark.parametrize("H,d,dv", SCAN_SIZES)
def test_decay_scan(dev, H, d, dv, chunk_min, monkeypatch):
    """a fixed decay per head (one near 1, one small); state carried over portions and batches, dirty slots; on the
    GPU token by token and in chunks"""
    from ipex_llm_amd.ops import statemix as SX
    monkeypatch.setattr(SX, "CHUNK_MIN", chunk_min)
    g = torch.Generator().manual_seed(H + d)
    decay = torch.tensor([0.999, 0.3, 0.9, 1.0][:H])
    for act in (torch.float32, torch.bfloat16):
        seqs = [torch.randn(n, 2 * H * d + H * dv + 4, generator=g).to(act) for n in (73, 64, 75)]
        state = torch.randn(5, H, d, dv, generator=g).to(dev)

        def split(rows):
            T = rows.shape[0]
            return (rows[:, 2:2 + H * d].view(T, H, d), rows[:, 2 + H * d:2 + 2 * H * d].view(T, H, d),
                    rows[:, 2 + 2 * H * d:2 + 2 * H * d + H * dv].view(T, H, dv))

        def f(rows, lens, cu, seq_of, slots, pos):
            o = SX.decay_scan(*split(rows), decay.to(dev), state, cu, slots, pos, lens)
            return o.reshape(rows.shape[0], -1)

        for x, o in zip(seqs, in_portions(f, seqs, CUTS, dev)):
            q, k, v = (O.silu(t.double()) for t in split(x))
            want = O.lightning_scan(q, k, v, decay.double().tolist()).reshape(x.shape[0], -1)
            assert (o - want).abs().max() < 2e-5 * max(1.0, float(want.abs().max()))


def delta_inputs(g, T, H, K, d, dv, act):
    q, k = torch.randn(T, K, d, generator=g), torch.randn(T, K, d, generator=g)
    v = torch.randn(T, H, dv, generator=g)
    ab = (torch.randn(T, 2 * H + 3, generator=g) * 1.5).to(act)
    return q, k, v, ab


def delta_want(q, k, v, ab, rate, bias, H):
    q, k, v, ab = (t.double() for t in (q, k, v, ab))
    g = torch.exp(-rate.double() * O.softplus(ab[:, 1:1 + H] + bias.double()))
    beta = O.sigmoid(ab[:, 2 + H:2 + 2 * H])
    return O.delta_scan(O.unit(q) * q.shape[2] ** -0.5, O.unit(k), v, g, beta)


@pytest.mark.parametrize("chunk_min", [0, 2])
@pytest.mark.parametrize("H,K,d,dv", [(4, 2, 6, 10), (2, 2, 48, 64), (1, 1, 70, 70), (6, 2, 130, 8), (1, 1, 1, 1),
                                      (2, 1, 300, 20), (4, 4, 64, 128), (3, 1, 16, 17)])
def test_delta_scan(dev, H, K, d, dv, chunk_min, monkeypatch):
    """the gated delta rule over portions and batches, key heads shared by several value heads, dirty slots; on the
    GPU token by token and in chunks"""
    from ipex_llm_amd.ops import statemix as SX
    monkeypatch.setattr(SX, "CHUNK_MIN", chunk_min)
    g = torch.Generator().manual_seed(H + d)
    rate, bias = torch.rand(H, generator=g), torch.randn(H, generator=g)
    for act in (torch.float32, torch.bfloat16):
        ins = [delta_inputs(g, n, H, K, d, dv, act) for n in (73, 64, 75)]
        seqs = [torch.cat([t.reshape(t.shape[0], -1).float() for t in i], 1) for i in ins]
        state = torch.randn(5, H, d, dv, generator=g).to(dev)

        def f(rows, lens, cu, seq_of, slots, pos):
            T, n = rows.shape[0], K * d
            u = rows[:, :2 * n + H * dv]
            ab = rows[:, 2 * n + H * dv:].to(act)
            o = SX.delta_scan(u[:, :n].view(T, K, d), u[:, n:2 * n].view(T, K, d), u[:, 2 * n:].view(T, H, dv),
                              ab[:, 1:1 + H], ab[:, 2 + H:2 + 2 * H], rate.to(dev), bias.to(dev), d ** -0.5, state, cu,
                              slots, pos, lens)
            return o.reshape(T, -1)

        for i, o in zip(ins, in_portions(f, seqs, CUTS, dev)):
            want = delta_want(*i, rate, bias, H).reshape(o.shape)
            assert (o - want).abs().max() < 2e-5 * max(1.0, float(want.abs().max()))


def test_long_portions_of_the_state_scans(dev):
    """portions of thousands of tokens (on the GPU: many chunks, more than one segment of them) beside short ones and
    one that continues; equal keys with steps near 1, and decays that all but clear the state now and then"""
    from ipex_llm_amd.ops import statemix as SX
    g = torch.Generator().manual_seed(6)
    H, d, dv = 1, 5, 3
    lens, starts = [8400, 1, 130, 64], [0, 9, 3, 0]
    T = sum(lens)
    cu, _, slots, pos = ragged(lens, starts, dev)
    q, k, v = torch.randn(T, H, d, generator=g), torch.randn(T, H, d, generator=g), torch.randn(T, H, dv, generator=g)
    k[100:300] = k[100]
    a, b = torch.randn(T, H, generator=g) - 4, torch.randn(T, H, generator=g)
    a[torch.arange(50, T, 97)] = 300.0
    b[100:200] = 9.0
    rate, bias, decay = torch.tensor([2.0]), torch.tensor([0.3]), torch.tensor([0.997])
    S0 = torch.randn(6, H, d, dv, generator=g)

    def check(got, state, step):
        t0 = 0
        for s, n in enumerate(lens):
            S = torch.zeros(H, d, dv, dtype=F64) if starts[s] == 0 else S0[s + 1].double()
            want = torch.empty(n, H, dv, dtype=F64)
            for t in range(n):
                S, want[t] = step(S, t0 + t)
            tol = 3e-5 * max(1.0, float(want.abs().max()))
            assert (got[t0:t0 + n].double().cpu() - want).abs().max() < tol, s
            assert (state[s + 1].double().cpu() - S).abs().max() < 3e-5 * max(1.0, float(S.abs().max())), s
            t0 += n

    state = S0.clone().to(dev)
    got = SX.decay_scan(q.to(dev), k.to(dev), v.to(dev), decay.to(dev), state, cu, slots, pos, lens)
    qs, ks, vs = O.silu(q.double()), O.silu(k.double()), O.silu(v.double())

    def light(S, t):
        S = decay.double() * S + ks[t][:, :, None] * vs[t][:, None, :]
        return S, (S * qs[t][:, :, None]).sum(1)
    check(got, state, light)
    state = S0.clone().to(dev)
    got = SX.delta_scan(q.to(dev), k.to(dev), v.to(dev), a.to(dev), b.to(dev), rate.to(dev), bias.to(dev), 0.5, state, cu,
                        slots, pos, lens)
    qu, ku = O.unit(q.double()) * 0.5, O.unit(k.double())
    gd = torch.exp(-2.0 * O.softplus(a.double() + bias.double()))
    be = O.sigmoid(b.double())

    def rule(S, t):
        S = gd[t][:, None, None] * S
        u = be[t][:, None] * (v[t].double() - (S * ku[t][:, :, None]).sum(1))
        S = S + ku[t][:, :, None] * u[:, None, :]
        return S, (S * qu[t][:, :, None]).sum(1)
    check(got, state, rule)


@pytest.mark.parametrize("nb,n", [(3, 8), (1, 5), (2, 35), (4, 64), (2, 136), (1, 1)])
def test_gates_of_the_linear_recurrent_unit(dev, nb, n):
    """block-diagonal gates, decays and inputs; 16-bit weights with f32 inputs keep f32 precision; slow decays (log a
    near 0) keep the input factor's relative precision"""
    from ipex_llm_amd.ops import statemix as SX
    g = torch.Generator().manual_seed(nb + n)
    C = nb * n
    lam = torch.randn(C, generator=g) * 3 - 4
    base = (-8.0 * O.softplus(lam.double())).float()
    for act in (torch.float32, torch.bfloat16):
        wr, wi = (torch.randn(nb, n, n, generator=g) * n ** -0.5).to(act), (torch.randn(nb, n, n, generator=g) * n ** -0.5).to(act)
        br, bi = torch.randn(C, generator=g), torch.randn(C, generator=g)
        for T in (1, 9, 150):
            u = torch.randn(T, C, generator=g) * 2
            a, x = SX.rglru_gates(u.to(dev), wr.to(dev), br.to(dev), wi.to(dev), bi.to(dev), base.to(dev))
            ub = u.double().view(T, nb, n)
            zr = torch.stack([ub[:, b] @ wr[b].double().T for b in range(nb)], 1).reshape(T, C) + br.double()
            zi = torch.stack([ub[:, b] @ wi[b].double().T for b in range(nb)], 1).reshape(T, C) + bi.double()
            la = O.sigmoid(zr) * base.double()
            want = torch.sqrt(-torch.expm1(2 * la)) * O.sigmoid(zi) * u.double()
            assert (a.double().cpu() - torch.exp(la)).abs().max() < 3e-6
            assert ((x.double().cpu() - want).abs() / (1e-3 + want.abs())).max() < 3e-5


@pytest.mark.parametrize("C", [5, 64, 200])
def test_scan_of_the_linear_recurrent_unit(dev, C):
    """over portions and batches, and long portions that the kernel cuts into pieces"""
    from ipex_llm_amd.ops import statemix as SX
    g = torch.Generator().manual_seed(C)
    for act in (torch.float32, torch.bfloat16):
        for lens, cuts in (((73, 64, 75), CUTS), ((700, 64, 1), [[300, 1, 0], [400, 63, 1]])):
            seqs = [torch.cat([torch.rand(n, C, generator=g), torch.randn(n, 2 * C, generator=g)], 1) for n in lens]
            for s in seqs:
                s[:, 2 * C:] = s[:, 2 * C:].to(act).float()
            state = torch.randn(5, C, generator=g).to(dev)

            def f(rows, ln, cu, seq_of, slots, pos):
                return SX.rglru_scan(rows[:, :C].contiguous(), rows[:, C:2 * C].contiguous(), rows[:, 2 * C:].to(act), state,
                                     cu, slots, pos, ln)

            for s, o in zip(seqs, in_portions(f, seqs, cuts, dev)):
                s = s.double()
                S, want = torch.zeros(C, dtype=F64), []
                for t in range(s.shape[0]):
                    S = s[t, :C] * S + s[t, C:2 * C]
                    want.append(S * O.gelu_tanh(s[t, 2 * C:]))
                want = torch.stack(want)
                assert ((o - want).abs() / (1 + want.abs())).max() < (2e-5 if act == torch.float32 else 1e-2)


@pytest.mark.parametrize("E,top,groups,keep", [(6, 2, 3, 2), (20, 4, 4, 3), (7, 7, 1, 1), (130, 5, 13, 2), (512, 8, 64, 4),
                                               (9, 3, 9, 4), (4, 1, 2, 1)])
def test_routing_in_groups(dev, E, top, groups, keep):
    """the choice goes by corrected scores, which may all be negative inside a kept group, the weights are the plain
    scores; ties to the lowest index; unkept groups never win even when a kept group's scores are lower"""
    from ipex_llm_amd.ops import statemix as SX
    g = torch.Generator().manual_seed(E)
    z = torch.randn(40, E, generator=g) * 2
    corr = torch.randn(E, generator=g) * 0.1 - 0.3
    zt = torch.zeros(2, E)
    for zz, cc in ((z, corr), (z, None), (zt, torch.zeros(E))):
        idx, w = SX.route_groups(zz.to(dev), cc.to(dev) if cc is not None else None, top, groups, keep)
        assert idx.dtype == torch.int32
        for t in range(zz.shape[0]):
            want = O.route(zz[t].double(), cc.double() if cc is not None else torch.zeros(E, dtype=F64), top,
                           {"count": groups, "keep": keep})
            assert idx[t].tolist() == [e for e, _ in want]
            assert (w[t].double().cpu() - torch.stack([s for _, s in want])).abs().max() < 1e-6


@pytest.mark.parametrize("act", [torch.float32, torch.bfloat16])
def test_router_logits_and_choice(dev, act):
    """few tokens (on the GPU one launch) and many (a product, then the choice)"""
    from ipex_llm_amd.ops import statemix as SX
    g = torch.Generator().manual_seed(9)
    for T, Wd, E, top, groups, keep in ((3, 37, 6, 2, 3, 2), (64, 40, 20, 4, 4, 3), (65, 40, 20, 4, 4, 3), (1, 300, 33, 1, 1, 1)):
        h = torch.randn(T, Wd, generator=g).to(act)
        rw, corr = torch.randn(E, Wd, generator=g), 0.1 * torch.randn(E, generator=g)
        idx, w = SX.route(h.to(dev), rw.to(dev), corr.to(dev), top, groups, keep)
        z = h.double() @ rw.double().T
        for t in range(T):
            want = O.route(z[t], corr.double(), top, {"count": groups, "keep": keep})
            assert idx[t].tolist() == [e for e, _ in want]
            assert (w[t].double().cpu() - torch.stack([s for _, s in want])).abs().max() < 1e-5


def test_group_choice_shows(dev):
    """two groups: the best score decides the group, the second best score of all sits in the other group and loses"""
    from ipex_llm_amd.ops import statemix as SX
    z = torch.tensor([[3.0, 2.9, -5.0, 0.0, 3.1, -6.0]])
    idx, _ = SX.route_groups(z.to(dev), None, 2, 2, 1)
    assert idx.tolist() == [[4, 3]]
    corr = torch.tensor([0.0, -2.0, -2.0, -2.0, -2.0, -2.0])          # every choice score but one negative
    idx, w = SX.route_groups(z.to(dev), corr.to(dev), 3, 2, 1)
    assert idx.tolist() == [[0, 1, 2]]
    assert (w.cpu() - torch.softmax(z, -1)[:, :3]).abs().max() < 1e-6


@pytest.mark.parametrize("E,ident,top,ff,Wd,T", [(5, 1, 2, 12, 40, 9), (11, 3, 3, 88, 64, 150), (3, 0, 3, 8, 24, 4),
                                                 (2, 6, 4, 8, 16, 33), (1, 1, 1, 5, 9, 3)])
def test_experts_and_identity_experts(dev, E, ident, top, ff, Wd, T):
    """weights on the experts' results, identity experts add their weight times the input; tokens whose experts are all
    identity experts"""
    from ipex_llm_amd.models.hybrid import ExpertSpec, MoESpec, ScoredMoE
    g = torch.Generator().manual_seed(E + T)
    for act in (torch.float32, torch.bfloat16):
        W = {"router": torch.randn(E + ident, Wd, generator=g), "correction": 0.1 * torch.randn(E + ident, generator=g)}
        if ident >= top:
            W["correction"][E:] += 2.0                                 # only identity experts win
        for e in range(E):
            W.update({f"e{e}.gate": torch.randn(ff, Wd, generator=g) * Wd ** -0.5,
                      f"e{e}.up": torch.randn(ff, Wd, generator=g) * Wd ** -0.5,
                      f"e{e}.down": torch.randn(Wd, ff, generator=g) * ff ** -0.5})
        W = {k: v.to(act) for k, v in W.items()}
        h = torch.randn(T, Wd, generator=g).to(act)
        moe = ScoredMoE(MoESpec(E, top, ExpertSpec(ff), identity=ident), W["router"], W["correction"],
                        torch.stack([torch.cat([W[f"e{e}.gate"], W[f"e{e}.up"]]) for e in range(E)]),
                        torch.stack([W[f"e{e}.down"] for e in range(E)])).to(dev)
        got = moe(h.to(dev))[0].double().cpu()
        cfg = {"router": {"experts": E, "top": top}}
        want = O.experts({k: v.double() for k, v in W.items()}, "", cfg, h.double())
        assert (got - want).abs().max() < (1e-4 if act == torch.float32 else 8e-2)


def test_clamped_feed_forward(dev):
    """gate clamped from above only, up on both sides"""
    from ipex_llm_amd.models.hybrid import DenseFF
    g = torch.Generator().manual_seed(3)
    W = {n: torch.randn(s, generator=g) for n, s in (("gate", (20, 12)), ("up", (20, 12)), ("down", (12, 20)))}
    h = torch.randn(9, 12, generator=g)
    for limit in (0.5, 3.0, 1e9):
        ff = DenseFF(W["gate"], W["up"], W["down"], act="clamp", limit=limit).to(dev)
        want = O.dense({k: v.double() for k, v in W.items()}, "", {"limit": limit}, h.double())
        assert (ff(h.to(dev)).double().cpu() - want).abs().max() < 1e-4 * max(1.0, float(want.abs().max()))


@pytest.mark.parametrize("d,dv,dims", [(12, 10, 8), (16, 8, 6), (96, 24, 48), (128, 128, 128), (40, 16, 40), (8, 6, 2)])
@pytest.mark.parametrize("act", [torch.float32, torch.bfloat16])
def test_query_factor_and_head_gate(dev, act, d, dv, dims):
    from ipex_llm_amd.ops import maskattn as MA
    from ipex_llm_amd.ops.seqmix import rope_table
    g = torch.Generator().manual_seed(4)
    T, H, G = 11, 6, 2
    y = torch.randn(T, H * d + G * (d + dv), generator=g).to(act)
    q, k, v = y[:, :H * d].view(T, H, d), y[:, H * d:(H + G) * d].view(T, G, d), y[:, (H + G) * d:].view(T, G, dv)
    qn, kn = (1 + 0.3 * torch.randn(d, generator=g)).to(act), (1 + 0.3 * torch.randn(d, generator=g)).to(act)
    temp = torch.rand(H, generator=g) + 0.5
    rot = {"dims": dims, "base": 3000.0, "scaling": O.YARN}
    tab = rope_table(64, dims, 3000.0, O.YARN)
    pos = torch.arange(20, 20 + T)
    rows = torch.zeros(2, 64, G * (d + dv), dtype=act, device=dev)
    yd = y.to(dev)
    got = MA.qkv_norm_rope_store(yd[:, :H * d].view(T, H, d), yd[:, H * d:(H + G) * d].view(T, G, d),
                                 yd[:, (H + G) * d:].view(T, G, dv), qn.to(dev), kn.to(dev), False, 1e-5, tab.to(dev), "pairs",
                                 pos.to(dev), (pos + 30).to(dev), rows, temp=temp.to(dev)).double().cpu()
    want = O.turn_pairs(O.unit_rms(q.double(), 1e-5) * qn.double(), rot, pos) * temp.double()[:, None]
    assert (got - want).abs().max() < 2e-5
    keys = O.turn_pairs(O.unit_rms(k.double(), 1e-5) * kn.double(), rot, pos).reshape(T, -1)
    stored = rows.view(128, -1)[50:50 + T].double().cpu()
    tol = 2e-5 if act == torch.float32 else 3e-2
    assert (stored[:, :G * d] - keys).abs().max() < tol and (stored[:, G * d:] - v.double().reshape(T, -1)).abs().max() < tol
    o = torch.randn(T, H * dv, generator=g).to(act)
    gate = torch.randn(T, H + 5, generator=g).to(act)
    got = MA.sigmoid_gate(o.clone().to(dev), gate.to(dev)[:, 2:2 + H]).double().cpu()
    want = (o.double().view(T, H, dv) * O.sigmoid(gate[:, 2:2 + H].double())[..., None]).reshape(T, -1)
    assert (got - want).abs().max() < tol


def test_yarn_frequencies(dev):
    """kept, slowed and blended pairs all present; the magnitude applies to the rotated values only"""
    from ipex_llm_amd.ops.seqmix import rope_table
    rot = {"dims": 16, "base": 3000.0, "scaling": {"factor": 4.0, "original": 64, "fast": 8.0, "slow": 1.0}}
    f, mag = O.rotary(rot)
    plain = O.rotary({"dims": 16, "base": 3000.0})[0]
    kinds = {("kept" if a == b else ("slowed" if abs(a - b / 4) < 1e-15 else "blend")) for a, b in zip(f.tolist(), plain.tolist())}
    assert kinds == {"kept", "slowed", "blend"}
    tab = rope_table(50, 16, 3000.0, rot["scaling"]).double()
    ang = torch.arange(50, dtype=F64)[:, None] * f[None]
    assert (tab[..., 0] - ang.cos() * mag).abs().max() < 1e-6 and (tab[..., 1] - ang.sin() * mag).abs().max() < 1e-6


# ------------------------------------------------------------------ whole models
_want = {}


def oracle(cfg, W, toks, key):
    if key not in _want:
        _want[key] = O.forward(cfg, W, toks)
    return _want[key]


LAYER_CASES = [
    [O.lightning_layer(heads=3, dim=6, vdim=10, mlp=O.dense_ff(20, 0.8))],
    [O.lightning_layer(heads=1, dim=1, vdim=1), O.lightning_layer(heads=2, dim=17, vdim=70, decay=[1.0, 0.5], mlp=O.moe(1, 0, 1, 8, None))],
    [O.delta_layer(heads=4, kv_heads=2, dim=12, vdim=10, taps=3, mlp=O.moe(4, 2, 4, 8, (3, 2)))],
    [O.delta_layer(heads=1, kv_heads=1, dim=1, vdim=1, taps=1), O.delta_layer(heads=6, kv_heads=1, dim=9, vdim=5, taps=5, mlp=O.dense_ff(7, 0.1))],
    [O.pair_layer(mlp=O.moe(3, 1, 2, 8, (2, 2)))],
    [O.pair_layer(heads=2, kv_heads=1, dim=16, vdim=8, window=1, dims=16, width=4, blocks=4, taps=1)],
    [O.pair_layer(heads=3, kv_heads=3, dim=6, vdim=6, window=64, dims=2, scaling=None, width=35, blocks=1, taps=5, scale=1.0)],
    [O.pair_layer(heads=8, kv_heads=1, dim=10, vdim=20, window=65, dims=4, width=18, blocks=2, taps=3,
                  scaling={"factor": 1.0, "original": 32, "fast": 4.0, "slow": 1.0}), O.lightning_layer(mlp=O.dense_ff(3, 5.0))],
]


@pytest.mark.parametrize("case", range(len(LAYER_CASES)))
def test_small_models(dev, case):
    """each mixer alone and in pairs, sizes that are 1 or equal to each other, layers without a feed-forward"""
    cfg = O.config(LAYER_CASES[case], width=24 + 2 * case, eps=[1e-5, 1e-3][case % 2], logit_scale=1.0 if case == 2 else 0.4)
    W = O.random_weights(cfg, case)
    toks = O.random_tokens(cfg, 75, case)
    want = O.forward(cfg, W, toks)
    got = replay(engine(cfg, W, dev), {"a": toks}, [[("a", 40)], [("a", 30)]] + [[("a", 1)]] * 5)["a"]
    assert rel_err(got, want) < TOL[torch.float32]
    got = replay(engine(cfg, W, dev, torch.bfloat16), {"a": toks}, [[("a", 70)], [("a", 3)]] + [[("a", 1)]] * 2)["a"]
    # 16-bit: rows of 1 to 40 values average little rounding away
    assert rel_err(got, want) < 0.25


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_odd_sizes(dev, dtype):
    """widths, head sizes, expert sizes and vocabulary that are multiples of nothing"""
    cfg = O.config([O.pair_layer(heads=3, kv_heads=1, dim=9, vdim=7, window=5, dims=4, width=33, blocks=3, taps=3,
                                 mlp=O.moe(5, 2, 3, 5, (7, 4))),
                    O.delta_layer(heads=3, kv_heads=1, dim=7, vdim=5, taps=2, mlp=O.moe(2, 1, 1, 7, (3, 1))),
                    O.lightning_layer(heads=5, dim=3, vdim=7, mlp=O.dense_ff(11, 0.6))], vocab=53, width=37)
    W = O.random_weights(cfg, 31)
    toks = O.random_tokens(cfg, 70, 31)
    got = replay(engine(cfg, W, dev, dtype), {"a": toks}, [[("a", 33)], [("a", 30)]] + [[("a", 1)]] * 7)["a"]
    assert rel_err(got, O.forward(cfg, W, toks)) < (TOL[dtype] if dtype == torch.float32 else 0.2)


def test_whole_prompt_and_layers(dev):
    cfg = std_cfg()
    W = O.random_weights(cfg, 7)
    toks = O.random_tokens(cfg, 141, 7)
    eng = engine(cfg, W, dev)
    eng.model.capture_layers = []
    got = replay(eng, {"a": toks}, [[("a", 141)]])["a"]
    layers = []
    want = O.forward(cfg, W, toks, layers_out=layers)
    assert rel_err(got, want) < TOL[torch.float32]
    assert len(eng.model.capture_layers) == len(layers)
    for a, b in zip(eng.model.capture_layers, layers):
        assert (a.double().cpu() - b).abs().max() < 1e-4 * float(b.abs().max())


def test_first_tokens(dev):
    """sequences of one to four tokens (shorter than the convolutions), each whole and decoded one by one"""
    cfg = std_cfg()
    W = O.random_weights(cfg, 8)
    for n in (1, 2, 3, 4):
        toks = O.random_tokens(cfg, n, n)
        want = O.forward(cfg, W, toks)
        assert rel_err(replay(engine(cfg, W, dev), {"a": toks}, [[("a", n)]])["a"], want) < TOL[torch.float32]
        assert rel_err(replay(engine(cfg, W, dev), {"a": toks}, [[("a", 1)]] * n)["a"], want) < TOL[torch.float32]


def test_prefill_equals_token_by_token(dev):
    cfg = std_cfg()
    W = O.random_weights(cfg, 9)
    toks = O.random_tokens(cfg, 80, 9)
    want = O.forward(cfg, W, toks)
    assert rel_err(replay(engine(cfg, W, dev), {"a": toks}, [[("a", 1)]] * 80)["a"], want) < TOL[torch.float32]
    assert rel_err(replay(engine(cfg, W, dev), {"a": toks}, [[("a", 80)]])["a"], want) < TOL[torch.float32]


@pytest.mark.parametrize("sizes", [[2] * 40, [63, 2, 64, 1, 3, 65], [5, 59, 1, 1, 62, 2, 70], [130, 2, 2, 66]])
def test_portions(dev, sizes):
    cfg = std_cfg()
    W = O.random_weights(cfg, 10)
    toks = O.random_tokens(cfg, 200, 10)
    got = replay(engine(cfg, W, dev), {"a": toks[:sum(sizes)]}, [[("a", n)] for n in sizes])["a"]
    assert rel_err(got, oracle(cfg, W, toks, "p10")[:sum(sizes)]) < TOL[torch.float32]


def test_unequal_batch_equals_each_alone(dev):
    cfg = std_cfg()
    W = O.random_weights(cfg, 11)
    P = {"a": O.random_tokens(cfg, 100, 1), "b": O.random_tokens(cfg, 9, 2), "c": O.random_tokens(cfg, 67, 3),
         "d": O.random_tokens(cfg, 30, 4)}
    schedule = [[("a", 50), ("b", 1)], [("a", 14), ("b", 1), ("c", 64), ("d", 2)], [("a", 1), ("b", 2), ("c", 2), ("d", 27)],
                [("a", 35), ("b", 5), ("c", 1), ("d", 1)]]
    got = replay(engine(cfg, W, dev), P, schedule)
    for name, toks in P.items():
        assert rel_err(got[name], oracle(cfg, W, toks, "b11" + name)) < TOL[torch.float32], name


def test_pages_and_slots_used_again(dev):
    """a pool of three pages and two slots serves five requests one after another and side by side"""
    cfg = std_cfg()
    W = O.random_weights(cfg, 12)
    P = {n: O.random_tokens(cfg, ln, i) for i, (n, ln) in enumerate([("a", 100), ("b", 60), ("c", 120), ("d", 3), ("e", 64)])}
    schedule = [[("a", 100)], [("b", 30)], [("b", 30)], [("c", 64), ("d", 1)], [("c", 56), ("d", 2)], [("e", 2)], [("e", 62)]]
    eng = engine(cfg, W, dev, max_batch=2, num_blocks=3)
    got = replay(eng, P, schedule)
    for name, toks in P.items():
        assert rel_err(got[name], oracle(cfg, W, toks, "s12" + name)) < TOL[torch.float32], name
    assert int(eng.sched.num_free_blocks()) == 3 and int(eng.sched.num_free_slots()) == 2


def test_long_decoding(dev):
    """decoded tokens walk over several windows and pages"""
    cfg = std_cfg()
    W = O.random_weights(cfg, 13)
    toks = O.random_tokens(cfg, 220, 13)
    got = replay(engine(cfg, W, dev), {"a": toks}, [[("a", 60)]] + [[("a", 1)]] * 160)["a"]
    assert rel_err(got, O.forward(cfg, W, toks)) < TOL[torch.float32]


def test_bfloat16_serving_precision(dev):
    cfg = std_cfg()
    W = O.random_weights(cfg, 14)
    toks = O.random_tokens(cfg, 90, 14)
    got = replay(engine(cfg, W, dev, torch.bfloat16), {"a": toks}, [[("a", 73)], [("a", 2)]] + [[("a", 1)]] * 15)["a"]
    assert rel_err(got, O.forward(cfg, W, toks)) < TOL[torch.bfloat16]


def edge_model(window, where):
    """one attention layer whose keys follow the token's embedding: a marked token's key towers over the others for
    every query, so its value shows in every position that sees it"""
    cfg = O.config([O.pair_layer(heads=2, kv_heads=1, dim=8, vdim=6, window=window, dims=2, scaling=None, width=6, blocks=2,
                                 taps=2, scale=1.0)], vocab=12, width=16)
    W = O.random_weights(cfg, 40)
    p = "l0.mix.left."
    W["embed"][:, 0] = 0.0
    W["embed"][11] *= 0.2
    W["embed"][11, 0] = 6.0                                            # the marked token: coordinate 0
    W["l0.norm1"][0], W["l0.norm1.b"][0] = 1.0, 0.0
    for n in ("q", "k"):
        W[p + n].zero_()
        W[p + n + ".b"].zero_()
    W[p + "q.b"][7::8] = 1.0                                           # queries: the same unrotated direction everywhere
    W[p + "k.b"][6] = 0.5
    W[p + "k"][7, 0] = 8.0                                             # the marked token's key points there
    W[p + "q.norm"].fill_(2.0)
    W[p + "k.norm"].fill_(2.0)
    W[p + "sink"].fill_(-1.0)
    return cfg, W


@pytest.mark.parametrize("window", [70, 64, 33, 1, 2])
@pytest.mark.parametrize("where", [0, 5, 63, 64])
def test_a_key_just_inside_and_just_outside(dev, window, where):
    """the marked token at position ``where``: the last position whose window holds it and the first that does not,
    as tokens of a prompt and decoded one by one; with the mark replaced the logits change inside and not outside
    (up to the short convolution's and the recurrence's own memory, which the plain form has as well)"""
    cfg, W = edge_model(window, where)
    n = where + window + 3
    toks = [1 + (i * 7) % 10 for i in range(n)]
    toks[where] = 11
    want = O.forward(cfg, W, toks)
    last = where + window - 1
    no_key = {k: v.clone() for k, v in W.items()}
    no_key["l0.mix.left.k"].zero_()
    blind = O.forward(cfg, no_key, toks)                               # what it would be if the key did not stand out
    if window > 2:
        assert (want[last] - blind[last]).abs().max() > 20 * (want[last + 1] - blind[last + 1]).abs().max()
    for schedule in ([[("a", n)]], [[("a", max(last - 1, 1))]] + [[("a", 1)]] * (n - max(last - 1, 1))):
        got = replay(engine(cfg, W, dev), {"a": toks}, schedule)["a"]
        assert (got - want).abs().max() < 2e-4 * float(want.abs().max())


def test_sink_factor_and_gate_show(dev):
    """leaving out the sink, a head's score factor or a head's gate changes the plain form's logits by far more than
    the framework differs from it"""
    cfg = O.config([O.pair_layer(scale=1.0)], width=24)
    W = O.random_weights(cfg, 41)
    W["l0.mix.left.sink"] += 1.5
    W["l0.mix.left.temp"] *= 2.5
    toks = O.random_tokens(cfg, 50, 41)
    want = O.forward(cfg, W, toks)
    got = replay(engine(cfg, W, dev), {"a": toks}, [[("a", 45)]] + [[("a", 1)]] * 5)["a"]
    err = (got - want).abs().max()
    for name, value in (("sink", -60.0), ("temp", 1.0), ("g", 0.0)):
        other = {k: v.clone() for k, v in W.items()}
        other["l0.mix.left." + name].fill_(value)
        assert (O.forward(cfg, other, toks) - want).abs().max() > 200 * err, name


@pytest.mark.parametrize("kind", ["lightning", "delta", "lru"])
def test_a_far_token_reaches_through_the_state(dev, kind):
    """changing the first token changes the logits hundreds of tokens later through the recurrent state alone; the
    framework follows the plain form on both prompts, over a prompt, a portion and decoded tokens"""
    layer = {"lightning": O.lightning_layer(heads=2, dim=6, vdim=8, decay=[0.9995, 0.5]), "delta": O.delta_layer(heads=2, kv_heads=1, taps=2),
             "lru": O.pair_layer(window=8)}[kind]
    cfg = O.config([layer], width=24)
    W = O.random_weights(cfg, 16)
    if kind == "delta":
        W["l0.mix.A_log"].fill_(-8.0)
        W["l0.mix.b"].zero_()
        W["l0.mix.b"][:, 0] = -6.0                                     # small steps: old content is hardly overwritten
        W["embed"][:, 0] = 2.0
    if kind == "lru":
        W["l0.mix.right.lam"].fill_(-9.0)
    a = O.random_tokens(cfg, 300, 16)
    b = [(a[0] + 1) % cfg["vocab"]] + a[1:]
    wa, wb = O.forward(cfg, W, a)[-1], O.forward(cfg, W, b)[-1]
    assert (wa - wb).abs().max() > 1e-3
    for toks, want in ((a, wa), (b, wb)):
        got = replay(engine(cfg, W, dev), {"a": toks}, [[("a", 170)], [("a", 120)]] + [[("a", 1)]] * 10)["a"][-1]
        assert (got - want).abs().max() < 0.05 * float((wa - wb).abs().max())


@pytest.mark.parametrize("window,sizes", [(100, [50, 390, 10]), (300, [300, 150]), (64, [5, 445])])
def test_long_windows_take_the_product_path(dev, window, sizes, monkeypatch):
    """portions long enough for the block-by-block product path of a sliding window on the GPU (its threshold and
    block lowered to this test's lengths), with a learned sink and score factors"""
    from ipex_llm_amd.ops import maskattn as MA
    monkeypatch.setattr(MA, "WINDOW_GEMM_MIN", 128)
    monkeypatch.setattr(MA, "WINDOW_Q_BLOCK", 160)
    cfg = O.config([O.pair_layer(heads=4, kv_heads=2, dim=16, vdim=24, window=window, dims=8, mlp=O.dense_ff(16))], width=32)
    W = O.random_weights(cfg, 17)
    toks = O.random_tokens(cfg, 450, 17)
    want = oracle(cfg, W, toks, f"w{window}")
    for dtype in (torch.float32, torch.bfloat16):
        got = replay(engine(cfg, W, dev, dtype), {"a": toks}, [[("a", n)] for n in sizes])["a"]
        assert rel_err(got, want) < TOL[dtype]


def test_mixed_steps_at_matrix_core_sizes(dev):
    """sizes that fill matrix-core tiles and ones that do not, long portions beside decoded tokens, both number formats"""
    cfg = O.config([O.pair_layer(heads=4, kv_heads=2, dim=40, vdim=56, window=50, dims=20, width=144, blocks=3, taps=4,
                                 mlp=O.moe(8, 4, 4, 40, (4, 3))),
                    O.delta_layer(heads=4, kv_heads=2, dim=80, vdim=48, taps=4, mlp=O.dense_ff(96, 1.5)),
                    O.lightning_layer(heads=2, dim=100, vdim=36, decay=[0.99, 0.7], mlp=O.moe(6, 2, 2, 64, (2, 1)))],
                   vocab=120, width=96)
    W = O.random_weights(cfg, 18)
    P = {"a": O.random_tokens(cfg, 260, 1), "b": O.random_tokens(cfg, 90, 2), "c": O.random_tokens(cfg, 150, 3)}
    schedule = [[("a", 100), ("b", 1)], [("a", 1), ("b", 2), ("c", 130)], [("a", 65), ("b", 86)],
                [("a", 92), ("b", 1), ("c", 19)], [("a", 1)], [("a", 1), ("c", 1)]]
    for dtype in (torch.float32, torch.bfloat16):
        got = replay(engine(cfg, W, dev, dtype), P, schedule)
        for name, toks in P.items():
            # 16-bit: the worst of hundreds of rows, a router's close calls among them
            assert rel_err(got[name], oracle(cfg, W, toks, "m18" + name)) < (TOL[dtype] if dtype == torch.float32 else 0.3), name


def test_greedy_generation_scheduler(dev):
    """LLMEngine.generate: C++ scheduler, chunked prompts (7 tokens a step in all), requests of unequal
    length side by side, greedy sampling"""
    from ipex_llm_amd.serving.engine import SamplingParams
    cfg = std_cfg()
    W = O.random_weights(cfg, 19)
    prompts = [O.random_tokens(cfg, n, 20 + n) for n in (23, 3, 70, 11)]
    want = [O.greedy(cfg, W, p, 6) for p in prompts]
    for prefill, batch, graph in ((7, 4, False), (1 << 30, 2, True)):
        eng = engine(cfg, W, dev, max_batch=batch, num_blocks=8, prefill=prefill, graph=graph)
        got = eng.generate(prompts, SamplingParams(max_new_tokens=6))
        assert got == want
        assert int(eng.sched.num_free_blocks()) == 8 and int(eng.sched.num_free_slots()) == batch


@pytest.mark.gpu
def test_decode_graph_replays_equal_eager():
    """pure-decode steps replayed from a captured graph (padded rows on the scratch page and slot), with eager
    prompt steps and synchronisations between the replays"""
    if not torch.cuda.is_available():
        pytest.skip("no GPU")
    cfg = std_cfg()
    W = O.random_weights(cfg, 21)
    P = {"a": O.random_tokens(cfg, 90, 1), "b": O.random_tokens(cfg, 40, 2), "c": O.random_tokens(cfg, 75, 3)}
    schedule = [[("a", 60), ("b", 20)]] + [[("a", 1), ("b", 1)]] * 10 + [[("c", 66)]] + \
               [[("a", 1), ("b", 1), ("c", 1)]] * 9 + [[("a", 11)]]
    dev = torch.device("cuda")
    eager = replay(engine(cfg, W, dev, torch.bfloat16), P, schedule, keep_open=P)
    graph = replay(engine(cfg, W, dev, torch.bfloat16, graph=True), P, schedule, keep_open=P)
    for name in P:
        assert torch.equal(eager[name], graph[name]), name


def write_checkpoint(path, cfg, W):
    from safetensors.torch import save_file
    os.makedirs(path, exist_ok=True)
    with open(os.path.join(path, "config.json"), "w") as f:
        json.dump(cfg, f)
    save_file({k: v.to(torch.bfloat16).contiguous() for k, v in W.items()}, os.path.join(path, "model.safetensors"))


def test_checkpoint_registry_and_generate(tmp_path, dev):
    """a checkpoint folder is recognised by its architecture name and generates through the engine"""
    from ipex_llm_amd.models.registry import NativeCheckpointLM, native_architecture
    cfg = std_cfg()
    W = O.random_weights(cfg, 22)
    write_checkpoint(str(tmp_path / "m"), cfg, W)
    assert native_architecture(str(tmp_path / "m")) == "Sudosun"
    lm = NativeCheckpointLM(str(tmp_path / "m"), dtype=torch.float32, device=dev.type)
    prompt = O.random_tokens(cfg, 12, 5)
    out = lm.generate([prompt], max_new_tokens=5)
    assert out[0][len(prompt):] == O.greedy(cfg, W, prompt, 5)


def test_command_line_generates(tmp_path, dev, capsys):
    """``generate --prompt-ids`` (32-bit on the CPU, 16-bit on the GPU)"""
    from ipex_llm_amd.cli.main import main
    cfg = std_cfg()
    W = O.random_weights(cfg, 24)
    write_checkpoint(str(tmp_path / "m"), cfg, W)
    prompt = O.random_tokens(cfg, 9, 24)
    main(["generate", "-m", str(tmp_path / "m"), "--device", dev.type, "-n", "4", "--prompt-ids", ",".join(map(str, prompt))])
    got = [int(t) for t in capsys.readouterr().out.strip().splitlines()[-1].split(",")]
    if dev.type == "cpu":
        assert got == O.greedy(cfg, W, prompt, 4)
    assert len(got) == 4 and all(0 <= t < cfg["vocab"] for t in got)


def test_random_model_and_shapes():
    """the reader's tensor list is the plain form's, and its random weights build"""
    from ipex_llm_amd.models import sudosun as S
    cfg = std_cfg()
    spec = S.spec_from_config(cfg)
    assert S.tensor_shapes(spec) == O.tensor_shapes(cfg)
    assert S.random_model(spec, 0, torch.float32, "cpu").spec is spec


def test_reader_refuses_what_it_does_not_know():
    from ipex_llm_amd.models import sudosun as S

    def broken(change, layer=None):
        cfg = O.config([layer or O.pair_layer(mlp=O.moe())])
        cfg = json.loads(json.dumps(cfg))
        change(cfg["layers"][0])
        with pytest.raises(ValueError):
            S.spec_from_config(cfg)
    broken(lambda L: L.update(type="something"))
    broken(lambda L: L["mixer"]["left"].update(kv_heads=3))
    broken(lambda L: L["mixer"]["left"]["mask"].update(size=0))
    broken(lambda L: L["mixer"]["left"]["rot"].update(dims=14))
    broken(lambda L: L["mixer"]["right"].update(blocks=5))
    broken(lambda L: L["mlp"].update(kind="other"))
    broken(lambda L: L["mlp"]["router"]["groups"].update(count=4))
    broken(lambda L: L["mlp"]["router"].update(top=5))
    broken(lambda L: L["mixer"].update(decay=[0.5]), O.lightning_layer(heads=3))
    broken(lambda L: L["mixer"].update(kv_heads=3), O.delta_layer())
    cfg = O.config([O.pair_layer(mlp=O.moe())])
    W = O.random_weights(cfg)
    del W["l0.mix.left.temp"]
    with pytest.raises(KeyError):
        S.build(S.spec_from_config(cfg), W, torch.float32, "cpu")


def test_trace_replay_program(tmp_path, dev):
    """bin/trace_run: steps on standard input, logits files out, pages and slots given back at 'end'"""
    cfg = std_cfg()
    W = O.random_weights(cfg, 23)
    write_checkpoint(str(tmp_path / "m"), cfg, W)
    a, b = O.random_tokens(cfg, 70, 1), O.random_tokens(cfg, 20, 2)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": a[:40], "want": [0, 39]}], "end": []},
             {"step": 1, "entries": [{"id": "a", "tokens": a[40:69], "want": []}, {"id": "b", "tokens": b[:19], "want": [18]}], "end": []},
             {"step": 2, "entries": [{"id": "b", "tokens": b[19:], "want": [0]}, {"id": "a", "tokens": a[69:], "want": [0]}], "end": ["a", "b"]},
             {"step": 3, "entries": [{"id": "c", "tokens": b, "want": [19]}], "end": ["c"]}]
    env = dict(os.environ, ILLM_TRACE_DEVICE=dev.type)
    r = subprocess.run([sys.executable, os.path.join(ROOT, "bin", "trace_run"), "--model", str(tmp_path / "m"), "--dtype",
                        "float32", "--out", str(tmp_path / "out"), "--max-tokens", "192"],
                       input="\n".join(json.dumps(s) for s in steps) + "\n", capture_output=True, text=True, env=env,
                       timeout=600)
    assert r.returncode == 0, r.stderr[-2000:]
    assert [ln for ln in r.stdout.splitlines() if ln.startswith("done")] == [f"done {i}" for i in range(4)]
    import numpy as np
    V = cfg["vocab"]
    wa, wb = O.forward(cfg, W, a), O.forward(cfg, W, b)
    rd = lambda i: torch.from_numpy(np.fromfile(str(tmp_path / "out" / f"{i}.f32"), dtype="<f4").reshape(-1, V)).double()  # noqa: E731
    assert rel_err(rd(0), wa[[0, 39]]) < TOL[torch.float32]
    assert rel_err(rd(1), wb[[18]]) < TOL[torch.float32]
    assert rel_err(rd(2), torch.stack([wb[19], wa[69]])) < TOL[torch.float32]
    assert rel_err(rd(3), wb[[19]]) < TOL[torch.float32]
