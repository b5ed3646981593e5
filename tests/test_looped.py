"""Pre-norm decoders some of whose layers run several times over (Lokolorn
layout): the framework -- checkpoint reader, paged rows and state slots of every
pass, scheduler, ragged engine steps, kernels -- against the plain float64 forms of
tests/looped_oracle.py.

Every test runs on the CPU (torch forms of ops/chanmix.py, ops/seqmix.py,
...) and, marked ``gpu``, on the HIP kernels.  Models are small random ones
made here.
"""
import json
import os
import subprocess
import sys

import pytest
import torch

from . import looped_oracle as O

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
    """all three mixers, two of them inside the loop and one behind it; windows shorter than a page and one that
    straddles pages; value sizes that differ from key sizes; a layer without a feed-forward"""
    return O.config([O.delta_layer(heads=4, kv_heads=2, dim=12, vdim=10, taps=3, mlp=O.moe(6, 2, 12, (3, 2))),
                     O.latent_layer(heads=3, dim=10, rot_dim=8, vdim=6, kv_rank=20, window=9, mlp=O.moe(4, 3, 8, (2, 2))),
                     O.pair_layer(heads=4, kv_heads=2, dim=12, vdim=10, dims=8, taps=3, rheads=3, rdim=6,
                                  mlp=O.moe(8, 3, 8, (4, 3), 0.6)),
                     O.latent_layer(heads=2, dim=8, rot_dim=4, vdim=12, kv_rank=12, window=70, scaling=None),
                     O.delta_layer(heads=3, kv_heads=3, dim=20, vdim=70, taps=1, mlp=O.moe(4, 2, 12, None))], width=40)


def public(cfg):
    """the configuration as a checkpoint holds it (the ranks of the low-rank projections come from the tensors)"""
    c = json.loads(json.dumps(cfg))
    for L in c["layers"]:
        L.pop("_rank", None)
        L.pop("_grank", None)
    return c


def no_close_calls(cfg):
    """every expert chosen: 16-bit runs then differ from the plain form by rounding alone"""
    c = json.loads(json.dumps(cfg))
    for L in c["layers"]:
        if L["mlp"] is not None:
            r = L["mlp"]["router"]
            r["top"] = r["experts"]
            if "groups" in r:
                r["groups"]["keep"] = r["groups"]["count"]
    return c


def calm(W):
    """smaller steps of the residual stream: a net of a few narrow layers with random weights otherwise amplifies 16-bit
    rounding many times over"""
    return {k: v * 0.375 if k.endswith((".ls1", ".ls2")) else v for k, v in W.items()}


def spec_of(cfg):
    from ipex_llm_amd.models import lokolorn as M
    return M.spec_from_config(public(cfg), M.ranks_of(O.tensor_shapes(cfg)))


def build(cfg, W, dev, dtype=torch.float32):
    from ipex_llm_amd.models import lokolorn as M
    return M.build(spec_of(cfg), W, dtype, dev)


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
@pytest.mark.parametrize("act", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("Wd", [5, 37, 40, 1100, 4160, 17000])
def test_scaled_residual_and_norm(dev, act, Wd):
    """nothing, one result (activation dtype or f32), two results, or expert rows: scaled, added, normed; and the same
    sources in front of a loop's projection"""
    from ipex_llm_amd.ops import chanmix as CX
    g = torch.Generator().manual_seed(Wd)
    T, top, V = 5, 3, 11
    rel = 1e-5 if act == torch.float32 else 5e-3

    def close(got, want):
        return ((got.double().cpu() - want).abs() / (1 + want.abs())).max() < rel
    x0 = torch.randn(T, Wd, generator=g) * 2
    w = 1 + 0.2 * torch.randn(Wd, generator=g)
    sa, sb = torch.randn(Wd, generator=g), torch.randn(Wd, generator=g)
    a, b = torch.randn(T, Wd, generator=g).to(act), torch.randn(T, Wd, generator=g).to(act)
    a32, rows = torch.randn(T, Wd, generator=g), torch.randn(T, top, Wd, generator=g)
    table, ids = torch.randn(V, Wd, generator=g).to(act), torch.tensor([0, 3, 10, 3, 7])
    sad, sbd = sa.double(), sb.double()
    for y, want in ((None, 0.0), (CX.Pending(a.to(dev), sa.to(dev)), sad * a.double()),
                    (CX.Pending(a32.to(dev), sa.to(dev)), sad * a32.double()),
                    (CX.Pending(a.to(dev), sa.to(dev), b.to(dev), sb.to(dev)), sad * a.double() + sbd * b.double()),
                    (CX.Pending(rows.to(dev), sa.to(dev)), sad * rows.double().sum(1))):
        x = x0.clone().to(dev)
        xn = x0.double() + want
        inp = CX.loop_input(x, y, table.to(dev), ids.to(dev))
        assert inp.dtype == act and torch.equal(x.cpu(), x0)
        assert close(inp, torch.cat([xn, table.double()[ids]], -1))
        got = CX.add_scaled_norm_(x, y, w.to(dev), 1e-5, act)
        assert (x.double().cpu() - xn).abs().max() < 2e-5
        assert got.dtype == act and close(got, O.unit_rms(xn, 1e-5) * w.double())
        if y is not None:
            idx = torch.tensor([3, 1])
            assert (y.select(idx.to(dev)).value().double().cpu() - want[idx]).abs().max() < 2e-5


@pytest.mark.parametrize("act", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("Wd", [6, 37, 1040])
def test_blends_with_the_previous_token(dev, act, Wd):
    """over portions, batches and slots with an earlier owner's content; a blend of 0 is the token's own row, of 1 its
    predecessor's"""
    from ipex_llm_amd.ops import chanmix as CX
    g = torch.Generator().manual_seed(Wd)
    mu = torch.stack([torch.zeros(Wd), torch.ones(Wd), torch.randn(Wd, generator=g)])
    seqs = [torch.randn(n, Wd, generator=g).to(act) for n in (73, 64, 75)]
    state = torch.randn(5, Wd, generator=g).to(dev)

    def f(rows, lens, cu, seq_of, slots, pos):
        return CX.token_mixes(rows, mu.to(dev), state, cu, seq_of, slots, pos, lens).permute(1, 0, 2).reshape(rows.shape[0], -1)

    for x, o in zip(seqs, in_portions(f, seqs, CUTS, dev)):
        x = x.double()
        want = torch.cat([x + (O.shifted(x) - x) * m.double() for m in mu], -1)
        assert (o - want).abs().max() < (1e-5 if act == torch.float32 else 5e-2)


@pytest.mark.parametrize("N,R", [(24, 5), (70, 16), (1, 1), (130, 24), (64, 33), (200, 72)])
@pytest.mark.parametrize("kind,squash", [("softplus", False), ("exp", True), ("softplus", True), ("exp", False)])
def test_lowrank_decay(dev, N, R, kind, squash):
    """decays from near 0 to near 1 keep f32 precision (16-bit weights and inputs enter the sums unrounded)"""
    from ipex_llm_amd.ops import chanmix as CX
    g = torch.Generator().manual_seed(N + R)
    rate, bias = torch.rand(N, generator=g) * 3, torch.randn(N, generator=g) * 2
    for act in (torch.float32, torch.bfloat16):
        w = (torch.randn(N, R, generator=g) * R ** -0.5).to(act)
        for T in (1, 9, 150):
            y = (torch.randn(T, R + 7, generator=g) * 2).to(act)
            got = CX.lowrank_decay(y.to(dev)[:, 3:3 + R], w.to(dev), rate.to(dev), bias.to(dev), kind, squash)
            a = y[:, 3:3 + R].double()
            z = (torch.tanh(a) if squash else a) @ w.double().T + bias.double()
            want = torch.exp(-rate.double() * O.softplus(z)) if kind == "softplus" else torch.exp(-torch.exp(z))
            assert got.dtype == torch.float32 and (got.double().cpu() - want).abs().max() < 5e-6


@pytest.mark.parametrize("M", [1, 5, 16])
@pytest.mark.parametrize("K,sizes", [(64, [16, 1, 33]), (320, [40, 24, 24, 24, 24, 5]), (1088, [130])])
def test_row_groups_with_inputs_of_their_own(dev, M, K, sizes):
    from ipex_llm_amd.ops import chanmix as CX
    g = torch.Generator().manual_seed(K)
    xs = [torch.randn(M, K, generator=g).bfloat16() for _ in sizes]
    w, b = (torch.randn(sum(sizes), K, generator=g) * K ** -0.5).bfloat16(), torch.randn(sum(sizes), generator=g).bfloat16()
    want = torch.cat([x.double() @ p.double().T for x, p in zip(xs, w.split(sizes))], -1)
    for bias, f32 in ((b, False), (None, True)):
        got = CX.grouped_linear([x.to(dev) for x in xs], sizes, w.to(dev), bias.to(dev) if bias is not None else None, f32)
        ref = want if bias is None else want + b.double()
        assert (got.double().cpu() - ref).abs().max() < (1e-4 if f32 else 3e-2)
    if len(sizes) == 1:
        for n in (M, 30):
            x = torch.randn(n, K, generator=g).bfloat16()
            got = CX.linear_f32(x.to(dev), w.to(dev))
            assert got.dtype == torch.float32 and (got.double().cpu() - x.double() @ w.double().T).abs().max() < 1e-4


SIZES = [(4, 2, 6, 10), (2, 2, 48, 64), (1, 1, 70, 70), (6, 2, 130, 8), (1, 1, 1, 1), (2, 1, 300, 20), (4, 4, 64, 128),
         (3, 1, 16, 17), (2, 1, 128, 16), (3, 3, 33, 5)]


def decays(g, *shape):
    """all but clearing, middling and near 1, mixed over tokens and channels"""
    z = torch.randn(*shape, generator=g)
    return torch.exp(-torch.exp(3.0 * z - 3.0))


@pytest.mark.parametrize("chunk_min", [0, 2])
@pytest.mark.parametrize("H,K,d,dv", SIZES)
def test_channel_delta_scan(dev, H, K, d, dv, chunk_min, monkeypatch):
    """over portions and batches, key heads shared by several value heads, dirty slots; on the GPU token by token and in
    chunks"""
    from ipex_llm_amd.ops import chanmix as CX
    monkeypatch.setattr(CX, "CHUNK_MIN", chunk_min)
    g = torch.Generator().manual_seed(H + d)
    for act in (torch.float32, torch.bfloat16):
        seqs, want = [], []
        for n in (73, 64, 75):
            q, k, v = torch.randn(n, K, d, generator=g), torch.randn(n, K, d, generator=g), torch.randn(n, H, dv, generator=g)
            dec, b = decays(g, n, H, d), (torch.randn(n, H + 3, generator=g) * 1.5).to(act)
            seqs.append(torch.cat([t.reshape(n, -1).float() for t in (q, k, v, dec, b)], 1))
            want.append(O.channel_delta_scan(O.unit(q.double()) * d ** -0.5, O.unit(k.double()), v.double(), dec.double(),
                                             O.sigmoid(b[:, 2:2 + H].double())).reshape(n, -1))
        state = torch.randn(5, H, d, dv, generator=g).to(dev)

        def f(rows, lens, cu, seq_of, slots, pos):
            T, n = rows.shape[0], K * d
            u, dec, b = rows[:, :2 * n + H * dv], rows[:, 2 * n + H * dv:-(H + 3)], rows[:, -(H + 3):].to(act)
            return CX.channel_delta_scan(u[:, :n].view(T, K, d), u[:, n:2 * n].view(T, K, d), u[:, 2 * n:].view(T, H, dv),
                                         dec.reshape(T, H, d), b[:, 2:2 + H], d ** -0.5, state, cu, slots, pos,
                                         lens).reshape(T, -1)

        for o, w in zip(in_portions(f, seqs, CUTS, dev), want):
            assert (o - w).abs().max() < 2e-5 * max(1.0, float(w.abs().max()))


@pytest.mark.parametrize("chunk_min", [0, 2])
@pytest.mark.parametrize("H,_,d,dv", SIZES)
def test_bonus_scan(dev, H, _, d, dv, chunk_min, monkeypatch):
    """read-out before the write, the bonus for the current token only; over portions and batches, dirty slots; on the
    GPU token by token and in chunks"""
    from ipex_llm_amd.ops import chanmix as CX
    monkeypatch.setattr(CX, "CHUNK_MIN", chunk_min)
    g = torch.Generator().manual_seed(H + d)
    u = torch.randn(H, d, generator=g)
    for act in (torch.float32, torch.bfloat16):
        seqs, want = [], []
        for n in (73, 64, 75):
            r, k, v = (torch.randn(n, H, e, generator=g).to(act) for e in (d, d, dv))
            dec = decays(g, n, H, d)
            seqs.append(torch.cat([t.reshape(n, -1).float() for t in (r, k, v, dec)], 1))
            want.append(O.bonus_scan(r.double(), k.double(), v.double(), dec.double(), u.double()).reshape(n, -1))
        state = torch.randn(5, H, d, dv, generator=g).to(dev)

        def f(rows, lens, cu, seq_of, slots, pos):
            T, n = rows.shape[0], H * d
            a = rows[:, :2 * n + H * dv].to(act)
            return CX.bonus_scan(a[:, :n].view(T, H, d), a[:, n:2 * n].view(T, H, d), a[:, 2 * n:].view(T, H, dv),
                                 rows[:, 2 * n + H * dv:].reshape(T, H, d), u.to(dev), state, cu, slots, pos,
                                 lens).reshape(T, -1)

        for o, w in zip(in_portions(f, seqs, CUTS, dev), want):
            assert (o - w).abs().max() < 2e-5 * max(1.0, float(w.abs().max()))


def test_long_portions_of_the_scans(dev):
    """portions of thousands of tokens (on the GPU: many chunks, more than one segment of them) beside short ones and
    one that continues; equal keys with steps near 1, decays that all but clear single channels now and then beside
    channels that hardly decay"""
    from ipex_llm_amd.ops import chanmix as CX
    g = torch.Generator().manual_seed(6)
    H, d, dv = 1, 5, 3
    lens, starts = [8400, 1, 130, 64], [0, 9, 3, 0]
    T = sum(lens)
    cu, _, slots, pos = ragged(lens, starts, dev)
    q, k, v = torch.randn(T, H, d, generator=g), torch.randn(T, H, d, generator=g), torch.randn(T, H, dv, generator=g)
    k[100:300] = k[100]
    dec = torch.exp(-torch.exp(torch.randn(T, H, d, generator=g) - 5.0))
    dec[torch.arange(50, T, 97), 0, 1] = 0.0
    dec[torch.arange(20, T, 61), 0, 2] = 1e-30
    dec[:, :, 3] = 1.0
    b = torch.randn(T, H, generator=g)
    b[100:200] = 9.0
    u = torch.randn(H, d, generator=g)
    S0 = torch.randn(6, H, d, dv, generator=g)

    def check(got, state, step):
        t0 = 0
        for s, n in enumerate(lens):
            S = torch.zeros(H, d, dv, dtype=F64) if starts[s] == 0 else S0[s + 1].double()
            want = torch.empty(n, H, dv, dtype=F64)
            for t in range(n):
                S, want[t] = step(S, t0 + t)
            tol = 5e-5 * max(1.0, float(want.abs().max()))
            assert (got[t0:t0 + n].double().cpu() - want).abs().max() < tol, s
            assert (state[s + 1].double().cpu() - S).abs().max() < 5e-5 * max(1.0, float(S.abs().max())), s
            t0 += n

    state = S0.clone().to(dev)
    got = CX.channel_delta_scan(q.to(dev), k.to(dev), v.to(dev), dec.to(dev), b.to(dev), 0.5, state, cu, slots, pos, lens)
    qu, ku, vd, dd, be = O.unit(q.double()) * 0.5, O.unit(k.double()), v.double(), dec.double(), O.sigmoid(b.double())

    def rule(S, t):
        S = dd[t][:, :, None] * S
        uu = be[t][:, None] * (vd[t] - (S * ku[t][:, :, None]).sum(1))
        S = S + ku[t][:, :, None] * uu[:, None, :]
        return S, (S * qu[t][:, :, None]).sum(1)
    check(got, state, rule)
    # (channel 3 never decays: small keys keep its sum small)
    kb = 0.05 * k
    state = S0.clone().to(dev)
    got = CX.bonus_scan(q.to(dev), kb.to(dev), v.to(dev), dec.to(dev), u.to(dev), state, cu, slots, pos, lens)
    qd, kd, ud = q.double(), kb.double(), u.double()

    def bonus(S, t):
        kv = kd[t][:, :, None] * vd[t][:, None, :]
        o = ((S + ud[:, :, None] * kv) * qd[t][:, :, None]).sum(1)
        return dd[t][:, :, None] * S + kv, o
    check(got, state, bonus)


ROUTES = [(6, 2, 3, 2), (20, 4, 4, 3), (7, 7, 1, 1), (130, 5, 13, 2), (512, 8, 64, 4), (9, 3, 9, 4), (4, 1, 2, 1), (8, 3, 4, 3)]


@pytest.mark.parametrize("E,top,groups,keep", ROUTES)
def test_routing_by_sigmoid_scores(dev, E, top, groups, keep):
    """groups ranked by their two best corrected scores (one, when a group has one expert), which may be negative;
    weights renormalised over the winners and scaled"""
    from ipex_llm_amd.ops import statemix as SX
    rule = SX.RouteRule("sigmoid", "top2", True, 2.2)
    g = torch.Generator().manual_seed(E)
    z, corr = torch.randn(40, E, generator=g) * 2, torch.randn(E, generator=g) * 0.1 - 0.8
    h, rw = torch.randn(30, 24, generator=g), torch.randn(E, 24, generator=g)
    idx, w = SX.route_groups(z.to(dev), corr.to(dev), top, groups, keep, rule)
    idx2, w2 = SX.route(h.to(dev), rw.to(dev), corr.to(dev), top, groups, keep, rule)
    for i, ww, zz in ((idx, w, z.double()), (idx2, w2, h.double() @ rw.double().T)):
        for t in range(zz.shape[0]):
            want = O.route(zz[t], corr.double(), top, {"count": groups, "keep": keep}, 2.2)
            assert i[t].tolist() == [e for e, _ in want]
            assert (ww[t].double().cpu() - torch.stack([s for _, s in want])).abs().max() < 2e-6


def test_group_choice_by_the_two_best(dev):
    """the best single score sits in a group that loses to a group with the better pair; choice scores that are all
    negative still win over experts of groups that are not kept"""
    from ipex_llm_amd.ops import statemix as SX
    rule = SX.RouteRule("sigmoid", "top2", True, 1.0)
    z = torch.tensor([[3.0, -6.0, 1.5, 1.4]])
    idx, w = SX.route_groups(z.to(dev), None, 2, 2, 1, rule)
    assert idx.tolist() == [[2, 3]] and abs(float(w.sum()) - 1.0) < 1e-6
    corr = torch.tensor([-4.0, -4.0, -1.5, -1.5])
    idx, w = SX.route_groups(z.to(dev), corr.to(dev), 2, 2, 1, rule)
    assert idx.tolist() == [[2, 3]]
    s = torch.sigmoid(z[0, 2:])
    assert (w.cpu()[0] - s / s.sum()).abs().max() < 1e-6


@pytest.mark.parametrize("r,dr,H", [(20, 8, 3), (96, 32, 8), (130, 4, 5), (64, 64, 16)])
@pytest.mark.parametrize("act", [torch.float32, torch.bfloat16])
def test_latent_attention_with_a_sink(dev, act, r, dr, H, monkeypatch):
    """decoded tokens, short portions and (threshold lowered) the product path of long ones, over shuffled pages; sinks
    that take next to nothing and almost everything"""
    from ipex_llm_amd.ops import seqmix as SM
    g = torch.Generator().manual_seed(r)
    rows = torch.randn(9, 64, r + dr, generator=g).to(act)
    bt = torch.tensor([[7, 2, 5, 0], [3, 8, 1, 0]], dtype=torch.int32)
    sink = torch.linspace(-30.0, 30.0, H)
    for lens, ctx in (([1, 1], [150, 70]), ([5, 1], [64, 129]), ([60, 3], [180, 3])):
        cu, seq_of, _, pos = ragged(lens, [c - n for c, n in zip(ctx, lens)], dev)
        T = sum(lens)
        ql, qr = torch.randn(T, H, r, generator=g).to(act), torch.randn(T, H, dr, generator=g).to(act)
        for window in (0, 1, 30, 64):
            want, t = torch.empty(T, H, r, dtype=F64), 0
            for b, (n, c) in enumerate(zip(lens, ctx)):
                kv = rows[bt[b].long()].reshape(-1, r + dr)[:c].double()
                for p in range(c - n, c):
                    lo = max(0, p - window + 1) if window else 0
                    for h in range(H):
                        s = kv[lo:p + 1] @ torch.cat([ql[t, h], qr[t, h]]).double() * 0.1
                        want[t, h] = O.sink_weights(s, sink[h]) @ kv[lo:p + 1, :r]
                    t += 1
            for limit in (SM.GEMM_MIN_Q, 2):
                monkeypatch.setattr(SM, "GEMM_MIN_Q", limit)
                got = SM.latent_attention(ql.to(dev), qr.to(dev), rows.to(dev), bt.to(dev), seq_of, pos, 0.1, None, lens, ctx,
                                          act, window=window, sink=sink.to(dev))
                assert (got.double().cpu() - want).abs().max() < (1e-4 if act == torch.float32 else 3e-2)
            monkeypatch.undo()


@pytest.mark.parametrize("d,dv,dims", [(12, 10, 8), (16, 8, 6), (96, 24, 48), (128, 128, 128), (40, 16, 40), (8, 6, 2), (64, 48, 64)])
@pytest.mark.parametrize("act", [torch.float32, torch.bfloat16])
def test_rotation_and_weightless_norm(dev, act, d, dv, dims):
    """the op norms and then turns; the plain form turns and then norms"""
    from ipex_llm_amd.ops import maskattn as MA
    from ipex_llm_amd.ops.seqmix import rope_table
    g = torch.Generator().manual_seed(4)
    T, H, G = 11, 6, 2
    y = torch.randn(T, H * d + G * (d + dv), generator=g)
    q, k, v = y[:, :H * d].view(T, H, d), y[:, H * d:(H + G) * d].view(T, G, d), y[:, (H + G) * d:].view(T, G, dv)
    rot, one = {"dims": dims, "base": 3000.0}, torch.ones(d, dtype=act, device=dev)
    tab, pos = rope_table(64, dims, 3000.0).to(dev), torch.arange(20, 20 + T)
    rows = torch.zeros(2, 64, G * (d + dv), dtype=act, device=dev)
    yd = y.to(dev)
    got = MA.qkv_norm_rope_store(yd[:, :H * d].view(T, H, d), yd[:, H * d:(H + G) * d].view(T, G, d),
                                 yd[:, (H + G) * d:].view(T, G, dv), one, one, False, 1e-5, tab, "half", pos.to(dev),
                                 (pos + 30).to(dev), rows).double().cpu()
    assert (got - O.unit_rms(O.turn_half(q.double(), rot, pos), 1e-5)).abs().max() < 2e-5
    keys = O.unit_rms(O.turn_half(k.double(), rot, pos), 1e-5).reshape(T, -1)
    stored = rows.view(128, -1)[50:50 + T].double().cpu()
    tol = 2e-5 if act == torch.float32 else 3e-2
    assert (stored[:, :G * d] - keys).abs().max() < tol and (stored[:, G * d:] - v.double().reshape(T, -1)).abs().max() < tol


@pytest.mark.parametrize("act", [torch.float32, torch.bfloat16])
def test_head_norm_gates(dev, act):
    from ipex_llm_amd.ops import seqmix as SM
    g = torch.Generator().manual_seed(1)
    for T, H, dv in ((6, 3, 10), (3, 2, 130), (70, 4, 64), (2, 1, 1)):
        o, w = torch.randn(T, H, dv, generator=g) * 3, (1 + 0.2 * torch.randn(H * dv, generator=g)).to(act)
        gate = torch.randn(T, H * dv + 9, generator=g).to(act)[:, 4:4 + H * dv]
        n = O.unit_rms(o.double(), 1e-5).reshape(T, -1) * w.double()
        for silu in (False, True):
            got = SM.head_rms_gate(o.to(dev), w.to(dev), gate.to(dev), 1e-5, act, silu=silu)
            want = n * (O.silu if silu else O.sigmoid)(gate.double())
            assert got.dtype == act and (got.double().cpu() - want).abs().max() < (3e-5 if act == torch.float32 else 8e-2)


@pytest.mark.parametrize("E,top,ff,Wd,T,groups", [(6, 2, 12, 40, 9, (3, 2)), (8, 3, 88, 64, 150, (4, 3)), (3, 3, 8, 24, 4, (1, 1)),
                                                  (1, 1, 5, 9, 3, (1, 1))])
def test_experts(dev, E, top, ff, Wd, T, groups):
    from ipex_llm_amd.models.hybrid import ExpertSpec, MoESpec, ScoredMoE
    g = torch.Generator().manual_seed(E + T)
    for act in (torch.float32, torch.bfloat16):
        W = {"router": torch.randn(E, Wd, generator=g), "correction": 0.1 * torch.randn(E, generator=g) - 0.5}
        for e in range(E):
            W.update({f"e{e}.gate": torch.randn(ff, Wd, generator=g) * Wd ** -0.5,
                      f"e{e}.up": torch.randn(ff, Wd, generator=g) * Wd ** -0.5,
                      f"e{e}.down": torch.randn(Wd, ff, generator=g) * ff ** -0.5})
        W = {k: v.to(act) for k, v in W.items()}
        h = torch.randn(T, Wd, generator=g).to(act)
        spec = MoESpec(E, top, ExpertSpec(ff), groups=groups[0], keep=groups[1], score="sigmoid", group="top2", renorm=True,
                       scale=1.9)
        moe = ScoredMoE(spec, W["router"], W["correction"],
                        torch.stack([torch.cat([W[f"e{e}.gate"], W[f"e{e}.up"]]) for e in range(E)]),
                        torch.stack([W[f"e{e}.down"] for e in range(E)])).to(dev)
        cfg = {"router": {"experts": E, "top": top, "scale": 1.9, "groups": {"count": groups[0], "keep": groups[1]}}}
        want = O.experts({k: v.double() for k, v in W.items()}, "", cfg, h.double())
        assert (moe(h.to(dev))[0].double().cpu() - want).abs().max() < (2e-4 if act == torch.float32 else 0.1)


# ------------------------------------------------------------------ whole models
_want = {}


def oracle(cfg, W, toks, key):
    if key not in _want:
        _want[key] = O.forward(cfg, W, toks)
    return _want[key]


LAYER_CASES = [
    ([O.delta_layer(heads=4, kv_heads=2, dim=12, vdim=10, taps=3, mlp=O.moe(4, 3, 8, (2, 2)))], None),
    ([O.delta_layer(heads=1, kv_heads=1, dim=1, vdim=1, taps=1, rank=1, grank=1),
      O.delta_layer(heads=6, kv_heads=1, dim=9, vdim=5, taps=5, rank=9, grank=3, mlp=O.moe(1, 1, 7, None, 1.0))], (0, 1, 3)),
    ([O.latent_layer(mlp=O.moe(3, 2, 8, None))], (0, 1, 1)),
    ([O.latent_layer(heads=1, dim=1, rot_dim=2, vdim=1, kv_rank=1, window=1, scaling=None),
      O.latent_layer(heads=9, dim=4, rot_dim=6, vdim=9, kv_rank=7, window=64, scale=1.0,
                     scaling={"factor": 1.0, "original": 32, "fast": 4.0, "slow": 1.0}, mlp=O.moe(6, 2, 5, (3, 1)))], (1, 2, 2)),
    ([O.pair_layer(mlp=O.moe(6, 2, 8, (2, 2)))], (0, 1, 2)),
    ([O.pair_layer(heads=1, kv_heads=1, dim=2, vdim=1, dims=2, taps=1, rheads=1, rdim=1, rank=1, scales=(1.0, 1.0))], None),
    ([O.pair_layer(heads=3, kv_heads=3, dim=6, vdim=6, dims=6, taps=5, rheads=5, rdim=3, rank=17, scales=(-0.5, 1.6), scale=1.0)],
     (0, 1, 4)),
    ([O.pair_layer(heads=8, kv_heads=1, dim=10, vdim=20, dims=4, taps=2, rheads=2, rdim=20, scales=(0.0, 0.8)),
      O.delta_layer(mlp=O.moe(8, 4, 3, (4, 2), 0.3)), O.latent_layer(window=65)], (0, 3, 2)),
]


@pytest.mark.parametrize("case", range(len(LAYER_CASES)))
def test_small_models(dev, case):
    """each mixer alone and in pairs, sizes that are 1 or equal to each other, layers without a feed-forward, no loop, a
    loop over every layer, one pass, four passes"""
    layers, loop = LAYER_CASES[case]
    cfg = O.config(layers, width=24 + 2 * case, eps=[1e-5, 1e-3][case % 2], loop=loop)
    W = O.random_weights(cfg, case)
    toks = O.random_tokens(cfg, 75, case)
    want = O.forward(cfg, W, toks)
    got = replay(engine(cfg, W, dev), {"a": toks}, [[("a", 40)], [("a", 30)]] + [[("a", 1)]] * 5)["a"]
    assert rel_err(got, want) < 5 * TOL[torch.float32]                 # (heads of one value: norms of single numbers)
    got = replay(engine(cfg, W, dev, torch.bfloat16), {"a": toks}, [[("a", 70)], [("a", 3)]] + [[("a", 1)]] * 2)["a"]
    # 16-bit: rows of 1 to 40 values average little rounding away, so nine rows in ten are looked at
    d = got - want
    assert float((d - d.mean(-1, keepdim=True)).pow(2).mean(-1).sqrt().quantile(0.9) / want.std()) < 0.3


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_odd_sizes(dev, dtype):
    """widths, head sizes, expert sizes and vocabulary that are multiples of nothing"""
    cfg = O.config([O.pair_layer(heads=3, kv_heads=1, dim=9, vdim=7, dims=4, taps=3, rheads=3, rdim=11, rank=7,
                                 mlp=O.moe(7, 3, 5, (7, 4))),
                    O.delta_layer(heads=3, kv_heads=1, dim=7, vdim=5, taps=2, rank=3, grank=11, mlp=O.moe(9, 2, 7, (3, 1))),
                    O.latent_layer(heads=5, dim=3, rot_dim=6, vdim=7, kv_rank=13, window=5)], vocab=53, width=37, loop=(1, 3, 3))
    W = O.random_weights(cfg, 31)
    if dtype == torch.bfloat16:
        cfg, W = no_close_calls(cfg), calm(W)
    toks = O.random_tokens(cfg, 70, 31)
    got = replay(engine(cfg, W, dev, dtype), {"a": toks}, [[("a", 33)], [("a", 30)]] + [[("a", 1)]] * 7)["a"]
    # (16-bit: heads of three to eleven values average little rounding away)
    assert rel_err(got, O.forward(cfg, W, toks)) < (TOL[dtype] if dtype == torch.float32 else 0.2)


def test_whole_prompt_and_layers(dev):
    """the residual stream after every run of a layer (a looped layer counts each time)"""
    cfg = std_cfg()
    W = O.random_weights(cfg, 7)
    toks = O.random_tokens(cfg, 141, 7)
    eng = engine(cfg, W, dev)
    eng.model.capture_layers = []
    got = replay(eng, {"a": toks}, [[("a", 141)]])["a"]
    layers = []
    want = O.forward(cfg, W, toks, layers_out=layers)
    assert rel_err(got, want) < TOL[torch.float32]
    assert len(eng.model.capture_layers) == len(layers) == 7
    for a, b in zip(eng.model.capture_layers, layers):
        assert (a.double().cpu() - b).abs().max() < 1e-4 * float(b.abs().max())


def test_every_pass_has_its_own_cache_and_state(dev):
    """as many cache entries as runs; a plain form whose second pass saw the first one's keys and states would differ,
    so would one pass fewer"""
    cfg = O.config([O.latent_layer(window=30), O.delta_layer()], width=24, loop=(0, 2, 2))
    W = O.random_weights(cfg, 5)
    toks = O.random_tokens(cfg, 60, 5)
    eng = engine(cfg, W, dev)
    assert eng.cache.num_layers == 4
    assert [r is not None for r in eng.cache.rows] == [True, False, True, False]
    assert eng.model.cache_bytes_per_token() == 2 * 28 * 4
    want = O.forward(cfg, W, toks)
    got = replay(eng, {"a": toks}, [[("a", 45)]] + [[("a", 1)]] * 15)["a"]
    err = (got - want).abs().max()
    once = O.forward(dict(cfg, loop={"start": 0, "stop": 2, "times": 1}), W, toks)
    assert rel_err(got, want) < TOL[torch.float32] and (once - want).abs().max() > 200 * err


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
    cfg = no_close_calls(std_cfg())
    W = calm(O.random_weights(cfg, 14))
    toks = O.random_tokens(cfg, 90, 14)
    got = replay(engine(cfg, W, dev, torch.bfloat16), {"a": toks}, [[("a", 73)], [("a", 2)]] + [[("a", 1)]] * 15)["a"]
    assert rel_err(got, O.forward(cfg, W, toks)) < TOL[torch.bfloat16]


def edge_model(window):
    """one latent-attention layer whose keys follow the token's embedding: a marked token's key towers over the others
    for every query, so its value shows in every position that sees it"""
    cfg = O.config([O.latent_layer(heads=2, dim=8, rot_dim=2, vdim=6, kv_rank=8, window=window, scaling=None, scale=1.0)],
                   vocab=12, width=16, loop=None)
    W = O.random_weights(cfg, 40)
    p = "l0.mix."
    W["embed"][:, 0] = 0.0
    W["embed"][:, 1] = 1.0
    W["embed"][11] *= 0.2
    W["embed"][11, 0] = 6.0                                            # the marked token: coordinate 0
    W["l0.norm1"].zero_()
    W[p + "dkv"][0].zero_()
    W[p + "dkv"][0, 0] = 8.0                                           # ... fills the latent's first value
    W[p + "dkv.norm"].fill_(1.0)
    for n in ("q", "uk"):
        W[p + n].zero_()
    W[p + "dkv"][8:].zero_()                                           # no rotated part
    W[p + "q"][7::10, 1] = 3.0                                         # queries: the same unrotated direction everywhere
    W[p + "uk"][7::8, 0] = 4.0                                         # the latent's first value is the key there
    W[p + "sink"].fill_(-1.0)
    return cfg, W


@pytest.mark.parametrize("window", [70, 64, 33, 1, 2])
@pytest.mark.parametrize("where", [0, 5, 63, 64])
def test_a_key_just_inside_and_just_outside(dev, window, where):
    """the marked token at position ``where``: the last position whose window holds it and the first that does not,
    as tokens of a prompt and decoded one by one"""
    cfg, W = edge_model(window)
    n = where + window + 3
    toks = [1 + (i * 7) % 10 for i in range(n)]
    toks[where] = 11
    want = O.forward(cfg, W, toks)
    last = where + window - 1
    no_key = {k: v.clone() for k, v in W.items()}
    no_key["l0.mix.uk"].zero_()
    blind = O.forward(cfg, no_key, toks)                               # what it would be if the key did not stand out
    if window > 2:
        assert (want[last] - blind[last]).abs().max() > 2 * (want[last + 1] - blind[last + 1]).abs().max()
        assert (want[last] - want[last + 1]).abs().max() > 0.1 * want.abs().max()
    for schedule in ([[("a", n)]], [[("a", max(last - 1, 1))]] + [[("a", 1)]] * (n - max(last - 1, 1))):
        got = replay(engine(cfg, W, dev), {"a": toks}, schedule)["a"]
        assert (got - want).abs().max() < 2e-4 * float(want.abs().max())


@pytest.mark.parametrize("at", [0, 63, 64, 130])
def test_a_far_key_of_the_causal_attention(dev, at):
    """a token whose key towers is asked for hundreds of positions later, from a prompt and decoded"""
    cfg = O.config([O.pair_layer(heads=2, kv_heads=1, dim=8, vdim=6, dims=2, base=1e6, taps=1, scale=3.0, rheads=1, rdim=2,
                                 scales=(1.0, 0.0))], vocab=12, width=16, loop=None)
    W = O.random_weights(cfg, 43)
    p = "l0.mix.left."
    W["embed"][:, 0] = 0.0
    W["embed"][11, 0] = 9.0
    W["l0.norm1"].zero_()
    for n in ("q", "k"):
        W[p + n].zero_()
        W[p + n + ".b"].zero_()
        W[p + n + ".conv"].fill_(1.0)
    W[p + "q.b"][7::8] = 1.0
    W[p + "k.b"][6] = 0.5
    W[p + "k"][7, 0] = 8.0
    toks = [1 + (i * 7) % 10 for i in range(330)]
    other = list(toks)
    toks[at] = 11
    want, without = O.forward(cfg, W, toks), O.forward(cfg, W, other)
    assert (want[-1] - without[-1]).abs().max() > 0.1 * want.abs().max()
    for schedule in ([[("a", 330)]], [[("a", 320)]] + [[("a", 1)]] * 10):
        got = replay(engine(cfg, W, dev), {"a": toks}, schedule)["a"]
        assert (got - want).abs().max() < 2e-4 * float(want.abs().max())


def test_what_could_be_left_out_shows(dev):
    """leaving out a mechanism, or one of its numbers, changes the plain form's logits by far more than the framework
    differs from it"""
    cfg = O.config([O.delta_layer(), O.latent_layer(scale=1.0), O.pair_layer(mlp=O.moe())], width=24, loop=(1, 2, 2))
    W = O.random_weights(cfg, 41)
    W["l1.mix.sink"] += 1.5
    toks = O.random_tokens(cfg, 60, 41)
    want = O.forward(cfg, W, toks)
    got = replay(engine(cfg, W, dev), {"a": toks}, [[("a", 50)]] + [[("a", 1)]] * 10)["a"]
    err = (got - want).abs().max()
    for name, value in (("l1.mix.sink", -60.0), ("l0.ls1", 1.0), ("l2.ls2", 1.0), ("l2.mix.right.u", 0.0), ("l2.mix.left.o.b", 0.0),
                        ("l2.mix.left.v.b", 0.0), ("l2.mix.right.mu.w", 0.0), ("l2.mix.right.mu.g", 0.0), ("l0.mix.a2", 0.0),
                        ("l0.mix.g2", 0.0), ("l2.mlp.correction", 0.0), ("l2.norm1", 0.0), ("final.norm", 0.0),
                        ("l1.mix.dkv.norm", 1.0), ("l0.mix.b", 0.0), ("l2.mix.right.w2", 0.0)):
        other = {k: v.clone() for k, v in W.items()}
        other[name].fill_(value)
        assert (O.forward(cfg, other, toks) - want).abs().max() > 100 * err, name
    half = {k: v.clone() for k, v in W.items()}
    half["loop.in"][:, 24:] = 0.0                                      # the embedding's half of the projection
    assert (O.forward(cfg, half, toks) - want).abs().max() > 100 * err


@pytest.mark.parametrize("kind", ["delta", "time_mix"])
def test_a_far_token_reaches_through_the_state(dev, kind):
    """changing the first token changes the logits hundreds of tokens later through the recurrent state alone; the
    framework follows the plain form on both prompts, over a prompt, a portion and decoded tokens"""
    layer = {"delta": O.delta_layer(heads=2, kv_heads=1, taps=2), "time_mix": O.pair_layer(scales=(0.0, 1.0))}[kind]
    cfg = O.config([layer], width=24, loop=None)
    W = O.random_weights(cfg, 16)
    if kind == "delta":
        W["l0.mix.A_log"].fill_(-8.0)
        W["l0.mix.b"].zero_()
        W["l0.mix.b"][:, 0] = -6.0                                     # tiny steps: old content is hardly overwritten ...
        W["embed"][:, 0] = 2.0
        W["embed"][-2:, 0] = -2.0                                      # ... but a large one at the first token
    else:
        W["l0.mix.right.w0"].fill_(-8.0)
    V = cfg["vocab"]
    rest = [t % (V - 2) for t in O.random_tokens(cfg, 299, 16)]
    a, b = [V - 1] + rest, [V - 2] + rest
    wa, wb = O.forward(cfg, W, a)[-1], O.forward(cfg, W, b)[-1]
    assert (wa - wb).abs().max() > 1e-3
    for toks, want in ((a, wa), (b, wb)):
        got = replay(engine(cfg, W, dev), {"a": toks}, [[("a", 170)], [("a", 120)]] + [[("a", 1)]] * 10)["a"][-1]
        assert (got - want).abs().max() < 0.05 * float((wa - wb).abs().max())


@pytest.mark.parametrize("sizes", [[50, 390, 10], [300, 150], [5, 445]])
def test_long_portions_take_the_product_path(dev, sizes, monkeypatch):
    """portions long enough for the block-by-block product paths on the GPU (thresholds and blocks lowered to this
    test's lengths), of the causal attention and of the latent one with its sink and window"""
    from ipex_llm_amd.ops import maskattn as MA
    from ipex_llm_amd.ops import seqmix as SM
    monkeypatch.setattr(MA, "CAUSAL_GEMM_MIN", 128)
    monkeypatch.setattr(MA, "WINDOW_Q_BLOCK", 160)
    monkeypatch.setattr(SM, "GEMM_Q_BLOCK", 96)
    cfg = O.config([O.pair_layer(heads=4, kv_heads=2, dim=16, vdim=24, dims=8), O.latent_layer(window=100, mlp=O.moe(3, 3, 12, None))], width=32,
                   loop=None)
    W = O.random_weights(cfg, 17)
    toks = O.random_tokens(cfg, 450, 17)
    want = oracle(cfg, W, toks, "w17")
    for dtype in (torch.float32, torch.bfloat16):
        got = replay(engine(cfg, W, dev, dtype), {"a": toks}, [[("a", n)] for n in sizes])["a"]
        assert rel_err(got, want) < TOL[dtype]


def test_mixed_steps_at_matrix_core_sizes(dev):
    """sizes that fill matrix-core tiles and ones that do not, long portions beside decoded tokens, both number formats"""
    cfg = O.config([O.delta_layer(heads=4, kv_heads=2, dim=80, vdim=48, taps=4, rank=24, grank=40, mlp=O.moe(8, 4, 40, (4, 3))),
                    O.latent_layer(heads=8, dim=32, rot_dim=16, vdim=40, kv_rank=80, window=50, scale=0.2),
                    O.pair_layer(heads=4, kv_heads=2, dim=40, vdim=56, dims=20, taps=4, rheads=3, rdim=72, rank=24,
                                 mlp=O.moe(6, 2, 64, (2, 1)))], vocab=120, width=128, loop=(1, 3, 2))
    W = O.random_weights(cfg, 18)
    P = {"a": O.random_tokens(cfg, 260, 1), "b": O.random_tokens(cfg, 90, 2), "c": O.random_tokens(cfg, 150, 3)}
    schedule = [[("a", 100), ("b", 1)], [("a", 1), ("b", 2), ("c", 130)], [("a", 65), ("b", 86)],
                [("a", 92), ("b", 1), ("c", 19)], [("a", 1)], [("a", 1), ("c", 1)]]
    for dtype in (torch.float32, torch.bfloat16):
        c, w = (cfg, W) if dtype == torch.float32 else (no_close_calls(cfg), calm(W))
        got = replay(engine(c, w, dev, dtype), P, schedule)
        for name, toks in P.items():
            assert rel_err(got[name], oracle(c, w, toks, f"m18{name}{dtype}")) < TOL[dtype], name


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


def wide_cfg():
    """sizes that the decode kernels' matrix-core forms hold: projections over row groups, wide latent tiles, per-head
    products"""
    return O.config([O.delta_layer(heads=4, kv_heads=2, dim=32, vdim=32, taps=4, rank=16, grank=16, mlp=O.moe(8, 2, 32, (4, 3))),
                     O.latent_layer(heads=9, dim=32, rot_dim=16, vdim=24, kv_rank=136, window=70, mlp=O.moe(4, 2, 32, (2, 1))),
                     O.pair_layer(heads=4, kv_heads=1, dim=32, vdim=16, dims=32, taps=2, rheads=2, rdim=32, rank=16,
                                  mlp=O.moe(4, 3, 64, None))], vocab=100, width=128, loop=(1, 3, 2))


def test_decode_kernels_at_their_sizes(dev):
    """long decoding beside other requests with the sizes of ``wide_cfg``, in both number formats"""
    cfg = no_close_calls(wide_cfg())
    W = calm(O.random_weights(cfg, 26))
    P = {"a": O.random_tokens(cfg, 150, 1), "b": O.random_tokens(cfg, 70, 2), "c": O.random_tokens(cfg, 25, 3)}
    schedule = [[("a", 100), ("b", 20)]] + [[("a", 1), ("b", 1), ("c", 1)]] * 25 + [[("a", 1), ("b", 1)]] * 25
    for dtype in (torch.float32, torch.bfloat16):
        got = replay(engine(cfg, W, dev, dtype), P, schedule)
        for name, toks in P.items():
            # (16-bit: the worst of 250 rows)
            err = rel_err(got[name], oracle(cfg, W, toks, "wide" + name))
            assert err < (TOL[dtype] if dtype == torch.float32 else 0.2), name


@pytest.mark.gpu
@pytest.mark.parametrize("sizes", ["narrow", "wide"])
def test_decode_graph_replays_equal_eager(sizes):
    """pure-decode steps replayed from a captured graph (padded rows on the scratch page and slot), with eager
    prompt steps and synchronisations between the replays"""
    if not torch.cuda.is_available():
        pytest.skip("no GPU")
    cfg = std_cfg() if sizes == "narrow" else wide_cfg()
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
        json.dump(public(cfg), f)
    save_file({k: v.to(torch.bfloat16).contiguous() for k, v in W.items()}, os.path.join(path, "model.safetensors"))


def test_checkpoint_registry_and_generate(tmp_path, dev):
    """a checkpoint folder is recognised by its architecture name and generates through the engine"""
    from ipex_llm_amd.models.registry import NativeCheckpointLM, native_architecture
    cfg = std_cfg()
    W = O.random_weights(cfg, 22)
    write_checkpoint(str(tmp_path / "m"), cfg, W)
    assert native_architecture(str(tmp_path / "m")) == "Lokolorn"
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
    from ipex_llm_amd.models import lokolorn as M
    cfg = std_cfg()
    spec = spec_of(cfg)
    assert M.tensor_shapes(spec) == O.tensor_shapes(cfg)
    assert M.random_model(spec, 0, torch.float32, "cpu").spec is spec


def test_reader_refuses_what_it_does_not_know():
    from ipex_llm_amd.models import lokolorn as M

    def broken(change, layer=None):
        cfg = public(O.config([layer or O.pair_layer(mlp=O.moe())], loop=None))
        change(cfg["layers"][0], cfg)
        with pytest.raises(ValueError):
            M.spec_from_config(cfg)
    broken(lambda L, c: L.update(type="something"))
    broken(lambda L, c: L["mixer"]["left"].update(kv_heads=3))
    broken(lambda L, c: L["mixer"]["left"]["rot"].update(dims=14))
    broken(lambda L, c: L["mixer"]["left"]["rot"].update(scaling=O.YARN))
    broken(lambda L, c: L["mlp"].update(kind="other"))
    broken(lambda L, c: L["mlp"]["router"]["groups"].update(count=4))
    broken(lambda L, c: L["mlp"]["router"].update(top=5))
    broken(lambda L, c: L["mixer"]["mask"].update(size=0), O.latent_layer())
    broken(lambda L, c: L["mixer"]["rot"].update(dims=4), O.latent_layer())
    broken(lambda L, c: L["mixer"].update(kv_heads=3), O.delta_layer())
    broken(lambda L, c: c.update(loop={"start": 0, "stop": 2, "times": 1}))
    broken(lambda L, c: c.update(loop={"start": 0, "stop": 1, "times": 0}))
    cfg = O.config([O.pair_layer(mlp=O.moe())], loop=None)
    W = O.random_weights(cfg)
    del W["l0.mix.right.w0"]
    with pytest.raises(KeyError):
        M.build(spec_of(cfg), W, torch.float32, "cpu")


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
