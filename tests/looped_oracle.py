"""Plain float64 forms of a pre-norm decoder whose middle layers run several
times over (Lokolorn layout), written from the equations alone: whole
sequences, explicit loops over time, no cache, no batching.  Shares no code
with the framework.

A model is ``(cfg, W)``: the configuration dictionary a checkpoint's
``config.json`` holds and ``name -> float64 tensor``.

Layer:  x <- x + ls1 * mixer(N1(x)),  x <- x + ls2 * ff(N2(x)),
N(x) = x / sqrt(mean x^2 + eps) * (1 + w).
Loop:   in front of every pass over layers start .. stop - 1
        x <- W_in [x; embedding].
"""
import math

import torch

F64 = torch.float64


# ------------------------------------------------------------------ small pieces
def unit_rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def norm(x, w, eps):
    return unit_rms(x, eps) * (1.0 + w)


def sigmoid(z):
    return 1.0 / (1.0 + torch.exp(-z))


def silu(z):
    return z * sigmoid(z)


def softplus(z):
    return torch.logaddexp(z, torch.zeros_like(z))


def unit(x):
    return x / torch.sqrt((x * x).sum(-1, keepdim=True) + 1e-6)


def causal_conv(u, w):
    """u [T, C], w [C, taps]: y_t = sum_j w[:, j] u_(t - taps + 1 + j), zeros before the start"""
    T, taps = u.shape[0], w.shape[1]
    y = torch.zeros_like(u)
    for t in range(T):
        for j in range(taps):
            s = t - taps + 1 + j
            if s >= 0:
                y[t] += w[:, j] * u[s]
    return y


# ------------------------------------------------------------------ rotary positions
def rotary(rot):
    """(frequencies of the pairs, magnitude of cos and sin)"""
    dims, base = int(rot["dims"]), float(rot["base"])
    f = [base ** (-2.0 * i / dims) for i in range(dims // 2)]
    sc = rot.get("scaling")
    if not sc:
        return torch.tensor(f, dtype=F64), 1.0
    factor = float(sc["factor"])

    def turns(t):
        return dims * math.log(float(sc["original"]) / (2.0 * math.pi * float(t))) / (2.0 * math.log(base))
    lo = max(math.floor(turns(sc["fast"])), 0)
    hi = min(math.ceil(turns(sc["slow"])), dims - 1)
    out = []
    for i, fi in enumerate(f):
        r = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        out.append(fi / factor * r + fi * (1.0 - r))
    return torch.tensor(out, dtype=F64), 0.1 * math.log(factor) + 1.0


def _angles(rot, positions):
    f, mag = rotary(rot)
    a = positions.to(F64)[:, None] * f[None]
    return (torch.cos(a) * mag)[:, None], (torch.sin(a) * mag)[:, None]


def turn_pairs(x, rot, positions):
    """x [T, heads, d]: value 2i is paired with 2i + 1 on the first rot.dims values"""
    dims = int(rot["dims"])
    c, s = _angles(rot, positions)
    out = x.clone()
    u, v = x[..., 0:dims:2], x[..., 1:dims:2]
    out[..., 0:dims:2] = u * c - v * s
    out[..., 1:dims:2] = v * c + u * s
    return out


def turn_half(x, rot, positions):
    """x [T, heads, d]: value i is paired with i + dims / 2 on the first rot.dims values"""
    dims = int(rot["dims"])
    h = dims // 2
    c, s = _angles(rot, positions)
    out = x.clone()
    u, v = x[..., :h], x[..., h:dims]
    out[..., :h] = u * c - v * s
    out[..., h:dims] = v * c + u * s
    return out


# ------------------------------------------------------------------ attention
def sink_weights(s, sink=None):
    """softmax of the scores s; with a sink one more term exp(sink) in the denominator"""
    top = float(s.max()) if sink is None else max(float(s.max()), float(sink))
    e = torch.exp(s - top)
    den = e.sum()
    if sink is not None:
        den = den + math.exp(float(sink) - top)
    return e / den


def latent_attention(W, p, m, h, eps):
    T = h.shape[0]
    H, d, dr, dv, r = int(m["heads"]), int(m["dim"]), int(m["rot_dim"]), int(m["vdim"]), int(m["kv_rank"])
    size, scale = int(m["mask"]["size"]), float(m["scale"])
    pos = torch.arange(T)
    q = (h @ W[p + "q"].T).view(T, H, d + dr)
    qn, qr = q[..., :d], turn_pairs(q[..., d:], m["rot"], pos)
    y = h @ W[p + "dkv"].T
    c = unit_rms(y[:, :r], eps) * W[p + "dkv.norm"]
    kr = turn_pairs(y[:, None, r:], m["rot"], pos)[:, 0]
    k = (c @ W[p + "uk"].T).view(T, H, d)
    v = (c @ W[p + "uv"].T).view(T, H, dv)
    out = torch.zeros(T, H, dv, dtype=F64)
    for hd in range(H):
        for i in range(T):
            lo = max(0, i - size + 1)
            s = (k[lo:i + 1, hd] @ qn[i, hd] + kr[lo:i + 1] @ qr[i, hd]) * scale
            out[i, hd] = sink_weights(s, W[p + "sink"][hd]) @ v[lo:i + 1, hd]
    return out.reshape(T, H * dv) @ W[p + "o"].T


def causal_attention(W, p, m, h, eps):
    T = h.shape[0]
    H, G, d, dv = int(m["heads"]), int(m["kv_heads"]), int(m["dim"]), int(m["vdim"])
    pos = torch.arange(T)
    q, k, v = (causal_conv(h @ W[p + n].T + W[p + n + ".b"], W[p + n + ".conv"]) for n in "qkv")
    q = unit_rms(turn_half(q.view(T, H, d), m["rot"], pos), eps)
    k = unit_rms(turn_half(k.view(T, G, d), m["rot"], pos), eps)
    v = v.view(T, G, dv)
    out = torch.zeros(T, H, dv, dtype=F64)
    for hd in range(H):
        g = hd // (H // G)
        for i in range(T):
            out[i, hd] = sink_weights((k[:i + 1, g] @ q[i, hd]) * float(m["scale"])) @ v[:i + 1, g]
    return out.reshape(T, H * dv) @ W[p + "o"].T + W[p + "o.b"]


# ------------------------------------------------------------------ recurrent mixers
def bonus_scan(r, k, v, w, u):
    """per head o_t = (S + diag(u) k_t v_t^T)^T r_t, then S <- diag(w_t) S + k_t v_t^T; r, k, w [T, H, d], v [T, H, dv],
    u [H, d]"""
    T, H, d = r.shape
    S = torch.zeros(H, d, v.shape[2], dtype=F64)
    o = torch.empty(T, H, v.shape[2], dtype=F64)
    for t in range(T):
        kv = k[t][:, :, None] * v[t][:, None, :]
        o[t] = ((S + u[:, :, None] * kv) * r[t][:, :, None]).sum(1)
        S = w[t][:, :, None] * S + kv
    return o


def shifted(h):
    """every token's predecessor, zeros in front of the first"""
    return torch.cat([torch.zeros_like(h[:1]), h[:-1]], 0)


def time_mix(W, p, m, h, eps):
    T = h.shape[0]
    H, d = int(m["heads"]), int(m["dim"])
    prev = shifted(h)
    mix = {n: h + (prev - h) * W[p + "mu." + n] for n in "rkvgw"}
    r, k, v = ((mix[n] @ W[p + n].T).view(T, H, d) for n in "rkv")
    gate = silu(mix["g"] @ W[p + "g"].T)
    w = torch.exp(-torch.exp(torch.tanh(mix["w"] @ W[p + "w1"].T) @ W[p + "w2"].T + W[p + "w0"])).view(T, H, d)
    o = unit_rms(bonus_scan(r, k, v, w, W[p + "u"]), eps).reshape(T, H * d)
    return (o * W[p + "norm"] * gate) @ W[p + "o"].T


def parallel(W, p, m, h, eps):
    a = causal_attention(W, p + "left.", m["left"], h, eps)
    b = time_mix(W, p + "right.", m["right"], h, eps)
    return float(m["left_scale"]) * a + float(m["right_scale"]) * b


def channel_delta_scan(q, k, v, g, beta):
    """per head S <- diag(g) S; u = beta (v - S^T k); S <- S + k u^T; o = S^T q; q, k [T, K, d] (head h reads key head
    h // (H / K)), v [T, H, dv], g [T, H, d], beta [T, H]"""
    T, H, dv = v.shape
    rep = H // q.shape[1]
    S = torch.zeros(H, q.shape[2], dv, dtype=F64)
    o = torch.empty(T, H, dv, dtype=F64)
    for t in range(T):
        kt, qt = k[t].repeat_interleave(rep, 0), q[t].repeat_interleave(rep, 0)
        S = g[t][:, :, None] * S
        u = beta[t][:, None] * (v[t] - (S * kt[:, :, None]).sum(1))
        S = S + kt[:, :, None] * u[:, None, :]
        o[t] = (S * qt[:, :, None]).sum(1)
    return o


def channel_delta(W, p, m, h, eps):
    T = h.shape[0]
    H, K, d, dv = int(m["heads"]), int(m["kv_heads"]), int(m["dim"]), int(m["vdim"])
    q, k, v = (silu(causal_conv(h @ W[p + n].T, W[p + n + ".conv"])) for n in "qkv")
    beta = sigmoid(h @ W[p + "b"].T)
    z = (h @ W[p + "a1"].T) @ W[p + "a2"].T + W[p + "dt_bias"]
    g = torch.exp(-torch.exp(W[p + "A_log"])[:, None] * softplus(z).view(T, H, d))
    o = channel_delta_scan(unit(q.view(T, K, d)) * d ** -0.5, unit(k.view(T, K, d)), v.view(T, H, dv), g, beta)
    o = (unit_rms(o, eps) * W[p + "norm"]).reshape(T, H * dv)
    return (o * sigmoid((h @ W[p + "g1"].T) @ W[p + "g2"].T)) @ W[p + "o"].T


# ------------------------------------------------------------------ experts
def route(z, correction, top, groups, scale):
    """one token's router logits -> [(expert, weight)]: sigmoid scores; the largest corrected scores inside the groups
    whose two largest corrected scores have the largest sum win; weights: the plain scores over their sum, times scale"""
    s = sigmoid(z)
    choice = [float(a) for a in s + correction]
    n = len(choice)
    allowed = list(range(n))
    if groups:
        size = n // int(groups["count"])
        best = [sum(sorted(choice[g * size:(g + 1) * size])[-2:]) for g in range(int(groups["count"]))]
        kept = sorted(range(len(best)), key=lambda g: (-best[g], g))[:int(groups["keep"])]
        allowed = [e for e in range(n) if e // size in kept]
    order = sorted(allowed, key=lambda e: (-choice[e], e))[:top]
    total = sum(s[e] for e in order) + 1e-20
    return [(e, s[e] / total * scale) for e in order]


def experts(W, p, m, h):
    r = m["router"]
    z = h @ W[p + "router"].T
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e, w in route(z[t], W[p + "correction"], int(r["top"]), r.get("groups"), float(r["scale"])):
            q = f"{p}e{e}."
            y = silu(W[q + "gate"] @ h[t]) * (W[q + "up"] @ h[t])
            out[t] += w * (W[q + "down"] @ y)
    return out


# ------------------------------------------------------------------ model
def runs(cfg):
    """the layers in the order they run: [(layer, first of a pass)]"""
    n = len(cfg["layers"])
    lp = cfg.get("loop")
    if not lp:
        return [(i, False) for i in range(n)]
    a, b = int(lp["start"]), int(lp["stop"])
    body = [(i, i == a) for i in range(a, b)] * int(lp["times"])
    return [(i, False) for i in range(a)] + body + [(i, False) for i in range(b, n)]


MIXERS = {"latent_attention": latent_attention, "parallel": parallel, "channel_delta": channel_delta}


def forward(cfg, W, tokens, layers_out=None):
    """logits f64 [T, vocab] of one sequence run whole"""
    eps = float(cfg["norm"]["eps"])
    x0 = W["embed"][torch.as_tensor(tokens, dtype=torch.long)]
    x = x0.clone()
    for i, first in runs(cfg):
        L, p = cfg["layers"][i], f"l{i}."
        if first:
            x = torch.cat([x, x0], -1) @ W["loop.in"].T
        h = norm(x, W[p + "norm1"], eps)
        x = x + W[p + "ls1"] * MIXERS[L["type"]](W, p + "mix.", L["mixer"], h, eps)
        if L.get("mlp") is not None:
            h = norm(x, W[p + "norm2"], eps)
            x = x + W[p + "ls2"] * experts(W, p + "mlp.", L["mlp"], h)
        if layers_out is not None:
            layers_out.append(x.clone())
    return norm(x, W["final.norm"], eps) @ W["head"].T


def greedy(cfg, W, prompt, n):
    toks = list(prompt)
    for _ in range(n):
        toks.append(int(forward(cfg, W, toks)[-1].argmax()))
    return toks[len(prompt):]


# ------------------------------------------------------------------ configurations and weights
def moe(experts=6, top=2, ff=12, groups=(3, 2), scale=1.7):
    r = {"experts": experts, "top": top, "scale": scale}
    if groups:
        r["groups"] = {"count": groups[0], "keep": groups[1]}
    return {"kind": "moe", "expert": {"ff": ff}, "router": r}


def delta_layer(heads=4, kv_heads=2, dim=12, vdim=10, taps=3, rank=5, grank=7, mlp=None):
    """``rank`` / ``grank``: of the decay's and the gate's low-rank projections (read from the tensors' shapes)"""
    return {"type": "channel_delta", "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": taps},
            "mlp": mlp, "_rank": rank, "_grank": grank}


YARN = {"factor": 4.0, "original": 64, "fast": 8.0, "slow": 1.0}


def latent_layer(heads=3, dim=10, rot_dim=8, vdim=6, kv_rank=20, window=9, base=3000.0, scaling=YARN, scale=0.3, mlp=None):
    rot = {"dims": rot_dim, "base": base}
    if scaling is not None:
        rot["scaling"] = dict(scaling)
    return {"type": "latent_attention", "mixer": {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim,
            "kv_rank": kv_rank, "mask": {"size": window}, "rot": rot, "scale": scale}, "mlp": mlp}


def pair_layer(heads=4, kv_heads=2, dim=12, vdim=10, dims=8, base=900.0, scale=0.3, taps=3, rheads=3, rdim=6, rank=5,
               scales=(0.7, 0.4), mlp=None):
    left = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": taps, "scale": scale,
            "rot": {"dims": dims, "base": base}}
    return {"type": "parallel", "mixer": {"left": left, "left_scale": scales[0], "right": {"heads": rheads, "dim": rdim},
            "right_scale": scales[1]}, "mlp": mlp, "_rank": rank}


def config(layers, vocab=89, width=40, eps=1e-5, loop=(1, 3, 2)):
    cfg = {"architecture": "Lokolorn", "vocab": vocab, "width": width, "norm": {"eps": eps}, "layers": layers}
    if loop:
        cfg["loop"] = {"start": loop[0], "stop": loop[1], "times": loop[2]}
    return cfg


def tensor_shapes(cfg):
    Wd, V = int(cfg["width"]), int(cfg["vocab"])
    out = {"embed": (V, Wd), "head": (V, Wd), "final.norm": (Wd,)}
    if cfg.get("loop"):
        out["loop.in"] = (Wd, 2 * Wd)
    for i, L in enumerate(cfg["layers"]):
        p, m = f"l{i}.", L["mixer"]
        out.update({p + "norm1": (Wd,), p + "ls1": (Wd,)})
        q = p + "mix."
        if L["type"] == "channel_delta":
            H, K, d, dv, taps = m["heads"], m["kv_heads"], m["dim"], m["vdim"], m["conv"]
            R, RG = L.get("_rank", 5), L.get("_grank", 7)
            out.update({q + "q": (K * d, Wd), q + "k": (K * d, Wd), q + "v": (H * dv, Wd), q + "q.conv": (K * d, taps),
                        q + "k.conv": (K * d, taps), q + "v.conv": (H * dv, taps), q + "b": (H, Wd), q + "A_log": (H,),
                        q + "norm": (dv,), q + "a1": (R, Wd), q + "a2": (H * d, R), q + "dt_bias": (H * d,),
                        q + "g1": (RG, Wd), q + "g2": (H * dv, RG), q + "o": (Wd, H * dv)})
        elif L["type"] == "latent_attention":
            H, d, dr, dv, r = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
            out.update({q + "q": (H * (d + dr), Wd), q + "dkv": (r + dr, Wd), q + "dkv.norm": (r,), q + "uk": (H * d, r),
                        q + "uv": (H * dv, r), q + "sink": (H,), q + "o": (Wd, H * dv)})
        else:
            a, b, R = m["left"], m["right"], L.get("_rank", 5)
            s = q + "left."
            for n, c in (("q", a["heads"] * a["dim"]), ("k", a["kv_heads"] * a["dim"]), ("v", a["kv_heads"] * a["vdim"])):
                out.update({s + n: (c, Wd), s + n + ".b": (c,), s + n + ".conv": (c, a["conv"])})
            out.update({s + "o": (Wd, a["heads"] * a["vdim"]), s + "o.b": (Wd,)})
            n, s = b["heads"] * b["dim"], q + "right."
            for c in "rkvgw":
                out[s + "mu." + c] = (Wd,)
            for c in "rkvg":
                out[s + c] = (n, Wd)
            out.update({s + "w1": (R, Wd), s + "w2": (n, R), s + "w0": (n,), s + "u": (b["heads"], b["dim"]),
                        s + "norm": (n,), s + "o": (Wd, n)})
        f, q = L.get("mlp"), p + "mlp."
        if f is not None:
            out.update({p + "norm2": (Wd,), p + "ls2": (Wd,)})
            ff, E = f["expert"]["ff"], f["router"]["experts"]
            for e in range(E):
                out.update({f"{q}e{e}.gate": (ff, Wd), f"{q}e{e}.up": (ff, Wd), f"{q}e{e}.down": (Wd, ff)})
            out.update({q + "router": (E, Wd), q + "correction": (E,)})
    return out


def random_weights(cfg, seed=0):
    """bf16-representable float64 weights"""
    g = torch.Generator().manual_seed(seed)
    W = {}
    for name, shape in tensor_shapes(cfg).items():
        r = torch.randn(shape, generator=g)
        if name.endswith(("norm1", "norm2", "final.norm")):
            w = 0.2 * r                             # stored around zero
        elif name.endswith(".norm"):
            w = 1.0 + 0.2 * r
        elif name.endswith((".ls1", ".ls2")):
            w = 0.8 + 0.2 * r
        elif ".mu." in name:
            w = 0.5 + 0.3 * r
        elif name.endswith("conv"):
            w = 0.6 * r
        elif name.endswith("correction"):
            w = 0.2 * r - 0.6                       # many choice scores are negative
        elif name.endswith(("A_log", "dt_bias", "w0")):
            w = -1.5 + 0.7 * r
        elif name.endswith((".router", "embed", ".u")):
            w = r
        elif len(shape) == 1:                       # biases, sinks
            w = 0.3 * r
        elif name == "loop.in":
            w = r * shape[1] ** -0.5
        else:
            w = r * 1.5 * shape[1] ** -0.5
        W[name] = w.to(torch.bfloat16).to(F64)
    return W


def random_tokens(cfg, n, seed=0):
    g = torch.Generator().manual_seed(1000 + seed)
    return torch.randint(0, int(cfg["vocab"]), (n,), generator=g).tolist()
