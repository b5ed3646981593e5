"""Plain float64 forms of a decoder whose sublayers are normed before and after
(Sudosun layout), written from the equations alone: whole sequences, explicit
loops over time, no cache, no batching.  Shares no code with the framework.

A model is ``(cfg, W)``: the configuration dictionary a checkpoint's
``config.json`` holds and ``name -> float64 tensor``.

Block:  x <- x + N1b(mixer(N1(x))),  x <- x + N2b(ff(N2(x)))  with the
statistics-free norm N(x) = tanh(alpha x) w + b.
"""
import math

import torch

F64 = torch.float64


# ------------------------------------------------------------------ small pieces
def dyn_tanh(x, alpha, w, b):
    return torch.tanh(alpha * x) * w + b


def norm(W, name, x):
    return dyn_tanh(x, W[name + ".alpha"], W[name], W[name + ".b"])


def unit_rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def sigmoid(z):
    return 1.0 / (1.0 + torch.exp(-z))


def silu(z):
    return z * sigmoid(z)


def softplus(z):
    return torch.logaddexp(z, torch.zeros_like(z))


def gelu_tanh(z):
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def causal_conv(u, w, b=None):
    """u [T, C], w [C, taps]: y_t = b + sum_j w[:, j] u_(t - taps + 1 + j), zeros before the start"""
    T, taps = u.shape[0], w.shape[1]
    y = torch.zeros_like(u)
    for t in range(T):
        for j in range(taps):
            s = t - taps + 1 + j
            if s >= 0:
                y[t] += w[:, j] * u[s]
    return y if b is None else y + b


# ------------------------------------------------------------------ attention
def rotary(rot):
    """(frequencies of the pairs, magnitude of cos and sin)"""
    dims = int(rot["dims"])
    base = float(rot["base"])
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


def turn_pairs(x, rot, positions):
    """x [T, heads, d]: value 2i is paired with 2i + 1 on the first rot.dims values"""
    dims = int(rot["dims"])
    f, mag = rotary(rot)
    a = positions.to(F64)[:, None] * f[None]
    c, s = (torch.cos(a) * mag)[:, None], (torch.sin(a) * mag)[:, None]
    out = x.clone()
    u, v = x[..., 0:dims:2], x[..., 1:dims:2]
    out[..., 0:dims:2] = u * c - v * s
    out[..., 1:dims:2] = v * c + u * s
    return out


def window_weights(s, sink):
    """softmax of the scores s with one more term exp(sink) in the denominator"""
    top = max(float(s.max()), float(sink))
    e = torch.exp(s - top)
    return e / (e.sum() + math.exp(float(sink) - top))


def window_attention(W, p, m, h, eps):
    T = h.shape[0]
    H, G, d, dv = int(m["heads"]), int(m["kv_heads"]), int(m["dim"]), int(m["vdim"])
    size = int(m["mask"]["size"])
    pos = torch.arange(T)
    q = (h @ W[p + "q"].T + W[p + "q.b"]).view(T, H, d)
    k = (h @ W[p + "k"].T + W[p + "k.b"]).view(T, G, d)
    v = (h @ W[p + "v"].T + W[p + "v.b"]).view(T, G, dv)
    q = turn_pairs(unit_rms(q, eps) * W[p + "q.norm"], m["rot"], pos)
    k = turn_pairs(unit_rms(k, eps) * W[p + "k.norm"], m["rot"], pos)
    gate = sigmoid(h @ W[p + "g"].T)                                   # [T, H]
    out = torch.zeros(T, H, dv, dtype=F64)
    for hd in range(H):
        g = hd // (H // G)
        for i in range(T):
            lo = max(0, i - size + 1)
            s = (k[lo:i + 1, g] @ q[i, hd]) * float(m["scale"]) * W[p + "temp"][hd]
            out[i, hd] = (window_weights(s, W[p + "sink"][hd]) @ v[lo:i + 1, g]) * gate[i, hd]
    return out.reshape(T, H * dv) @ W[p + "o"].T


# ------------------------------------------------------------------ recurrent mixers
def gated_linear_unit_scan(log_a, gu):
    """S_t = a_t S_(t-1) + sqrt(1 - a_t^2) gu_t per channel from S = 0; log_a, gu [T, C]"""
    S = torch.zeros(gu.shape[1], dtype=F64)
    out = torch.empty_like(gu)
    for t in range(gu.shape[0]):
        a = torch.exp(log_a[t])
        S = a * S + torch.sqrt(1.0 - a * a) * gu[t]
        out[t] = S
    return out


def griffin(W, p, m, h):
    T = h.shape[0]
    n, nb = int(m["width"]), int(m["blocks"])
    y = gelu_tanh(h @ W[p + "y"].T + W[p + "y.b"])
    u = causal_conv(h @ W[p + "x"].T + W[p + "x.b"], W[p + "conv"], W[p + "conv.b"])
    ub = u.view(T, nb, n // nb)
    r, i = torch.empty_like(ub), torch.empty_like(ub)
    for b in range(nb):
        r[:, b] = sigmoid(ub[:, b] @ W[p + "ra"][b].T + W[p + "ra.b"][b])
        i[:, b] = sigmoid(ub[:, b] @ W[p + "ri"][b].T + W[p + "ri.b"][b])
    log_a = -8.0 * r.reshape(T, n) * softplus(W[p + "lam"])
    S = gated_linear_unit_scan(log_a, i.reshape(T, n) * u)
    return (S * y) @ W[p + "o"].T


def parallel(W, p, m, h, eps):
    a = window_attention(W, p + "left.", m["left"], h, eps)
    b = griffin(W, p + "right.", m["right"], h)
    return 0.5 * (unit_rms(a, eps) * W[p + "left.out"] + unit_rms(b, eps) * W[p + "right.out"])


def lightning_scan(q, k, v, decay):
    """S_t = decay_h S_(t-1) + k_t v_t^T, o_t = S_t^T q_t; q, k [T, H, d], v [T, H, dv]"""
    T, H, d = q.shape
    dec = torch.tensor(decay, dtype=F64)[:, None, None]
    S = torch.zeros(H, d, v.shape[2], dtype=F64)
    o = torch.empty(T, H, v.shape[2], dtype=F64)
    for t in range(T):
        S = dec * S + k[t][:, :, None] * v[t][:, None, :]
        o[t] = (S * q[t][:, :, None]).sum(1)
    return o


def lightning(W, p, m, h, eps):
    T = h.shape[0]
    H, d, dv = int(m["heads"]), int(m["dim"]), int(m["vdim"])
    q = silu(h @ W[p + "q"].T).view(T, H, d)
    k = silu(h @ W[p + "k"].T).view(T, H, d)
    v = silu(h @ W[p + "v"].T).view(T, H, dv)
    o = lightning_scan(q, k, v, [float(x) for x in m["decay"]]).reshape(T, H * dv)
    o = unit_rms(o, eps) * W[p + "norm"] * sigmoid(h @ W[p + "g"].T)
    return o @ W[p + "o"].T


def unit(x):
    return x / torch.sqrt((x * x).sum(-1, keepdim=True) + 1e-6)


def delta_scan(q, k, v, g, beta):
    """per head S <- g S; u = beta (v - S^T k); S <- S + k u^T; o = S^T q; q, k [T, K, d] (head h reads key head
    h // (H / K)), v [T, H, dv], g, beta [T, H]"""
    T, H, dv = v.shape
    rep = H // q.shape[1]
    S = torch.zeros(H, q.shape[2], dv, dtype=F64)
    o = torch.empty(T, H, dv, dtype=F64)
    for t in range(T):
        for h in range(H):
            kt, qt = k[t, h // rep], q[t, h // rep]
            S[h] = g[t, h] * S[h]
            u = beta[t, h] * (v[t, h] - S[h].T @ kt)
            S[h] = S[h] + kt[:, None] * u[None]
            o[t, h] = S[h].T @ qt
    return o


def delta(W, p, m, h, eps):
    T = h.shape[0]
    H, K, d, dv = int(m["heads"]), int(m["kv_heads"]), int(m["dim"]), int(m["vdim"])
    q = silu(causal_conv(h @ W[p + "q"].T, W[p + "q.conv"])).view(T, K, d)
    k = silu(causal_conv(h @ W[p + "k"].T, W[p + "k.conv"])).view(T, K, d)
    v = silu(causal_conv(h @ W[p + "v"].T, W[p + "v.conv"])).view(T, H, dv)
    beta = sigmoid(h @ W[p + "b"].T)
    g = torch.exp(-torch.exp(W[p + "A_log"]) * softplus(h @ W[p + "a"].T + W[p + "dt_bias"]))
    o = delta_scan(unit(q) * d ** -0.5, unit(k), v, g, beta)
    o = unit_rms(o, eps) * W[p + "norm"]
    return (o.reshape(T, H * dv) * silu(h @ W[p + "g"].T)) @ W[p + "o"].T


# ------------------------------------------------------------------ feed-forward
def dense(W, p, m, h):
    lim = float(m["limit"])
    g = torch.clamp(h @ W[p + "gate"].T, max=lim)
    u = torch.clamp(h @ W[p + "up"].T, min=-lim, max=lim)
    return (g * sigmoid(1.702 * g) * (u + 1.0)) @ W[p + "down"].T


def route(z, correction, top, groups):
    """one token's router logits -> [(expert, weight)]: softmax over all, the largest corrected scores of the groups
    with the largest best corrected score win, the weights are the uncorrected scores"""
    s = torch.softmax(z, 0)
    choice = [float(a) for a in s + correction]
    n = len(choice)
    allowed = range(n)
    if groups:
        size = n // int(groups["count"])
        best = [max(choice[g * size:(g + 1) * size]) for g in range(int(groups["count"]))]
        kept = sorted(range(len(best)), key=lambda g: (-best[g], g))[:int(groups["keep"])]
        allowed = [e for e in range(n) if e // size in kept]
    order = sorted(allowed, key=lambda e: (-choice[e], e))[:top]
    return [(e, s[e]) for e in order]


def experts(W, p, m, h):
    r = m["router"]
    E, top = int(r["experts"]), int(r["top"])
    z = h @ W[p + "router"].T
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e, w in route(z[t], W[p + "correction"], top, r.get("groups")):
            if e >= E:
                out[t] += w * h[t]
            else:
                q = f"{p}e{e}."
                y = silu(W[q + "gate"] @ h[t]) * (W[q + "up"] @ h[t])
                out[t] += w * (W[q + "down"] @ y)
    return out


# ------------------------------------------------------------------ model
def forward(cfg, W, tokens, layers_out=None):
    """logits f64 [T, vocab] of one sequence run whole"""
    eps = float(cfg["norm"]["eps"])
    x = W["embed"][torch.as_tensor(tokens, dtype=torch.long)].clone()
    for i, L in enumerate(cfg["layers"]):
        p, m = f"l{i}.", L["mixer"]
        h = norm(W, p + "norm1", x)
        if L["type"] == "lightning":
            y = lightning(W, p + "mix.", m, h, eps)
        elif L["type"] == "parallel":
            y = parallel(W, p + "mix.", m, h, eps)
        elif L["type"] == "delta":
            y = delta(W, p + "mix.", m, h, eps)
        else:
            raise ValueError(L["type"])
        x = x + norm(W, p + "norm1b", y)
        if L.get("mlp") is not None:
            h = norm(W, p + "norm2", x)
            ff = dense if L["mlp"]["kind"] == "dense" else experts
            x = x + norm(W, p + "norm2b", ff(W, p + "mlp.", L["mlp"], h))
        if layers_out is not None:
            layers_out.append(x.clone())
    return (norm(W, "final.norm", x) @ W["embed"].T) * float(cfg["logit_scale"])


def greedy(cfg, W, prompt, n):
    toks = list(prompt)
    for _ in range(n):
        toks.append(int(forward(cfg, W, toks)[-1].argmax()))
    return toks[len(prompt):]


# ------------------------------------------------------------------ configurations and weights
def dense_ff(ff=20, limit=0.8):
    return {"kind": "dense", "ff": ff, "limit": limit}


def moe(experts=5, identity=1, top=2, ff=12, groups=(3, 2)):
    r = {"experts": experts, "identity": identity, "top": top}
    if groups:
        r["groups"] = {"count": groups[0], "keep": groups[1]}
    return {"kind": "moe", "expert": {"ff": ff}, "router": r}


def lightning_layer(heads=3, dim=6, vdim=10, decay=None, mlp=None):
    decay = decay or [math.exp(-0.7 * 0.4 ** i) for i in range(heads)]
    return {"type": "lightning", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "decay": decay}, "mlp": mlp}


def delta_layer(heads=4, kv_heads=2, dim=12, vdim=10, taps=3, mlp=None):
    return {"type": "delta", "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": taps}, "mlp": mlp}


YARN = {"factor": 4.0, "original": 64, "fast": 8.0, "slow": 1.0}


def pair_layer(heads=4, kv_heads=2, dim=12, vdim=10, window=9, dims=8, base=3000.0, scaling=YARN, scale=0.3, width=24,
               blocks=3, taps=2, mlp=None):
    left = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "mask": {"size": window}, "scale": scale,
            "rot": {"dims": dims, "base": base, "scaling": scaling}}
    if scaling is None:
        del left["rot"]["scaling"]
    return {"type": "parallel", "mixer": {"left": left, "right": {"width": width, "blocks": blocks, "conv": taps}}, "mlp": mlp}


def config(layers, vocab=89, width=40, eps=1e-5, logit_scale=0.7):
    return {"architecture": "Sudosun", "vocab": vocab, "width": width, "norm": {"eps": eps}, "layers": layers,
            "logit_scale": logit_scale}


def tensor_shapes(cfg):
    Wd, V = int(cfg["width"]), int(cfg["vocab"])
    out = {"embed": (V, Wd)}

    def add_norm(name):
        out.update({name: (Wd,), name + ".b": (Wd,), name + ".alpha": ()})
    for i, L in enumerate(cfg["layers"]):
        p, m = f"l{i}.", L["mixer"]
        add_norm(p + "norm1")
        add_norm(p + "norm1b")
        q = p + "mix."
        if L["type"] == "lightning":
            H, d, dv = m["heads"], m["dim"], m["vdim"]
            out.update({q + "q": (H * d, Wd), q + "k": (H * d, Wd), q + "v": (H * dv, Wd), q + "g": (H * dv, Wd),
                        q + "o": (Wd, H * dv), q + "norm": (H * dv,)})
        elif L["type"] == "delta":
            H, K, d, dv, taps = m["heads"], m["kv_heads"], m["dim"], m["vdim"], m["conv"]
            out.update({q + "q": (K * d, Wd), q + "k": (K * d, Wd), q + "v": (H * dv, Wd), q + "q.conv": (K * d, taps),
                        q + "k.conv": (K * d, taps), q + "v.conv": (H * dv, taps), q + "b": (H, Wd), q + "a": (H, Wd),
                        q + "A_log": (H,), q + "dt_bias": (H,), q + "norm": (dv,), q + "g": (H * dv, Wd),
                        q + "o": (Wd, H * dv)})
        else:
            a, b = m["left"], m["right"]
            H, G, d, dv = a["heads"], a["kv_heads"], a["dim"], a["vdim"]
            s = q + "left."
            out.update({s + "q": (H * d, Wd), s + "q.b": (H * d,), s + "k": (G * d, Wd), s + "k.b": (G * d,),
                        s + "v": (G * dv, Wd), s + "v.b": (G * dv,), s + "q.norm": (d,), s + "k.norm": (d,),
                        s + "temp": (H,), s + "sink": (H,), s + "g": (H, Wd), s + "o": (Wd, H * dv), s + "out": (Wd,)})
            n, nb, taps = b["width"], b["blocks"], b["conv"]
            c = n // nb
            s = q + "right."
            out.update({s + "y": (n, Wd), s + "y.b": (n,), s + "x": (n, Wd), s + "x.b": (n,), s + "conv": (n, taps),
                        s + "conv.b": (n,), s + "ra": (nb, c, c), s + "ra.b": (nb, c), s + "ri": (nb, c, c),
                        s + "ri.b": (nb, c), s + "lam": (n,), s + "o": (Wd, n), s + "out": (Wd,)})
        if L.get("mlp") is not None:
            add_norm(p + "norm2")
            add_norm(p + "norm2b")
            f, q = L["mlp"], p + "mlp."
            if f["kind"] == "dense":
                out.update({q + "gate": (f["ff"], Wd), q + "up": (f["ff"], Wd), q + "down": (Wd, f["ff"])})
            else:
                ff, E = f["expert"]["ff"], f["router"]["experts"]
                for e in range(E):
                    out.update({f"{q}e{e}.gate": (ff, Wd), f"{q}e{e}.up": (ff, Wd), f"{q}e{e}.down": (Wd, ff)})
                n = E + f["router"].get("identity", 0)
                out.update({q + "router": (n, Wd), q + "correction": (n,)})
    add_norm("final.norm")
    return out


def random_weights(cfg, seed=0):
    """bf16-representable float64 weights"""
    g = torch.Generator().manual_seed(seed)
    W = {}
    for name, shape in tensor_shapes(cfg).items():
        r = torch.randn(shape, generator=g)
        if name.endswith(".alpha"):
            w = 0.6 + 0.1 * r
        elif name.endswith(("norm1", "norm2", "norm1b", "norm2b", ".norm", ".out", ".temp")):
            w = 1.0 + 0.2 * r
        elif name.endswith("conv"):
            w = 0.6 * r
        elif name.endswith("correction"):
            w = 0.2 * r - 0.1                       # some choice scores are negative
        elif name.endswith("lam"):
            w = -2.0 + r                            # decays between slow and fast
        elif name.endswith(("A_log", "dt_bias")):
            w = -1.5 + 0.7 * r
        elif name.endswith(("ra", "ri")):
            w = r * shape[2] ** -0.5
        elif name.endswith(("router", "embed")):
            w = r
        elif len(shape) == 1 or name.endswith(("ra.b", "ri.b")):       # biases, sinks
            w = 0.3 * r
        else:
            w = r * 1.5 * shape[1] ** -0.5
        W[name] = w.to(torch.bfloat16).to(F64)
    return W


def random_tokens(cfg, n, seed=0):
    g = torch.Generator().manual_seed(1000 + seed)
    return torch.randint(0, int(cfg["vocab"]), (n,), generator=g).tolist()
