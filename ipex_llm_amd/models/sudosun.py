"""Sudosun: a decoder whose sublayers are normed before and after with
statistics-free tanh norms, and whose layers mix lightning attention, a gated
delta rule, and a sliding-window attention with a sink beside a real-gated
linear recurrent unit; clamped dense feed-forwards and experts routed in groups
with identity experts.  Read from its own checkpoint layout.

A checkpoint folder holds ``config.json`` (``"architecture": "Sudosun"``) and
``model.safetensors`` (bf16 weights, linear weights stored [out, in]).  The
configuration lists the layers in order; each entry names its mixer type
(``lightning``, ``parallel``, ``delta``), the mixer's sizes and its
feed-forward (``dense``, ``moe`` or none).  Tensor names: ``embed`` (also the
head), ``l<i>.norm1`` / ``norm1b`` / ``norm2`` / ``norm2b`` (+ ``.alpha``,
``.b``), ``l<i>.mix.<name>``, ``l<i>.mlp.<name>``, ``final.norm``.  Every size
and constant comes from the configuration; the building blocks are the generic
ones of ``models/hybrid.py``:

* ``lightning``  -> ``LightningAttention`` (``q`` ``k`` ``v`` ``g`` ``norm`` ``o``)
* ``delta``      -> ``GatedDelta`` (``q`` ``k`` ``v`` + ``.conv``, ``a`` ``b`` ``A_log`` ``dt_bias``, ``g`` ``norm`` ``o``)
* ``parallel``   -> ``SideBySide`` of ``MaskedAttention`` (``left``: biased projections, RMS norm per head,
                    neighbouring rotary pairs with YaRN scaling, a number per head on the scores, a window of
                    ``mask.size``, a sink and an output gate per head) and ``RealGatedLRU`` (``right``)
* feed-forward   -> ``DenseFF`` with the clamped unit, or ``ScoredMoE``
"""
from __future__ import annotations

import json
import os
from typing import Dict, Optional

import torch

from .hybrid import (DenseFF, DenseFFSpec, DynTanh, ExpertSpec, GatedDelta, GatedDeltaSpec, HybridCausalLM, HybridSpec,
                     LayerSpec, LightningAttention, LightningSpec, MaskedAttention, MaskedAttentionSpec, MaskSpec, MoESpec,
                     RealGatedLRU, RealGatedLRUSpec, RotarySpec, SandwichLayer, ScoredMoE, SideBySide, SideBySideSpec)

ARCHITECTURE = "Sudosun"


def _heads(m: dict, i: int):
    H, G = int(m["heads"]), int(m.get("kv_heads", m["heads"]))
    if H < 1 or G < 1 or H % G:
        raise ValueError(f"layer {i}: heads must be a multiple of kv_heads")
    return H, G


def _attention_spec(m: dict, i: int) -> MaskedAttentionSpec:
    H, G = _heads(m, i)
    rot, rs = m.get("rot"), None
    if rot and int(rot.get("dims", 0)):
        rs = RotarySpec(int(rot["dims"]), float(rot["base"]), rot.get("scaling") or None, "pairs")
        if rs.dims > int(m["dim"]) or rs.dims % 2:
            raise ValueError(f"layer {i}: rot.dims must be even and at most dim")
    mask = MaskSpec("window", int(m["mask"]["size"]))
    if mask.size < 1:
        raise ValueError(f"layer {i}: mask.size must be at least 1")
    return MaskedAttentionSpec(heads=H, kv_heads=G, dim=int(m["dim"]), vdim=int(m["vdim"]), scale=float(m["scale"]),
                               rot=rs, mask=mask, qk_norm="head", bias=True, sink=True, out_gate=True, gate="head",
                               temp=True)


def _mlp_spec(m: Optional[dict], i: int):
    if m is None:
        return None
    kind = m.get("kind", "dense")
    if kind == "dense":
        limit = m.get("limit")
        return DenseFFSpec(int(m["ff"]), act="clamp", limit=float("inf") if limit is None else float(limit))
    if kind != "moe":
        raise ValueError(f"layer {i}: unknown feed-forward kind {kind!r}")
    r = m["router"]
    E, ident, top = int(r["experts"]), int(r.get("identity") or 0), int(r["top"])
    g = r.get("groups") or {"count": 1, "keep": 1}
    count, keep = int(g["count"]), int(g["keep"])
    if count < 1 or (E + ident) % count or not 1 <= keep <= count or not 1 <= top <= keep * ((E + ident) // count):
        raise ValueError(f"layer {i}: router.groups must split the router's outputs evenly and leave at least top of them")
    return MoESpec(experts=E, top=top, expert=ExpertSpec(ff=int(m["expert"]["ff"])), identity=ident, groups=count, keep=keep)


def spec_from_config(cfg: dict) -> HybridSpec:
    layers = []
    for i, L in enumerate(cfg["layers"]):
        m, kind = L["mixer"], L["type"]
        if kind == "lightning":
            mixer = LightningSpec(heads=int(m["heads"]), dim=int(m["dim"]), vdim=int(m["vdim"]),
                                  decay=[float(v) for v in m["decay"]])
            if len(mixer.decay) != mixer.heads:
                raise ValueError(f"layer {i}: one decay per head")
            name = "lightning"
        elif kind == "delta":
            H, K = _heads(m, i)
            mixer = GatedDeltaSpec(heads=H, kv_heads=K, dim=int(m["dim"]), vdim=int(m["vdim"]), taps=int(m["conv"]))
            name = "gated_delta"
        elif kind == "parallel":
            r = m["right"]
            right = RealGatedLRUSpec(width=int(r["width"]), blocks=int(r["blocks"]), taps=int(r["conv"]))
            if right.blocks < 1 or right.width % right.blocks:
                raise ValueError(f"layer {i}: width must split into equal blocks")
            mixer, name = SideBySideSpec(_attention_spec(m["left"], i), right, right_kind="real_gated_lru"), "side_by_side"
        else:
            raise ValueError(f"layer {i}: unknown mixer type {kind!r}")
        layers.append(LayerSpec(name, mixer, _mlp_spec(L.get("mlp"), i)))
    return HybridSpec(model_type="sudosun", vocab_size=int(cfg["vocab"]), hidden_size=int(cfg["width"]), layers=layers,
                      norm_eps=float(cfg["norm"]["eps"]), block="sandwich", norm="dyn_tanh", tied_head=True,
                      logit_scale=float(cfg.get("logit_scale", 1.0)))


def tensor_shapes(spec: HybridSpec) -> Dict[str, tuple]:
    """name -> shape of every tensor of a checkpoint of ``spec``"""
    W = spec.hidden_size
    out = {"embed": (spec.vocab_size, W)}

    def norm(name):
        out.update({name: (W,), name + ".b": (W,), name + ".alpha": ()})

    for i, L in enumerate(spec.layers):
        p, m = f"l{i}.", L.mixer
        norm(p + "norm1")
        norm(p + "norm1b")
        q = p + "mix."
        if L.kind == "lightning":
            n, nv = m.heads * m.dim, m.heads * m.vdim
            out.update({q + "q": (n, W), q + "k": (n, W), q + "v": (nv, W), q + "g": (nv, W), q + "norm": (nv,),
                        q + "o": (W, nv)})
        elif L.kind == "gated_delta":
            n, nv = m.kv_heads * m.dim, m.heads * m.vdim
            out.update({q + "q": (n, W), q + "k": (n, W), q + "v": (nv, W), q + "q.conv": (n, m.taps),
                        q + "k.conv": (n, m.taps), q + "v.conv": (nv, m.taps), q + "a": (m.heads, W),
                        q + "b": (m.heads, W), q + "A_log": (m.heads,), q + "dt_bias": (m.heads,), q + "g": (nv, W),
                        q + "norm": (m.vdim,), q + "o": (W, nv)})
        else:
            a, r = m.left, m.right
            s = q + "left."
            out.update({s + "q": (a.heads * a.dim, W), s + "q.b": (a.heads * a.dim,), s + "k": (a.kv_heads * a.dim, W),
                        s + "k.b": (a.kv_heads * a.dim,), s + "v": (a.kv_heads * a.vdim, W),
                        s + "v.b": (a.kv_heads * a.vdim,), s + "q.norm": (a.dim,), s + "k.norm": (a.dim,),
                        s + "temp": (a.heads,), s + "sink": (a.heads,), s + "g": (a.heads, W),
                        s + "o": (W, a.heads * a.vdim), s + "out": (W,)})
            n, c = r.width, r.width // r.blocks
            s = q + "right."
            out.update({s + "x": (n, W), s + "x.b": (n,), s + "y": (n, W), s + "y.b": (n,), s + "conv": (n, r.taps),
                        s + "conv.b": (n,), s + "ra": (r.blocks, c, c), s + "ra.b": (r.blocks, c),
                        s + "ri": (r.blocks, c, c), s + "ri.b": (r.blocks, c), s + "lam": (n,), s + "o": (W, n),
                        s + "out": (W,)})
        f, q = L.mlp, p + "mlp."
        if f is not None:
            norm(p + "norm2")
            norm(p + "norm2b")
        if isinstance(f, DenseFFSpec):
            out.update({q + "gate": (f.ff, W), q + "up": (f.ff, W), q + "down": (W, f.ff)})
        elif f is not None:
            for e in range(f.experts):
                out.update({f"{q}e{e}.gate": (f.expert.ff, W), f"{q}e{e}.up": (f.expert.ff, W),
                            f"{q}e{e}.down": (W, f.expert.ff)})
            out.update({q + "router": (f.experts + f.identity, W), q + "correction": (f.experts + f.identity,)})
    norm("final.norm")
    return out


def build(spec: HybridSpec, tensors: Dict[str, torch.Tensor], dtype=torch.bfloat16, device="cuda") -> HybridCausalLM:
    """Assemble the model from name -> tensor (any float dtype; cast to ``dtype``)."""
    want = tensor_shapes(spec)
    for name, shape in want.items():
        if name not in tensors:
            raise KeyError(f"checkpoint lacks tensor {name!r}")
        if tuple(tensors[name].shape) != tuple(shape):
            raise ValueError(f"tensor {name!r}: shape {tuple(tensors[name].shape)}, configuration says {tuple(shape)}")

    def t(name):
        return tensors[name].to(device=device, dtype=dtype).contiguous()

    def norm(name):
        return DynTanh(*(tensors[name + sfx].to(device=device) for sfx in (".alpha", "", ".b")))

    layers = []
    for i, L in enumerate(spec.layers):
        p = f"l{i}.mix."
        if L.kind == "lightning":
            mixer = LightningAttention(L.mixer, *(t(p + n) for n in ("q", "k", "v", "g", "norm", "o")))
        elif L.kind == "gated_delta":
            mixer = GatedDelta(L.mixer, *(t(p + n) for n in ("q", "k", "v", "g", "a", "b")),
                               conv=tuple(t(p + n + ".conv") for n in "qkv"), a_log=t(p + "A_log"), dt_bias=t(p + "dt_bias"),
                               norm=t(p + "norm"), w_o=t(p + "o"))
        else:
            a, r = p + "left.", p + "right."
            left = MaskedAttention(L.mixer.left, t(a + "q"), t(a + "k"), t(a + "v"), t(a + "q.b"), t(a + "k.b"),
                                   t(a + "v.b"), t(a + "q.norm"), t(a + "k.norm"), t(a + "sink"), t(a + "o"),
                                   w_g=t(a + "g"), temp=t(a + "temp"))
            right = RealGatedLRU(L.mixer.right, *(t(r + n) for n in ("x", "x.b", "y", "y.b", "conv", "conv.b", "ra", "ra.b",
                                                                     "ri", "ri.b", "lam", "o")))
            mixer = SideBySide(left, right, t(a + "out"), t(r + "out"))
        mlp, n2, q = None, (), f"l{i}.mlp."
        if L.mlp is not None:
            n2 = (norm(f"l{i}.norm2"), norm(f"l{i}.norm2b"))
        if isinstance(L.mlp, DenseFFSpec):
            mlp = DenseFF(t(q + "gate"), t(q + "up"), t(q + "down"), act=L.mlp.act, limit=L.mlp.limit, alpha=L.mlp.alpha)
        elif L.mlp is not None:
            E = L.mlp.experts
            w_gu = torch.stack([torch.cat([t(f"{q}e{e}.gate"), t(f"{q}e{e}.up")], 0) for e in range(E)])
            w_down = torch.stack([t(f"{q}e{e}.down") for e in range(E)])
            mlp = ScoredMoE(L.mlp, t(q + "router"), t(q + "correction"), w_gu, w_down)
        layers.append(SandwichLayer(mixer, norm(f"l{i}.norm1"), norm(f"l{i}.norm1b"), mlp, *n2))
    return HybridCausalLM(spec, t("embed"), None, layers, norm("final.norm"), None, dtype).eval()


def load(path: str, dtype=torch.bfloat16, device="cuda") -> HybridCausalLM:
    """Read ``config.json`` + ``model.safetensors`` of a checkpoint folder."""
    from safetensors import safe_open
    with open(os.path.join(path, "config.json")) as f:
        cfg = json.load(f)
    spec = spec_from_config(cfg)
    tensors = {}
    with safe_open(os.path.join(path, "model.safetensors"), "pt") as f:
        names = set(f.keys())
        for name in tensor_shapes(spec):
            if name in names:
                tensors[name] = f.get_tensor(name)
    model = build(spec, tensors, dtype, device)
    model.config = cfg
    return model


@torch.no_grad()
def random_tensors(spec: HybridSpec, seed: int = 0, std: Optional[float] = None) -> Dict[str, torch.Tensor]:
    """Random bf16 weights of ``spec``'s shapes (benchmarks and tests)."""
    g = torch.Generator().manual_seed(seed)
    out = {}
    for name, shape in tensor_shapes(spec).items():
        r = torch.randn(shape, generator=g)
        if name.endswith(".alpha"):
            w = 0.6 + 0.1 * r
        elif name.endswith(("norm1", "norm2", "norm1b", "norm2b", ".norm", ".out", ".temp")):
            w = 1.0 + 0.1 * r
        elif name.endswith("conv"):
            w = 0.5 * r
        elif name.endswith(("lam", "A_log", "dt_bias")):
            w = -1.5 + 0.7 * r
        elif name.endswith((".b", "sink")):
            w = 0.3 * r
        elif name.endswith("correction"):
            w = 0.1 * r
        elif len(shape) >= 2 and name != "embed":
            w = r * (std if std is not None else shape[-1] ** -0.5)
        else:
            w = r * (std if std is not None else 1.0)
        out[name] = w.to(torch.bfloat16)
    return out


def random_model(spec: HybridSpec, seed: int = 0, dtype=torch.bfloat16, device="cuda") -> HybridCausalLM:
    return build(spec, random_tensors(spec, seed), dtype, device)
