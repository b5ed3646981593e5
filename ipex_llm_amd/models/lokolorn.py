"""Lokolorn: a pre-norm decoder some of whose layers run several times over with
the same weights, each pass fed by the state it reached and the token embedding;
its layers mix a delta rule with one decay per key channel, latent attention in a
sliding window with a sink, and causal attention beside RWKV-6 time mixing; experts
behind a sigmoid router with groups.  Read from its own checkpoint layout.

A checkpoint folder holds ``config.json`` (``"architecture": "Lokolorn"``) and
``model.safetensors`` (bf16 weights, linear weights stored [out, in]).  The
configuration lists the layers in order; each entry names its mixer type
(``channel_delta``, ``latent_attention``, ``parallel``), the mixer's sizes and its
feed-forward (``moe`` or none); ``loop`` names the layers that run several times.
Tensor names: ``embed``, ``loop.in``, ``l<i>.norm1`` / ``norm2`` / ``ls1`` /
``ls2``, ``l<i>.mix.<name>``, ``l<i>.mlp.<name>``, ``final.norm``, ``head``.  Every
size and constant comes from the configuration (the ranks of the low-rank
projections from their tensors); the building blocks are the generic ones of
``models/hybrid.py``:

* ``channel_delta``    -> ``ChannelDelta`` (``q`` ``k`` ``v`` + ``.conv``, ``b``, ``a1`` ``a2`` ``A_log`` ``dt_bias``,
                          ``norm`` ``g1`` ``g2`` ``o``)
* ``latent_attention`` -> ``LatentAttention`` (neighbouring rotary pairs with YaRN scaling, a window, a sink per head)
* ``parallel``         -> ``ScaledSum`` of ``MaskedAttention`` (``left``: biased projections, convolutions, half-split rotary
                          pairs, RMS norm per head without a weight) and ``TimeMix`` (``right``)
* feed-forward         -> ``ScoredMoE`` (sigmoid scores, groups ranked by their two best, renormalised weights)

Norm weights are stored around zero; the product is with 1 + w, formed in f32.
"""
from __future__ import annotations

import json
import os
from typing import Dict, Optional

import torch

from .hybrid import (ChannelDelta, ChannelDeltaSpec, ExpertSpec, HybridCausalLM, HybridSpec, LatentAttention,
                     LatentAttentionSpec, LayerSpec, LoopSpec, MaskedAttention, MaskedAttentionSpec, MaskSpec, MoESpec,
                     PreNormLayer, RotarySpec, ScaledSum, ScaledSumSpec, ScoredMoE, TimeMix, TimeMixSpec)

ARCHITECTURE = "Lokolorn"
DEFAULT_RANK = 64               # low-rank projections of models that are not read from tensors


def _heads(m: dict, i: int):
    H, G = int(m["heads"]), int(m.get("kv_heads", m["heads"]))
    if H < 1 or G < 1 or H % G:
        raise ValueError(f"layer {i}: heads must be a multiple of kv_heads")
    return H, G


def _rotary(rot: Optional[dict], most: int, layout: str, i: int) -> Optional[RotarySpec]:
    if not rot or not int(rot.get("dims", 0)):
        return None
    rs = RotarySpec(int(rot["dims"]), float(rot["base"]), rot.get("scaling") or None, layout)
    if rs.dims > most or rs.dims % 2:
        raise ValueError(f"layer {i}: rot.dims must be even and at most {most}")
    return rs


def _mixer_spec(kind: str, m: dict, i: int, rank):
    """``rank(name)``: the rank of a low-rank projection, given the name of its first matrix"""
    if kind == "channel_delta":
        H, K = _heads(m, i)
        return "channel_delta", ChannelDeltaSpec(heads=H, kv_heads=K, dim=int(m["dim"]), vdim=int(m["vdim"]),
                                                 taps=int(m["conv"]), rank=rank("a1"), gate_rank=rank("g1"))
    if kind == "latent_attention":
        dr = int(m["rot_dim"])
        rs = _rotary(m.get("rot"), dr, "pairs", i)
        if rs is None or rs.dims != dr:
            raise ValueError(f"layer {i}: rot.dims must be rot_dim")
        window = int(m["mask"]["size"])
        if window < 1:
            raise ValueError(f"layer {i}: mask.size must be at least 1")
        return "latent_attention", LatentAttentionSpec(
            heads=int(m["heads"]), dim=int(m["dim"]), rot_dim=dr, vdim=int(m["vdim"]), kv_rank=int(m["kv_rank"]),
            scale=float(m["scale"]), rot=rs, out_gate=False, window=window, sink=True)
    if kind == "parallel":
        a, b = m["left"], m["right"]
        H, G = _heads(a, i)
        rs = _rotary(a.get("rot"), int(a["dim"]), "half", i)
        if rs is not None and rs.scaling:
            raise ValueError(f"layer {i}: the causal attention's rotary positions have no scaling")
        left = MaskedAttentionSpec(heads=H, kv_heads=G, dim=int(a["dim"]), vdim=int(a["vdim"]), scale=float(a["scale"]),
                                   rot=rs, mask=MaskSpec("causal"), qk_norm="unit", bias=True, out_bias=True, sink=False,
                                   taps=int(a["conv"]))
        right = TimeMixSpec(heads=int(b["heads"]), dim=int(b["dim"]), rank=rank("right.w1"))
        return "scaled_sum", ScaledSumSpec(left, right, float(m["left_scale"]), float(m["right_scale"]))
    raise ValueError(f"layer {i}: unknown mixer type {kind!r}")


def _mlp_spec(m: Optional[dict], i: int) -> Optional[MoESpec]:
    if m is None:
        return None
    if m.get("kind", "moe") != "moe":
        raise ValueError(f"layer {i}: unknown feed-forward kind {m['kind']!r}")
    r = m["router"]
    E, top = int(r["experts"]), int(r["top"])
    g = r.get("groups") or {"count": 1, "keep": 1}
    count, keep = int(g["count"]), int(g["keep"])
    if count < 1 or E % count or not 1 <= keep <= count or not 1 <= top <= keep * (E // count):
        raise ValueError(f"layer {i}: router.groups must split the experts evenly and leave at least top of them")
    return MoESpec(experts=E, top=top, expert=ExpertSpec(ff=int(m["expert"]["ff"])), groups=count, keep=keep, score="sigmoid",
                   group="top2", renorm=True, scale=float(r["scale"]))


def spec_from_config(cfg: dict, ranks: Optional[Dict[str, int]] = None) -> HybridSpec:
    """``ranks``: tensor name of a low-rank projection's first matrix -> its rows (``load`` reads them from the file);
    without it ``DEFAULT_RANK``"""
    layers = []
    for i, L in enumerate(cfg["layers"]):
        def rank(name, i=i):
            return int((ranks or {}).get(f"l{i}.mix.{name}", DEFAULT_RANK))
        layers.append(LayerSpec(*_mixer_spec(L["type"], L["mixer"], i, rank), _mlp_spec(L.get("mlp"), i)))
    loop = cfg.get("loop")
    if loop:
        loop = LoopSpec(int(loop["start"]), int(loop["stop"]), int(loop["times"]))
        if not 0 <= loop.start < loop.stop <= len(layers) or loop.times < 1:
            raise ValueError("loop: 0 <= start < stop <= layers and times >= 1")
    return HybridSpec(model_type="lokolorn", vocab_size=int(cfg["vocab"]), hidden_size=int(cfg["width"]), layers=layers,
                      norm_eps=float(cfg["norm"]["eps"]), block="pre_norm", norm="rms_offset", layer_scale=True,
                      loop=loop or None)


RANKED = ("a1", "g1", "right.w1")


def ranks_of(shapes: Dict[str, tuple]) -> Dict[str, int]:
    return {n: int(s[0]) for n, s in shapes.items() if ".mix." in n and n.split(".mix.", 1)[1] in RANKED}


def tensor_shapes(spec: HybridSpec) -> Dict[str, tuple]:
    """name -> shape of every tensor of a checkpoint of ``spec``"""
    W = spec.hidden_size
    out = {"embed": (spec.vocab_size, W)}
    if spec.loop is not None:
        out["loop.in"] = (W, 2 * W)
    for i, L in enumerate(spec.layers):
        p, m = f"l{i}.", L.mixer
        out.update({p + "norm1": (W,), p + "ls1": (W,)})
        q = p + "mix."
        if L.kind == "channel_delta":
            n, nv, nd = m.kv_heads * m.dim, m.heads * m.vdim, m.heads * m.dim
            out.update({q + "q": (n, W), q + "k": (n, W), q + "v": (nv, W), q + "q.conv": (n, m.taps),
                        q + "k.conv": (n, m.taps), q + "v.conv": (nv, m.taps), q + "b": (m.heads, W),
                        q + "A_log": (m.heads,), q + "norm": (m.vdim,), q + "a1": (m.rank, W), q + "a2": (nd, m.rank),
                        q + "dt_bias": (nd,), q + "g1": (m.gate_rank, W), q + "g2": (nv, m.gate_rank), q + "o": (W, nv)})
        elif L.kind == "latent_attention":
            out.update({q + "q": (m.heads * (m.dim + m.rot_dim), W), q + "dkv": (m.kv_rank + m.rot_dim, W),
                        q + "dkv.norm": (m.kv_rank,), q + "uk": (m.heads * m.dim, m.kv_rank),
                        q + "uv": (m.heads * m.vdim, m.kv_rank), q + "sink": (m.heads,), q + "o": (W, m.heads * m.vdim)})
        else:
            a, r = m.left, m.right
            s = q + "left."
            for name, n in (("q", a.heads * a.dim), ("k", a.kv_heads * a.dim), ("v", a.kv_heads * a.vdim)):
                out.update({s + name: (n, W), s + name + ".b": (n,), s + name + ".conv": (n, a.taps)})
            out.update({s + "o": (W, a.heads * a.vdim), s + "o.b": (W,)})
            n, s = r.heads * r.dim, q + "right."
            out.update({s + "mu." + c: (W,) for c in "rkvgw"})
            out.update({s + c: (n, W) for c in "rkvg"})
            out.update({s + "w1": (r.rank, W), s + "w2": (n, r.rank), s + "w0": (n,), s + "u": (r.heads, r.dim),
                        s + "norm": (n,), s + "o": (W, n)})
        f, q = L.mlp, p + "mlp."
        if f is not None:
            out.update({p + "norm2": (W,), p + "ls2": (W,)})
            for e in range(f.experts):
                out.update({f"{q}e{e}.gate": (f.expert.ff, W), f"{q}e{e}.up": (f.expert.ff, W),
                            f"{q}e{e}.down": (W, f.expert.ff)})
            out.update({q + "router": (f.experts, W), q + "correction": (f.experts,)})
    out.update({"final.norm": (W,), "head": (spec.vocab_size, W)})
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

    def f32(name):
        return tensors[name].to(device=device, dtype=torch.float32).contiguous()

    layers = []
    for i, L in enumerate(spec.layers):
        p = f"l{i}.mix."
        if L.kind == "channel_delta":
            mixer = ChannelDelta(L.mixer, *(t(p + n) for n in ("q", "k", "v", "b", "a1", "a2", "g1", "g2")),
                                 conv=tuple(t(p + n + ".conv") for n in "qkv"), a_log=f32(p + "A_log"),
                                 dt_bias=f32(p + "dt_bias"), norm=t(p + "norm"), w_o=t(p + "o"))
        elif L.kind == "latent_attention":
            mixer = LatentAttention(L.mixer, *(t(p + n) for n in ("q", "dkv", "dkv.norm", "uk", "uv")), None, t(p + "o"),
                                    sink=f32(p + "sink"))
        else:
            a, r = p + "left.", p + "right."
            left = MaskedAttention(L.mixer.left, t(a + "q"), t(a + "k"), t(a + "v"), t(a + "q.b"), t(a + "k.b"),
                                   t(a + "v.b"), None, None, None, t(a + "o"),
                                   conv=tuple(t(a + n + ".conv") for n in "qkv"), b_o=t(a + "o.b"))
            right = TimeMix(L.mixer.right, torch.stack([f32(r + "mu." + c) for c in "rkvgw"]), [t(r + c) for c in "rkvg"],
                            t(r + "w1"), t(r + "w2"), f32(r + "w0"), f32(r + "u"), t(r + "norm"), t(r + "o"))
            mixer = ScaledSum(left, right, L.mixer.left_scale, L.mixer.right_scale, spec.hidden_size)
        mlp, n2, ls2, q = None, None, None, f"l{i}.mlp."
        if L.mlp is not None:
            E = L.mlp.experts
            w_gu = torch.stack([torch.cat([t(f"{q}e{e}.gate"), t(f"{q}e{e}.up")], 0) for e in range(E)])
            w_down = torch.stack([t(f"{q}e{e}.down") for e in range(E)])
            mlp = ScoredMoE(L.mlp, t(q + "router"), f32(q + "correction"), w_gu, w_down)
            n2, ls2 = 1.0 + f32(f"l{i}.norm2"), f32(f"l{i}.ls2")
        layers.append(PreNormLayer(mixer, 1.0 + f32(f"l{i}.norm1"), mlp, n2, f32(f"l{i}.ls1"), ls2))
    return HybridCausalLM(spec, t("embed"), None, layers, 1.0 + f32("final.norm"), t("head"), dtype,
                          loop_in=t("loop.in") if spec.loop is not None else None).eval()


def load(path: str, dtype=torch.bfloat16, device="cuda") -> HybridCausalLM:
    """Read ``config.json`` + ``model.safetensors`` of a checkpoint folder."""
    from safetensors import safe_open
    with open(os.path.join(path, "config.json")) as f:
        cfg = json.load(f)
    with safe_open(os.path.join(path, "model.safetensors"), "pt") as f:
        shapes = {name: tuple(f.get_slice(name).get_shape()) for name in f.keys()}
        spec = spec_from_config(cfg, ranks_of(shapes))
        tensors = {name: f.get_tensor(name) for name in tensor_shapes(spec) if name in shapes}
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
        if name.endswith(("norm1", "norm2", "final.norm")):
            w = 0.1 * r
        elif name.endswith(".norm"):
            w = 1.0 + 0.1 * r
        elif name.endswith((".ls1", ".ls2")):
            w = 0.7 + 0.1 * r
        elif ".mu." in name:
            w = 0.5 + 0.2 * r
        elif name.endswith("conv"):
            w = 0.5 * r
        elif name.endswith(("A_log", "dt_bias", "w0")):
            w = -1.5 + 0.7 * r
        elif name.endswith("correction"):
            w = 0.1 * r
        elif len(shape) >= 2 and name != "embed":
            w = r * (std if std is not None else shape[-1] ** -0.5)
        elif len(shape) == 1:
            w = 0.3 * r
        else:
            w = r * (std if std is not None else 1.0)
        out[name] = w.to(torch.bfloat16)
    return out


def random_model(spec: HybridSpec, seed: int = 0, dtype=torch.bfloat16, device="cuda") -> HybridCausalLM:
    return build(spec, random_tensors(spec, seed), dtype, device)
