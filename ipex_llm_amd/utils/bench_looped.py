"""Prefill / decode throughput of a pre-norm decoder whose middle layers run twice
(Lokolorn layout: delta rule with per-channel decays, latent attention in a window
with a sink, causal attention beside time mixing; experts behind a sigmoid router
with groups) at layer sizes of a real model, beside the framework's closest
existing model -- the decoder normed before and after (Sudosun layout,
models/sudosun.py: delta rule with a decay per head, windowed attention beside a
linear recurrent unit, experts in groups; the same ragged serving steps, paged
rows and state slots) -- at equal width, attention sizes, state sizes, expert
sizes and as many layer runs.  Random bf16 weights, synthetic tokens.  Run through
``bench.py --looped``; one JSON line.

Both models go through ``LLMEngine.feed``.  Prefill: one request of P tokens
in one step, tokens / s.  Decode: B sequences at context P, one token each per
step (hipGraph on both sides), tokens / s.
"""
from __future__ import annotations

import json
import sys
from typing import List

import torch

from .bench_prenorm import bench_model

SIZES = {
    # width, vocab; attention (heads, kv heads, dim, vdim, rotated dims; the comparison model's window); latent attention
    # (heads, dim, rotated, vdim, rank, window); time mixing (heads, dim); the comparison model's linear recurrent unit
    # (width, blocks); taps of the convolutions; delta rules (heads, key heads, dim, vdim); rank of the low-rank
    # projections (the model's default); experts (count, groups, kept groups, top, ff)
    "small": dict(width=1024, vocab=32000, attn=(8, 2, 128, 128, 64, 1024), latent=(8, 64, 32, 64, 256, 1024), mix=(8, 64),
                  lru=(1024, 8), taps=4, state=(8, 4, 64, 128), moe=(8, 4, 3, 2, 1024)),
    "base": dict(width=2048, vocab=32000, attn=(16, 4, 128, 128, 64, 2048), latent=(16, 128, 64, 128, 512, 2048),
                 mix=(16, 64), lru=(2048, 8), taps=4, state=(16, 8, 64, 128), moe=(16, 4, 3, 2, 1408)),
}
YARN = {"factor": 4.0, "original": 4096, "fast": 32.0, "slow": 1.0}


def looped_config(sz: dict) -> dict:
    """delta rule, twice (latent attention, causal attention beside time mixing), delta rule: six layer runs"""
    H, G, d, dv, rd, _ = sz["attn"]
    lh, ld, lr, lv, rank, win = sz["latent"]
    sh, sk, sd, sv = sz["state"]
    E, groups, keep, top, ff = sz["moe"]
    moe = {"kind": "moe", "expert": {"ff": ff},
           "router": {"experts": E, "groups": {"count": groups, "keep": keep}, "top": top, "scale": 2.0}}
    delta = {"heads": sh, "kv_heads": sk, "dim": sd, "vdim": sv, "conv": sz["taps"]}
    latent = {"heads": lh, "dim": ld, "rot_dim": lr, "vdim": lv, "kv_rank": rank, "scale": (ld + lr) ** -0.5,
              "mask": {"size": win}, "rot": {"base": 500000.0, "dims": lr, "scaling": YARN}}
    left = {"heads": H, "kv_heads": G, "dim": d, "vdim": dv, "conv": sz["taps"], "scale": d ** -0.5,
            "rot": {"base": 50000.0, "dims": rd}}
    pair = {"left": left, "left_scale": 0.6, "right": {"heads": sz["mix"][0], "dim": sz["mix"][1]}, "right_scale": 0.5}
    return {"architecture": "Lokolorn", "vocab": sz["vocab"], "width": sz["width"], "norm": {"eps": 1e-6},
            "loop": {"start": 1, "stop": 3, "times": 2},
            "layers": [{"type": k, "mixer": m, "mlp": moe}
                       for k, m in (("channel_delta", delta), ("latent_attention", latent), ("parallel", pair),
                                    ("channel_delta", delta))]}


def reference_config(sz: dict) -> dict:
    """six layers: the delta rule of the same sizes first and last, windowed attention of the same sizes beside a linear
    recurrent unit between them, experts of the same size on every layer"""
    H, G, d, dv, rd, win = sz["attn"]
    sh, sk, sd, sv = sz["state"]
    E, groups, keep, top, ff = sz["moe"]
    moe = {"kind": "moe", "expert": {"ff": ff},
           "router": {"experts": E, "identity": 0, "groups": {"count": groups, "keep": keep}, "top": top}}
    delta = {"heads": sh, "kv_heads": sk, "dim": sd, "vdim": sv, "conv": sz["taps"]}
    left = {"heads": H, "kv_heads": G, "dim": d, "vdim": dv, "scale": d ** -0.5, "mask": {"size": win},
            "rot": {"base": 500000.0, "dims": rd, "scaling": YARN}}
    pair = {"left": left, "right": {"width": sz["lru"][0], "blocks": sz["lru"][1], "conv": sz["taps"]}}
    return {"architecture": "Sudosun", "vocab": sz["vocab"], "width": sz["width"], "norm": {"eps": 1e-6}, "logit_scale": 1.0,
            "layers": [{"type": k, "mixer": m, "mlp": moe}
                       for k, m in (("delta", delta), *[("parallel", pair)] * 4, ("delta", delta))]}


def main(args) -> dict:
    from ..models import lokolorn as L, sudosun as S
    dev = torch.device("cuda", 0)
    torch.cuda.set_device(dev)
    out: List[dict] = []
    for name in args.looped_sizes.split(","):
        sz = SIZES[name]
        for P in [int(p) for p in args.looped_prompts.split(",")]:
            row = {"size": name, "prompt_len": P, "batch": args.batch}
            todo = [("looped", L, looped_config(sz))]
            if not args.no_looped_ref:
                todo.append(("sandwich_reference", S, reference_config(sz)))
            for key, mod, cfg in todo:
                model = mod.random_model(mod.spec_from_config(cfg), 0, torch.bfloat16, dev)
                row[key] = {"weights": sum(p.numel() for p in model.parameters())}
                row[key].update({k: round(v, 3) for k, v in
                                 bench_model(model, dev, P, args.batch, args.steps, args.warmup).items()})
                del model
                torch.cuda.empty_cache()
            out.append(row)
            print(json.dumps(row), file=sys.stderr, flush=True)
    res = {"metric": "looped pre-norm decoder prefill / decode throughput (random weights, synthetic tokens)",
           "unit": "tokens/s", "dtype": "bf16", "data": "synthetic", "n_gpus": 1, "steps": args.steps,
           "warmup": args.warmup, "rows": out}
    print(json.dumps(res))
    return res
