"""Prefill / decode throughput of a decoder normed before and after every
sublayer (Sudosun layout: windowed attention beside a real-gated linear
recurrent unit, a gated delta rule, lightning attention; experts in groups with
identity experts, clamped dense feed-forwards) at layer sizes of a real model,
beside the framework's closest existing model -- the two-norm parallel-block
decoder (Zoguzen layout, models/zoguzen.py: windowed attention beside gated
linear attention, minGRU; softmax-routed experts; the same ragged serving steps,
paged rows and state slots) -- at equal width, attention sizes, state sizes,
expert size and as many layers.  Random bf16 weights, synthetic tokens.  Run
through ``bench.py --sandwich``; one JSON line.

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
    # width, vocab; attention (heads, kv heads, dim, vdim, window, rotated dims); linear recurrent unit (width, blocks;
    # the comparison model's minGRU has twice the width); taps of the convolutions; matrix-state mixers (heads, key
    # heads of the delta rule, dim, vdim); experts (count, identity experts, groups, kept groups, top, ff); the dense
    # feed-forward has top * ff rows
    "small": dict(width=1024, vocab=32000, attn=(8, 2, 128, 128, 1024, 64), lru=(1024, 8), taps=4, state=(8, 4, 64, 128),
                  moe=(8, 2, 5, 3, 2, 1024)),
    "base": dict(width=2048, vocab=32000, attn=(16, 4, 128, 128, 2048, 64), lru=(2048, 8), taps=4, state=(16, 8, 64, 128),
                 moe=(16, 4, 4, 3, 2, 1408)),
}


def sandwich_config(sz: dict) -> dict:
    H, G, d, dv, win, rd = sz["attn"]
    sh, sk, sd, sv = sz["state"]
    E, ident, groups, keep, top, ff = sz["moe"]
    moe = {"kind": "moe", "expert": {"ff": ff},
           "router": {"experts": E, "identity": ident, "groups": {"count": groups, "keep": keep}, "top": top}}
    dense = {"kind": "dense", "ff": top * ff, "limit": 7.0}
    left = {"heads": H, "kv_heads": G, "dim": d, "vdim": dv, "scale": d ** -0.5, "mask": {"size": win},
            "rot": {"base": 500000.0, "dims": rd, "scaling": {"factor": 4.0, "original": 4096, "fast": 32.0, "slow": 1.0}}}
    pair = {"left": left, "right": {"width": sz["lru"][0], "blocks": sz["lru"][1], "conv": sz["taps"]}}
    delta = {"heads": sh, "kv_heads": sk, "dim": sd, "vdim": sv, "conv": sz["taps"]}
    lightning = {"heads": sh, "dim": sd, "vdim": sv, "decay": [2.0 ** (-(2.0 ** -i)) for i in range(sh)]}
    return {"architecture": "Sudosun", "vocab": sz["vocab"], "width": sz["width"], "norm": {"eps": 1e-6}, "logit_scale": 1.0,
            "layers": [{"type": "parallel", "mixer": pair, "mlp": moe}, {"type": "delta", "mixer": delta, "mlp": moe},
                       {"type": "lightning", "mixer": lightning, "mlp": dense},
                       {"type": "parallel", "mixer": pair, "mlp": moe}]}


def reference_config(sz: dict) -> dict:
    """windowed attention of the same sizes beside gated linear attention of the same state size, minGRU layers in
    the places of the delta rule and of lightning attention, experts of the same size on every layer"""
    H, G, d, dv, win, rd = sz["attn"]
    sh, _, sd, sv = sz["state"]
    E, _, _, _, top, ff = sz["moe"]
    mlp = {"kind": "moe", "router": {"experts": E, "top": top}, "expert": {"ff": ff}}
    left = {"heads": H, "kv_heads": G, "dim": d, "vdim": dv, "conv": sz["taps"], "scale": d ** -0.5, "mask": {"size": win},
            "rot": {"base": 500000.0, "dims": rd, "scaling": {"factor": 8.0, "low": 1.0, "high": 4.0, "original": 8192}}}
    pair = {"left": left, "right": {"heads": sh, "dim": sd, "vdim": sv, "tau": 8.0, "rank": 64}}
    gru = {"width": 2 * sz["lru"][0]}
    return {"architecture": "Zoguzen", "vocab": sz["vocab"], "width": sz["width"], "norm": {"eps": 1e-6},
            "layers": [{"type": k, "mixer": m, "mlp": mlp}
                       for k, m in (("parallel", pair), ("mingru", gru), ("mingru", gru), ("parallel", pair))]}


def main(args) -> dict:
    from ..models import sudosun as S, zoguzen as Z
    dev = torch.device("cuda", 0)
    torch.cuda.set_device(dev)
    out: List[dict] = []
    for name in args.sandwich_sizes.split(","):
        sz = SIZES[name]
        for P in [int(p) for p in args.sandwich_prompts.split(",")]:
            row = {"size": name, "prompt_len": P, "batch": args.batch}
            todo = [("sandwich", S, sandwich_config(sz))]
            if not args.no_sandwich_ref:
                todo.append(("twonorm_reference", Z, reference_config(sz)))
            for key, mod, cfg in todo:
                model = mod.random_model(mod.spec_from_config(cfg), 0, torch.bfloat16, dev)
                row[key] = {"weights": sum(p.numel() for p in model.parameters())}
                row[key].update({k: round(v, 3) for k, v in
                                 bench_model(model, dev, P, args.batch, args.steps, args.warmup).items()})
                del model
                torch.cuda.empty_cache()
            out.append(row)
            print(json.dumps(row), file=sys.stderr, flush=True)
    res = {"metric": "before-and-after-normed decoder prefill / decode throughput (random weights, synthetic tokens)",
           "unit": "tokens/s", "dtype": "bf16", "data": "synthetic", "n_gpus": 1, "steps": args.steps,
           "warmup": args.warmup, "rows": out}
    print(json.dumps(res))
    return res
