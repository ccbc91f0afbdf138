"""Throughput of a layered decoder design beside the closest model of the zoo at equal size (bench.py --design NAME).

Both models have the same width, heads, head sizes, feed-forward width, vocabulary, batch and context, random weights, and run
through the same engine (LMBackend): chunked prefill of the whole batch, then decode steps replayed as hipGraphs.  A size has a
few layers of a real model's shape; `per_layer_us` takes the head and embedding out by timing two depths.

* furitar: the context fits one attention chunk, so both read the same number of keys per step;
* bufodra: latent rows of 512 + 64 numbers, heads of 128 + 64; the Llama-style model has as many heads of 128 (8 kv heads), so
  that both have the same output size per head; a quarter of the layers attends to another layer's cache.
"""
from __future__ import annotations

import json
import tempfile
import time
from pathlib import Path

import torch

# design -> name: (width, heads, kv heads, head size, ff, batch, prefix)
SIZES = {
    "furitar": {
        "1b-B64-2K": (2048, 32, 8, 64, 8192, 64, 2049),
        "8b-B64-2K": (4096, 32, 8, 128, 14336, 64, 2049),
        "8b-B8-8K": (4096, 32, 8, 128, 14336, 8, 8065),
    },
    "bufodra": {
        "1b-B64-2K": (2048, 16, 8, 128, 8192, 64, 2049),
        "8b-B64-2K": (4096, 32, 8, 128, 14336, 64, 2049),
        "8b-B8-8K": (4096, 32, 8, 128, 14336, 8, 8065),
    },
}
VOCAB = 32000
DEPTHS = {"furitar": (2, 6), "bufodra": (4, 8)}      # (bufodra: groups of four layers, three of them with a cache)


def _design_config(design, size, n_layer):
    from .Engine import designs
    W, H, KH, D, ff, _, prefix = SIZES[design][size]
    if design == "furitar":
        return designs._furitar_config(VOCAB, W, n_layer, H, KH, D, D, ff, prefix + 256, prefix + 256)
    return designs._bufodra_config(VOCAB, W, n_layer, H, D, 64, D, 3 * W // 8, 512, ff)


def _configs(design, size, n_layer):
    """(checkpoint path of the design, checkpoint path of the zoo model): neither file exists -> seeded random weights."""
    from .Engine import designs, model_core
    W, H, KH, D, ff, _, prefix = SIZES[design][size]
    root = Path(tempfile.gettempdir()) / "no-checkpoint"
    a, b = f"{design}-bench-{size}-{n_layer}".lower(), f"llama-bench-{size}-{n_layer}"
    designs.design_configs[a] = _design_config(design, size, n_layer)
    model_core.transformer_configs[b] = dict(block_size=prefix + 256, n_layer=n_layer, n_head=H, n_local_heads=KH, dim=W,
                                             intermediate_size=ff, vocab_size=VOCAB, rope_base=500000.0)
    return root / a / "model.pth", root / b / "model.pth"


def _measure(path, B, prefix, steps, warmup, dev):
    from .Engine.SnapKV.backend import LMBackend
    eng = LMBackend(dtype=torch.bfloat16, device=dev)
    eng.load_model(path, use_tp=False)
    eng.compile()
    eng.setup_caches(max_batch_size=B, max_seq_length=-(-(prefix + 64) // 128) * 128)
    ids = torch.randint(0, VOCAB, (B, prefix), generator=torch.Generator().manual_seed(1)).to(dev)
    eng.encode(ids)                                                 # warm-up: library handles, workspaces, allocations
    torch.cuda.synchronize()
    t0 = time.perf_counter()
    nxt = eng.encode(ids)[:, -1:]
    torch.cuda.synchronize()
    prefill = time.perf_counter() - t0
    for _ in range(warmup):
        eng.inference(nxt, benchmark=True)
    torch.cuda.synchronize()
    t0 = time.perf_counter()
    for _ in range(steps):
        eng.inference(nxt, benchmark=True)
    torch.cuda.synchronize()
    decode = (time.perf_counter() - t0) / steps
    del eng
    torch.cuda.empty_cache()
    return prefill, decode


def run(design="furitar", sizes=None, steps=40, warmup=8, dev="cuda:0", only=None):
    """One JSON-able record: per size, the design and the zoo model at two depths."""
    design = design.lower()
    if design not in SIZES:
        raise ValueError(f"unknown design {design!r}")
    out = []
    depths = DEPTHS[design]
    for size in sizes or SIZES[design]:
        B, prefix = SIZES[design][size][5:]
        rec = {"size": size, "batch": B, "prefix": prefix}
        for which, name in enumerate(("design", "zoo_llama")):
            if only and name != only:
                continue
            (p0, d0), (p1, d1) = (_measure(_configs(design, size, n)[which], B, prefix, steps, warmup, dev) for n in depths)
            span = depths[1] - depths[0]
            rec[name] = {"prefill_tokens_per_s": round(B * prefix / p1, 1), "decode_ms_per_step": round(d1 * 1e3, 4),
                         "decode_tokens_per_s": round(B / d1, 1), "layers": depths[1],
                         "decode_us_per_layer": round((d1 - d0) / span * 1e6, 2),
                         "prefill_us_per_layer_and_ktoken": round((p1 - p0) / span / (B * prefix) * 1e9, 2)}
            print(f"# {size} {name}: {rec[name]}", flush=True)
        out.append(rec)
    return out


def main(args):
    rec = run(args.design, args.design_sizes, args.steps, args.warmup, only=args.design_only)
    best = next((r["design"] for r in rec if "design" in r), None)
    print(json.dumps({"metric": "layered design decode throughput", "value": best["decode_tokens_per_s"] if best else None,
                      "unit": "tokens/s", "n_gpus": 1, "steps": args.steps, "warmup": args.warmup, "higher_is_better": True,
                      "dtype": "bf16", "data": "synthetic", "config": {"design": args.design, "sizes": rec}}))
    return 0
