"""Replay of a recorded trace through an engine's own `step` (Engine/backend_core.py: ragged batch, page pool, kernels).

    trace_run --model FOLDER --dtype bfloat16 --out RESULTS --max-tokens 4096 < trace.jsonl

One JSON object per input line is one engine step: `step` (a number), `entries` (per sequence its `id`, its next `tokens` and
in `want` the indexes among them whose logits are to be kept) and `end` (ids to release afterwards), for instance

    {"step": 7, "entries": [{"id": "x", "tokens": [11], "want": [0]}, {"id": "y", "tokens": [2], "want": []}], "end": ["y"]}

The kept logits of step 7 become RESULTS/7.f32 (rows of little-endian float32, entry by entry); `done 7` on standard output says
that the step is finished.
"""
from __future__ import annotations

import argparse
import json
import os
import sys

MAX_SLOTS = 256          # live sequences to make room for up front; a larger batch re-sizes the (then empty) pool


def parser():
    ap = argparse.ArgumentParser(prog="trace_run", description="Replay a trace of tokens and write logits.")
    ap.add_argument("--model", required=True, help="folder with config.json and model.safetensors")
    ap.add_argument("--dtype", required=True, choices=["bfloat16", "float32"])
    ap.add_argument("--out", required=True, help="folder for the <step>.f32 files")
    ap.add_argument("--max-tokens", type=int, default=8192, help="most tokens that live sequences hold at any time")
    ap.add_argument("--device", default="cuda:0")
    return ap


class Replay:
    def __init__(self, model_dir, dtype, max_tokens, device="cuda:0"):
        import torch

        from .Engine.SnapKV.backend import LMBackend
        if dtype == torch.float32:
            torch.backends.cuda.matmul.allow_tf32 = False
            torch.set_float32_matmul_precision("highest")
        self.max_tokens = max(int(max_tokens), 1)
        self.engine = LMBackend(dtype=dtype, device=device)
        self.engine.load_model(model_dir, use_tp=False)
        self._setup(min(self.max_tokens, MAX_SLOTS))

    def _setup(self, slots):
        from .Engine.backend_core import PAGE_SIZE
        eng = self.engine
        limit = getattr(getattr(eng.model, "spec", None), "max_positions", 0)
        self.slots = slots
        eng.setup_caches(max_batch_size=slots, max_seq_length=min(self.max_tokens, limit) if limit else self.max_tokens,
                         num_pages=-(-self.max_tokens // PAGE_SIZE) + slots)

    def step(self, msg):
        """One step; the wanted logits as float32 on the host, or None."""
        entries = [(e["id"], e["tokens"]) for e in msg["entries"]]
        want = [e.get("want", []) for e in msg["entries"]]
        if len(entries) > self.slots and not self.engine.pool.seqs:
            self._setup(len(entries))
        _, logits = self.engine.step(entries, want, sample=False)
        out = None
        if logits is not None:
            # engine.step returns each entry's wanted rows in ascending order, once
            row, pick = 0, []
            for w in want:
                order = {p: row + k for k, p in enumerate(sorted(set(w)))}
                row += len(order)
                pick += [order[p] for p in w]
            out = logits.float().cpu()[pick]
        for sid in msg.get("end", []):
            self.engine.end(sid)
        return out


def main(argv=None, stdin=None, stdout=None):
    args = parser().parse_args(argv)
    stdin, stdout = stdin or sys.stdin, stdout or sys.stdout
    from .build_lib import ensure_built
    ensure_built()
    import torch
    replay = Replay(args.model, getattr(torch, args.dtype), args.max_tokens, args.device)
    for line in stdin:
        if not line.strip():
            continue
        msg = json.loads(line)
        out = replay.step(msg)
        if out is not None:
            out.numpy().astype("<f4").tofile(os.path.join(args.out, f"{msg['step']}.f32"))
        print(f"done {msg['step']}", file=stdout, flush=True)
    return 0
