"""Trace replay: given tokens in, logits out, through SamplerEngine.step.

Nothing is sampled.  The engine is the one that generates: its paged pool is
made for the live requests' tokens and its state slots for four requests, so
pages and slots are used again as requests end."""
from __future__ import annotations

import argparse
import json
import os
import sys

import torch

from .build import ensure_built
from .models.registry import architecture_of
from .sampler import SamplerEngine, SeqState

LIVE_REQUESTS = 4


class TraceRunner:
    def __init__(self, model, max_tokens: int):
        self.engine = SamplerEngine(model, kv_pool_tokens=max_tokens, kv_cache_dtype="bf16",
                                    max_num_seqs=LIVE_REQUESTS, state_slots=LIVE_REQUESTS)
        self.live: dict[str, SeqState] = {}

    @torch.no_grad()
    def step(self, entries, end):
        """Logits [wanted, vocab] float32 of one step, or None."""
        batch = []
        for e in entries:
            s = self.live.get(e["id"])
            if s is None:
                s = self.live[e["id"]] = SeqState(len(self.live), [], out_index=0)
            s.tokens.extend(e["tokens"])
            batch.append((s, len(e["tokens"])))
        logits = None
        if batch:
            hidden, starts = self.engine.step(batch)
            rows = [r + w for e, r in zip(entries, starts) for w in e["want"]]
            if rows:
                index = torch.tensor(rows, device=hidden.device)
                logits = self.engine.model.logits(hidden[index]).float().cpu()
        for name in end:
            self.engine.pool.release(self.live.pop(name))
        return logits


def main(argv=None) -> int:
    ap = argparse.ArgumentParser(prog="trace_run", description=__doc__)
    ap.add_argument("--model", required=True)
    ap.add_argument("--dtype", required=True, choices=["bfloat16", "float32"])
    ap.add_argument("--out", required=True)
    ap.add_argument("--max-tokens", type=int, required=True)
    ap.add_argument("--device", default="cuda", help="cuda (default), or cpu for the "
                                                     "reference operations")
    args = ap.parse_args(argv)
    arch = architecture_of(args.model)
    if args.device != "cpu":
        ensure_built(arch.model.extensions)
    # true 32-bit products in float32
    torch.backends.cuda.matmul.allow_tf32 = False
    torch.set_float32_matmul_precision("highest")
    model = arch.load(args.model, dtype=args.dtype).to(args.device).eval()
    run = TraceRunner(model, args.max_tokens)
    for line in sys.stdin:
        if not line.strip():
            continue
        s = json.loads(line)
        logits = run.step(s["entries"], s["end"])
        if logits is not None:
            logits.numpy().astype("<f4").tofile(os.path.join(args.out, f"{s['step']}.f32"))
        print(f"done {s['step']}", flush=True)
    return 0
