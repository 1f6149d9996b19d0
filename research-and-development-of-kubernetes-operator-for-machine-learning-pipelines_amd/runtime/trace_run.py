"""Replay a trace of given token ids through an engine and write logits (``bin/trace_run``).

    trace_run --model DIR --dtype bfloat16|float32 --out DIR --max-tokens N

Steps come as JSON lines on standard input:

    {"step": 0, "entries": [{"id": "a", "tokens": [5, 17, 3], "want": [0, 2]}], "end": []}

``entries``: each request's next tokens and the places among them whose logits are wanted; a request
is admitted at its first entry.  ``end``: requests that give their row, pages and state back after the
step.  A step is one batch of the engine (``Engine.feed``).  Where something is wanted, DIR/<step>.f32
in --out gets the logits as little-endian fp32 [wanted, vocab]; after every step ``done <step>`` is
printed.  ``--max-tokens``: tokens that live requests hold at any time (the page pool's size).
"""
from __future__ import annotations

import argparse
import json
import os
import sys

MAX_LIVE = 4  # requests live at any time: rows and state slots of the engine


class TraceRunner:
    def __init__(self, engine, out_dir: str):
        self.engine, self.out = engine, out_dir
        self.live = {}

    def step(self, d: dict) -> None:
        eng, entries = self.engine, []
        for e in d.get("entries", []):
            if e["id"] not in self.live:
                self.live[e["id"]] = eng.open_sequence()
            entries.append((self.live[e["id"]], e["tokens"], e.get("want", [])))
        logits = eng.feed(entries)
        if logits is not None:
            path = os.path.join(self.out, f"{d['step']}.f32")
            logits.float().cpu().numpy().astype("<f4", copy=False).tofile(path)
        for rid in d.get("end", []):
            if rid in self.live:
                eng.close_sequence(self.live.pop(rid))


def build(model: str, dtype: str, max_tokens: int, device: str):
    import torch

    from ..models.loader import load_pretrained
    from .engine import Engine, EngineConfig
    from .kv_cache import blocks_needed

    dt = {"bfloat16": torch.bfloat16, "float32": torch.float32}[dtype]
    m = load_pretrained(model, device=device, dtype=dt)
    return Engine(m, EngineConfig(max_num_seqs=MAX_LIVE, max_num_batched_tokens=max_tokens, max_model_len=max_tokens,
                                  num_kv_blocks=blocks_needed(max_tokens) + 1, graph_buckets=(1, 2, 4),
                                  max_step_logits=max_tokens + MAX_LIVE))


def main(argv=None) -> int:
    ap = argparse.ArgumentParser(description=__doc__, formatter_class=argparse.RawDescriptionHelpFormatter)
    ap.add_argument("--model", required=True)
    ap.add_argument("--dtype", choices=("bfloat16", "float32"), default="bfloat16")
    ap.add_argument("--out", required=True)
    ap.add_argument("--max-tokens", type=int, required=True)
    ap.add_argument("--device", default="cuda")
    a = ap.parse_args(argv)
    runner = TraceRunner(build(a.model, a.dtype, a.max_tokens, a.device), a.out)
    for line in sys.stdin:
        if not line.strip():
            continue
        d = json.loads(line)
        runner.step(d)
        print(f"done {d['step']}", flush=True)
    return 0


if __name__ == "__main__":
    sys.exit(main())
