"""Replay a trace of token ids through a model, step by step, and write the logits asked for.

    bin/trace_run --model DIR --dtype bfloat16|float32 --out DIR --max-tokens N < steps.jsonl

Every input line is a JSON object: ``step`` (a number), ``entries`` (for each request its ``id``, its next
``tokens`` and ``want``, the places among them whose logits are written) and ``end`` (the requests that are
finished after the step).  All entries of a step are one batch.  A step in which something is wanted writes
``<out>/<step>.f32``: little-endian fp32 ``[wanted, vocab]``, in the order of the entries.  ``done <step>`` on
standard output says that a step is finished.

Nothing is sampled.  The tokens go through the serving engine of the model: first tokens as one packed
prefill, single next tokens through its captured decode step, with the requests in its slots.
"""
from __future__ import annotations

import argparse
import json
import os
import sys
from typing import Dict, List, Optional, Sequence

import numpy as np


class TraceRunner:
    def __init__(self, model, max_tokens: int):
        self.model, self.max_len = model, max(2, max_tokens + 1)
        self.engine = None
        self.slots: Dict[str, int] = {}
        self.free: List[int] = []

    def _room(self, new: int) -> None:
        """Slots for ``new`` more requests; a larger engine is only made while none is live."""
        if self.engine is not None and new <= len(self.free):
            return
        if self.slots:
            raise ValueError(f"{new} requests start while {len(self.slots)} are live and {len(self.free)} slots are free")
        self.engine = self.model.engine(max_len=self.max_len, max_batch=new)
        self.engine.reset()
        self.free = list(range(self.engine.B))[::-1]

    def step(self, entries: Sequence[dict], end: Sequence[str]):
        import torch
        logits = None
        if entries:
            new = [e["id"] for e in entries if e["id"] not in self.slots]
            if new:
                self._room(len(new))
            for i in new:
                self.slots[i] = self.free.pop()
            logits = self.engine.extend([self.slots[e["id"]] for e in entries],
                                        [torch.tensor(e["tokens"], dtype=torch.int32) for e in entries],
                                        [e.get("want", []) for e in entries])
        if end:
            gone = [self.slots.pop(i) for i in end if i in self.slots]
            if gone:
                self.engine.release(gone)
                self.free += gone
        return logits


def ensure_built() -> None:
    from .. import build
    if not os.path.exists(build.LAYERED_SO_PATH):
        build.build_layered(jobs=min(16, os.cpu_count() or 1))


def main(argv: Optional[Sequence[str]] = None) -> int:
    ap = argparse.ArgumentParser(prog="trace_run", description=__doc__.split("\n\n")[0])
    ap.add_argument("--model", required=True, help="checkpoint directory (config.json, model.safetensors)")
    ap.add_argument("--dtype", choices=["bfloat16", "float32"], default="bfloat16")
    ap.add_argument("--out", required=True, help="folder the logits are written to")
    ap.add_argument("--max-tokens", type=int, default=4096, help="most tokens that live requests hold at any time")
    args = ap.parse_args(argv)

    import torch
    from ..models.registry import load_model, read_config
    entry, _ = read_config(args.model)
    if entry.modality != "text":
        raise SystemExit("trace_run replays token ids; this model takes event frames")
    ensure_built()
    if not torch.cuda.is_available():
        raise SystemExit("trace_run needs a GPU")
    model = load_model(args.model, getattr(torch, args.dtype), torch.device("cuda:0"))
    runner = TraceRunner(model, args.max_tokens)
    os.makedirs(args.out, exist_ok=True)
    for line in sys.stdin:
        if not line.strip():
            continue
        s = json.loads(line)
        logits = runner.step(s.get("entries", []), s.get("end", []))
        if logits is not None:
            logits.float().cpu().numpy().astype(np.dtype("<f4")).tofile(os.path.join(args.out, f"{s['step']}.f32"))
        else:
            torch.cuda.synchronize()
        print(f"done {s['step']}", flush=True)
    return 0
