"""Trace runner: feeds given token ids through an engine's mixed-batch step.

One step per input line,

    {"step": 0,
     "entries": [{"id": "a", "tokens": [5, 17, 3], "want": [0, 2]}],
     "end": []}

All entries of a step run as one batch from the cache that earlier steps
left.  A request is admitted at its first entry; ``end`` gives its pages
and slot back after the step.  When logits are wanted they go to
OUT/<step>.f32 (little-endian fp32, [wanted, vocab], in the order of the
entries and of ``want``); then ``done <step>`` is printed.
"""

from __future__ import annotations

import argparse
import json
import os
import sys

DTYPES = {"bfloat16": "bf16", "float32": "fp32"}
LIVE = 4            # requests that can be live at a time


class TraceRunner:
    def __init__(self, model):
        self.model = model
        self.live = {}

    def run(self, step: dict):
        """One step; returns the wanted logits [wanted, vocab] fp32."""
        from ..models.layered import StepEntry

        entries = []
        for e in step.get("entries", []):
            rid = e["id"]
            if rid not in self.live:
                self.live[rid] = self.model.open_sequence()
            entries.append(StepEntry(self.live[rid], e["tokens"],
                                     e.get("want", [])))
        out = self.model.step(entries).cpu().numpy() if entries else None
        for rid in step.get("end", []):
            self.model.close_sequence(self.live.pop(rid))
        return out


def main(argv=None) -> int:
    ap = argparse.ArgumentParser(prog="trace_run")
    ap.add_argument("--model", required=True,
                    help="folder with config.json and model.safetensors")
    ap.add_argument("--dtype", required=True, choices=sorted(DTYPES))
    ap.add_argument("--out", required=True, help="folder for <step>.f32")
    ap.add_argument("--max-tokens", type=int, required=True,
                    help="tokens the cache pool holds")
    args = ap.parse_args(argv)

    from ..io.loader import LazyCheckpointWeights, load_config
    from ..models.registry import engine_class, kernel_libraries

    config = load_config(args.model)
    cls = engine_class(config)
    if not hasattr(cls, "step"):
        print(f"trace_run: {config.model_type} has no mixed-batch step",
              file=sys.stderr)
        return 2
    from csrc.build import ensure_built
    ensure_built(names=kernel_libraries(config))
    model = cls(config, LazyCheckpointWeights(args.model),
                dtype=DTYPES[args.dtype], max_seq=args.max_tokens,
                pool_tokens=args.max_tokens, max_batch=LIVE)
    runner = TraceRunner(model)
    for line in sys.stdin:
        if not line.strip():
            continue
        step = json.loads(line)
        out = runner.run(step)
        if out is not None and len(out):
            path = os.path.join(args.out, f"{step['step']}.f32")
            out.astype("<f4", copy=False).tofile(path)
        print(f"done {step['step']}", flush=True)
    return 0
