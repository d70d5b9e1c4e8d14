"""Replay of a token trace: `bin/trace_run --model DIR --dtype bfloat16|float32 --out DIR --max-tokens N`.

Steps come on standard input, one JSON object a line: `entries` (id, new tokens, the places whose logits are wanted) and `end` (ids whose
state is given back behind the step).  The wanted logits of a step go to OUT/<step>.f32 (little-endian f32 [wanted, vocab]); 'done <step>'
is printed behind every step.  The tokens run through the model's own engine: one packed batch per step."""
from __future__ import annotations

import argparse
import json
import os
import sys
from typing import Dict, List

import torch

from . import _build, _native


def _ensure_built() -> None:
    if not _native.LIB_PATH.exists() and not _native.CORE_LIB_PATH.exists() and "MI355_LLAMA_LIB" not in os.environ:
        _build.build_core(verbose=False)


def main(argv=None) -> int:
    ap = argparse.ArgumentParser(prog="trace_run", description=__doc__.split("\n")[0])
    ap.add_argument("--model", required=True)
    ap.add_argument("--dtype", choices=["bfloat16", "float32"], required=True)
    ap.add_argument("--out", required=True)
    ap.add_argument("--max-tokens", type=int, required=True, help="most tokens live requests hold at any time")
    a = ap.parse_args(argv)
    _ensure_built()
    from .hybrid_engine import Entry
    from .registry import load_model

    model = load_model(a.model, getattr(torch, a.dtype))
    engine = model.engine()
    if not getattr(engine, "supports_batches", False):
        print("trace_run: this model's engine takes no batches", file=sys.stderr)
        return 2
    engine.ensure(1, max(1, a.max_tokens))
    slot: Dict[str, int] = {}
    fed: Dict[str, int] = {}
    for line in sys.stdin:
        if not line.strip():
            continue
        step = json.loads(line)
        entries: List[Entry] = []
        fresh = [e["id"] for e in step["entries"] if e["id"] not in slot]
        if fresh:
            engine.ensure(len(slot) + len(fresh), engine.max_len)
        for e in step["entries"]:
            i = e["id"]
            if i not in slot:
                slot[i], fed[i] = engine.acquire(), 0
            entries.append(Entry(slot[i], fed[i], e["tokens"], e["want"]))
            fed[i] += len(e["tokens"])
        logits = engine.step(entries) if entries else None
        if any(len(e["want"]) for e in step["entries"]):
            data = logits.float().cpu().contiguous().numpy().astype("<f4", copy=False)
            with open(os.path.join(a.out, f"{step['step']}.f32"), "wb") as f:
                f.write(data.tobytes())
        for i in step.get("end", []):
            engine.release(slot.pop(i))
            del fed[i]
        print(f"done {step['step']}", flush=True)
    return 0


if __name__ == "__main__":
    sys.exit(main())
