"""Replay a trace of steps through a token language model and write the logits it asks for.

    bin/trace_run --model DIR --dtype bfloat16|float32 --out DIR --max-tokens N  < steps.jsonl

One JSON object per input line: {"step": n, "entries": [{"id": .., "tokens": [..], "want": [..]}], "end": [..]}.  The entries of a line
are one batch of the engine's own step; `want` names places among an entry's tokens.  The logits go to OUT/<step>.f32 (little-endian
fp32, entries and places in order), and `done <step>` is printed after every step.  Requests are admitted at their first entry and
give back their slot and pages when a line's `end` names them.
"""
from __future__ import annotations

import argparse
import json
import sys
from pathlib import Path
from typing import Dict, Optional

SLOTS = 4


def replay(lm, lines, out: Path, emit) -> None:
    slots: Dict[str, int] = {}
    for line in lines:
        if not line.strip():
            continue
        step = json.loads(line)
        entries = []
        for e in step["entries"]:
            if e["id"] not in slots:
                slots[e["id"]] = lm.open()
            if e["tokens"]:
                entries.append((slots[e["id"]], e["tokens"], e.get("want", [])))
        if entries:
            logits = lm.step(entries)
            if logits.shape[0]:
                logits.cpu().numpy().astype("<f4").tofile(out / f"{step['step']}.f32")
        for rid in step.get("end", []):
            if rid in slots:
                lm.close(slots.pop(rid))
        emit(f"done {step['step']}")


def main(argv: Optional[list] = None) -> int:
    ap = argparse.ArgumentParser(description=__doc__, formatter_class=argparse.RawDescriptionHelpFormatter)
    ap.add_argument("--model", required=True, help="folder with config.json and model.safetensors")
    ap.add_argument("--dtype", choices=["bfloat16", "float32"], default="bfloat16")
    ap.add_argument("--out", required=True, help="folder the logits are written to")
    ap.add_argument("--max-tokens", type=int, required=True, help="tokens the cache pool holds over all live requests")
    ap.add_argument("--device", default="cuda")
    args = ap.parse_args(argv)
    from . import build
    if build.needs_build("tlm"):
        print("building libmoshi_tlm.so", file=sys.stderr, flush=True)
        build.build(which="tlm", verbose=False)
    import torch
    from . import loaders
    with torch.no_grad():
        pool = -(-args.max_tokens // 64) * 64
        lm = loaders.get_token_lm(args.model, device=args.device, dtype=getattr(torch, args.dtype), max_slots=SLOTS, max_tokens=pool,
                                  max_step_tokens=pool)
        replay(lm, sys.stdin, Path(args.out), lambda s: print(s, flush=True))
    return 0


if __name__ == "__main__":
    sys.exit(main())
