"""Replays a trace of token ids through a model and writes logits (the program behind bin/trace_run).

Standard input holds one step per line, {"step": 0, "entries": [{"id": "a", "tokens": [5, 17], "want": [1]}], "end": []}:
the next tokens of a request and the places among them whose logits are wanted.  A step with wanted places writes
OUT/<step>.f32 ([wanted, vocab], little-endian fp32); every step prints `done <step>` when it is complete.  The tokens
run through the runtime the generation path uses (its decode graph and prompt passes); one request is live at a time,
and `end` gives its state back.
"""
from __future__ import annotations

import argparse
import json
import os
import sys


def main(argv=None) -> int:
    ap = argparse.ArgumentParser(prog="trace_run", description="feed token ids through a model step by step and write logits")
    ap.add_argument("--model", required=True, help="checkpoint directory")
    ap.add_argument("--dtype", choices=["bfloat16", "float32"], default="bfloat16")
    ap.add_argument("--out", required=True, help="directory for <step>.f32")
    ap.add_argument("--max-tokens", type=int, default=4096, help="most tokens the live request holds")
    args = ap.parse_args(argv)
    from . import registry
    fam = registry.family_of(registry.read_config(args.model))
    act = 32 if args.dtype == "float32" else 16
    if act not in fam.acts:
        print(f"trace_run: models of family '{fam.name}' do not run in {args.dtype}", file=sys.stderr)
        return 3
    cfg, w = fam.load(args.model, max(args.max_tokens, 64), act)
    rt = fam.runtime(cfg, w)
    rt.reset()
    live = None
    for line in sys.stdin:
        if not line.strip():
            continue
        s = json.loads(line)
        wanted = []
        for e in s["entries"]:
            if live is not None and e["id"] != live:
                raise ValueError(f"request {e['id']!r} begins while {live!r} is live: this runtime holds one sequence")
            if live is None:
                rt.reset()
                live = e["id"]
            wanted.append(rt.step(e["tokens"], e.get("want", [])))
        if any(len(v) for v in wanted):
            with open(os.path.join(args.out, f"{s['step']}.f32"), "wb") as f:
                for v in wanted:
                    f.write(v.astype("<f4").tobytes())
        if live in s.get("end", []):
            live = None
        print(f"done {s['step']}", flush=True)
    return 0
