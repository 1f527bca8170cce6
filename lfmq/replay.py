"""Trace replay: feed given token ids through a model step by step and
write the logits that the trace asks for (bin/trace_run).

One JSON object a line on standard input:
    {"step": 0, "entries": [{"id": "a", "tokens": [5, 17], "want": [1]}],
     "end": ["a"]}
writes <out>/<step>.f32 ([wanted, vocab] little-endian fp32, in the order
of the entries) if anything is wanted, and prints `done <step>`.
"""
from __future__ import annotations

import argparse
import json
import os
import sys


def main(argv=None) -> int:
    ap = argparse.ArgumentParser(prog="trace_run", description=__doc__,
                                 formatter_class=argparse.RawDescriptionHelpFormatter)
    ap.add_argument("--model", required=True,
                    help="folder with config.json and model.safetensors")
    ap.add_argument("--dtype", default="bfloat16",
                    choices=["bfloat16", "float32"])
    ap.add_argument("--out", required=True, help="folder for the logits")
    ap.add_argument("--max-tokens", type=int, required=True,
                    help="most tokens that live requests hold at a time")
    args = ap.parse_args(argv)

    from .ops.build import ensure_built
    ensure_built("lfmq_seq")
    import torch

    from . import api
    from .models.generation import PackedStepper
    model = api.load(args.model, device="cuda",
                     dtype=getattr(torch, args.dtype))
    if not getattr(model, "packed", False):
        print(f"trace_run: {model.cfg.arch} has no packed batches",
              file=sys.stderr)
        return 2
    st = PackedStepper(model, args.max_tokens)
    for line in sys.stdin:
        if not line.strip():
            continue
        s = json.loads(line)
        logits = st.step([(e["id"], e["tokens"], e["want"])
                          for e in s["entries"]])
        if logits.shape[0]:
            logits.float().cpu().numpy().astype("<f4").tofile(
                os.path.join(args.out, f"{s['step']}.f32"))
        st.end(s.get("end", []))
        print(f"done {s['step']}", flush=True)
    return 0
