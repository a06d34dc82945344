"""Trace runner: feeds given token ids through a model step by step and writes logits; samples nothing.

Steps come on standard input, one JSON object a line:

    {"step": 0, "entries": [{"id": "a", "tokens": [5, 17, 3], "want": [0, 2]}], "end": []}

An entry brings a request's next tokens and the places among them whose logits are wanted; "end" names the requests
that are finished after the step.  A step in which something is wanted writes <out>/<step>.f32 (little-endian floats,
[wanted, vocab], in the order of entries and of "want"); after every step a line "done <step>" is printed.  The models of
this package hold one live sequence, so requests come one after the other.
"""
import argparse
import json
import os
import sys

import numpy as np

from .registry import load_model


def run_step(model, live, step, out_dir):
    """One step; returns the id of the live request after it (or None)."""
    rows = []
    for entry in step["entries"]:
        if live is not None and live != entry["id"]:
            raise ValueError("request %r starts before %r has ended" % (entry["id"], live))
        live = entry["id"]
        want = np.asarray(entry["want"], np.int64)
        places, back = np.unique(want, return_inverse=True)
        rows.append(model.step(entry["tokens"], places)[back.reshape(-1)])
    if sum(len(r) for r in rows):
        np.concatenate(rows).astype("<f4").tofile(os.path.join(out_dir, "%d.f32" % step["step"]))
    if live is not None and live in step.get("end", ()):
        model.reset()
        live = None
    return live


def main(argv=None):
    ap = argparse.ArgumentParser(prog="trace_run", description="replay a trace of token ids and write logits")
    ap.add_argument("--model", required=True, help="folder with config.json and model.safetensors")
    ap.add_argument("--dtype", choices=["bfloat16", "float32"], required=True, help="storage of the weights")
    ap.add_argument("--out", required=True, help="folder for <step>.f32")
    ap.add_argument("--max-tokens", type=int, required=True, help="the most tokens a live request holds")
    args = ap.parse_args(argv)
    model = load_model(args.model, args.dtype, args.max_tokens)
    live = None
    for line in sys.stdin:
        if not line.strip():
            continue
        step = json.loads(line)
        live = run_step(model, live, step, args.out)
        print("done %d" % step["step"], flush=True)
    return 0
