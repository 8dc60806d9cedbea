"""Replays a trace of token ids through a model, step by step, and writes logits (bin/trace_run).

Steps come on standard input, one JSON object a line:
    {"step": 0, "entries": [{"id": "a", "tokens": [5, 17, 3], "want": [0, 2]}], "end": []}
An entry gives a request's next tokens and the places among them whose logits are asked for; "end" lists the requests that
are over after the step.  A step that wants logits writes <out>/<step>.f32 (float32, [wanted][vocab], in the order of the
entries and of their places); after every step a line "done <step>" is printed."""
import argparse
import json
import os
import sys

import numpy as np


def run_entry(model, entry):
    """Logits of an entry's wanted places, in their order."""
    slot = model.pool.slot(entry["id"])
    want = entry.get("want") or []
    places = sorted(set(want))
    logits = model.step(slot, entry["tokens"], places)
    return logits[[places.index(w) for w in want]] if want else None


def main(argv=None):
    ap = argparse.ArgumentParser(prog="trace_run")
    ap.add_argument("--model", required=True, help="folder with config.json and model.safetensors")
    ap.add_argument("--dtype", required=True, choices=("bfloat16", "float32"))
    ap.add_argument("--out", required=True, help="folder for the logits")
    ap.add_argument("--max-tokens", type=int, required=True, help="most tokens that live requests hold at any time")
    ap.add_argument("--slots", type=int, default=1, help="requests that may be live at once")
    a = ap.parse_args(argv)
    from .registry import load_model
    model = load_model(a.model, dtype=a.dtype, max_pos=max(a.max_tokens, 1), slots=a.slots)
    for line in sys.stdin:
        if not line.strip():
            continue
        step = json.loads(line)
        parts = [run_entry(model, e) for e in step["entries"] if e["tokens"]]
        parts = [p for p in parts if p is not None]
        model.check()
        if parts:
            np.concatenate(parts).astype("<f4").tofile(os.path.join(a.out, "%d.f32" % step["step"]))
        for key in step.get("end") or []:
            if key in model.pool:
                model.pool.release(key)
        print("done %d" % step["step"], flush=True)
    model.close()
    return 0
