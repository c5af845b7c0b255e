"""Replays a trace: feeds given token ids through a model step by step and writes
logits.  Nothing is sampled; every step is a pass of the model over the tokens
it brings, on the cache that earlier steps left.

    bin/trace_run --model DIR --dtype bfloat16|float32 --out DIR --max-tokens N

Steps come on standard input, one JSON object a line:

    {"step": 0, "entries": [{"id": "a", "tokens": [5, 17, 3], "want": [0, 2]}], "end": []}

An entry brings a request's next tokens and names the places among them whose
logits are wanted; "end" lists the requests that are finished.  The logits of a
step go to OUT/<step>.f32 (little-endian floats [wanted, vocab], no file if
nothing is wanted), then a line "done <step>" is printed.  A model holds one
sequence: requests follow one another, and a request that ends gives its cache
rows to the next.
"""
import argparse
import json
import os
import sys

import numpy as np


class Replay:
    """One sequence at a time through a loaded model."""

    def __init__(self, model):
        self.model = model
        self.live = None
        self.pos = 0

    def run(self, entries, end):
        """Logits [wanted, vocab] of the entries' wanted places, in order."""
        out = []
        for e in entries:
            if self.live is None:
                self.live, self.pos = e["id"], 0
            elif self.live != e["id"]:
                raise ValueError("request %r comes before %r has ended: a model holds one sequence"
                                 % (e["id"], self.live))
            if e["tokens"]:
                out.append(self.model.forward_rows(e["tokens"], self.pos, e["want"]))
                self.pos += len(e["tokens"])
        if self.live in end:
            self.live = None
        return np.concatenate(out) if out else np.empty((0, 0), np.float32)


def main(argv=None):
    ap = argparse.ArgumentParser(description=__doc__, formatter_class=argparse.RawDescriptionHelpFormatter)
    ap.add_argument("--model", required=True, help="folder with config.json and model.safetensors, or a GGUF file")
    ap.add_argument("--dtype", choices=("bfloat16", "float32"), default=None)
    ap.add_argument("--out", required=True, help="folder for the logits")
    ap.add_argument("--max-tokens", type=int, default=0, help="most tokens a live request holds")
    ap.add_argument("--device", type=int, default=0)
    args = ap.parse_args(argv)

    from . import build
    build.ensure_built()
    from . import model as M
    os.makedirs(args.out, exist_ok=True)
    m = M.CausalModel.load(args.model, args.dtype, args.max_tokens, args.device)
    replay = Replay(m)
    for line in sys.stdin:
        if not line.strip():
            continue
        step = json.loads(line)
        logits = replay.run(step.get("entries", []), step.get("end", []))
        if logits.shape[0]:
            logits.astype("<f4", copy=False).tofile(os.path.join(args.out, "%d.f32" % step["step"]))
        print("done %d" % step["step"], flush=True)
    m.close()
    return 0
