"""Replays recorded token ids: runs them through a model step by step, without
sampling, and writes the logits that the recording asks for.  Every step is an
ordinary pass of the model over new tokens, on the cache earlier steps left.

    bin/trace_run --model FOLDER --dtype float32 --out LOGITS --max-tokens 4096 < STEPS

Standard input holds one JSON object per line, for instance

    {"step": 7, "entries": [{"id": "chat-2", "tokens": [311, 40], "want": [1]}], "end": ["chat-2"]}

"tokens" continues the request "id"; "want" numbers the tokens of this entry
whose logits go to LOGITS/<step>.f32 (raw little-endian floats, one row of the
vocabulary each; no file without any).  "done <step>" on standard output follows
every step.  "end" closes requests.  A model holds one sequence, so requests
follow one another, each on the cache rows of the one before.
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
