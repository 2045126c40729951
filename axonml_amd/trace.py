"""Replays a trace of token ids through a model and writes the logits it asks for.

    python -m axonml_amd trace --model DIR --dtype bfloat16|float32 --out DIR --max-tokens N

Standard input holds one step per line: {"step": 0, "entries": [{"id": "a", "tokens": [..], "want": [..]}], "end": [..]}.
A step feeds its entry's tokens behind what the request has had; `want` lists the places among them whose logits go to
OUT/<step>.f32 (little-endian f32, [wanted, vocab]); `end` lists the requests that are finished.  After every step a line
"done <step>" is printed.  Nothing is sampled.
"""
import argparse
import json
import os
import sys

import numpy as np

from .registry import load_model


class Replay:
    """Feeds requests, one after the other, to a model that holds one sequence."""

    def __init__(self, model):
        self.model, self.live = model, None

    def step(self, entries, end):
        out = []
        for e in entries:
            if self.live is None:
                self.model.reset()
                self.live = e["id"]
            if e["id"] != self.live:
                raise ValueError(f"request {e['id']!r} while {self.live!r} is live: one request at a time")
            want = [int(w) for w in e.get("want", [])]
            order = sorted(set(want))
            rows = self.model.feed([int(t) for t in e["tokens"]], order)
            out.append(rows[[order.index(w) for w in want]])
        if self.live in end:
            self.model.reset()
            self.live = None
        return np.concatenate(out) if out else np.empty((0, self.model.vocab_size), np.float32)


def run(model, lines, out_dir, report):
    replay = Replay(model)
    for line in lines:
        if not line.strip():
            continue
        s = json.loads(line)
        logits = replay.step(s["entries"], s.get("end", []))
        if logits.shape[0]:
            logits.astype("<f4").tofile(os.path.join(out_dir, f"{s['step']}.f32"))
        report(f"done {s['step']}")


def add_arguments(ap):
    ap.add_argument("--model", required=True, help="directory with config.json and model.safetensors")
    ap.add_argument("--dtype", choices=("bfloat16", "float32"), default="bfloat16")
    ap.add_argument("--out", required=True, help="directory for the logits")
    ap.add_argument("--max-tokens", type=int, default=None, help="the most tokens a request holds (sizes the cache)")


def main(args):
    model = load_model(args.model, dtype=args.dtype, max_positions=args.max_tokens)
    run(model, sys.stdin, args.out, lambda text: print(text, flush=True))
    model.close()
    return 0


if __name__ == "__main__":
    ap = argparse.ArgumentParser(description="replay a trace of token ids through a model")
    add_arguments(ap)
    sys.exit(main(ap.parse_args()))
