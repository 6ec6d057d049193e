"""Trace replay: drives a model with token ids that are already known and records logits.

Every input line is one step, a JSON object with
    step      its number
    entries   list of {"id", "tokens", "want"}: the request, the tokens to append to it, and the indexes into those tokens
              where logits are to be recorded
    end       ids whose requests are over once the step has run
A step that records anything leaves <out>/<step>.f32, raw little-endian fp32 rows of vocabulary length in input order, and
each step is acknowledged with the line "done <step>".  A single token runs as a decode step, several as a prompt chunk: the
calls that generation makes."""
from __future__ import annotations

import argparse
import json
import os
import sys

import numpy as np

from . import model as registry


class Replay:
    """One decoder and the request its cache currently holds."""

    def __init__(self, model):
        self.model = model
        self.live = None 

    def run(self, request_id, tokens, want) -> np.ndarray:
        if self.live is None:
            self.model.set_past_len(0)
            self.live = request_id
        elif self.live != request_id:
            raise RuntimeError("request %r starts while %r is live: a decoder holds one sequence" % (request_id, self.live))
        if len(tokens) == 1:
            self.model.step(int(tokens[0]))
            logits = self.model.logits() if want else None
            return np.stack([logits for _ in want]) if want else np.empty((0, self.model.cfg["vocab"]), np.float32)
        places = sorted(set(want))
        rows = self.model.prefill_logits(tokens, places)
        return rows[[places.index(w) for w in want]]

    def end(self, request_id) -> None:
        if self.live == request_id:
            self.live = None


def main(argv=None) -> int:
    ap = argparse.ArgumentParser(prog="trace_run", description="Replay token ids through a model and record logits.")
    ap.add_argument("--model", required=True, help="model folder (config.json, model.safetensors) or .gguf file")
    ap.add_argument("--dtype", required=True, choices=sorted(registry.PRECISIONS))
    ap.add_argument("--out", required=True, help="where the logits files go")
    ap.add_argument("--max-tokens", type=int, required=True, help="context the cache is sized for")
    a = ap.parse_args(argv)
    if a.max_tokens <= 0:
        ap.error("--max-tokens must be positive")
    os.makedirs(a.out, exist_ok=True)
    model = registry.load(a.model, max_seq=a.max_tokens + 1, precision=a.dtype)
    replay = Replay(model)
    for line in sys.stdin:
        if not line.strip():
            continue
        step = json.loads(line)
        got = [replay.run(e["id"], e["tokens"], e["want"]) for e in step["entries"]]
        if any(len(g) for g in got):
            np.concatenate(got).astype("<f4").tofile(os.path.join(a.out, "%d.f32" % step["step"]))
        for r in step["end"]:
            replay.end(r)
        print("done %d" % step["step"], flush=True)
    model.close()
    return 0
