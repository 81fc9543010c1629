"""Replays a trace of given token ids through a model, step by step, and writes the logits asked for.

    bin/trace_run --model DIR --dtype bfloat16|float32 --out DIR --max-tokens N

Standard input holds one JSON object a line: {"step": n, "entries": [{"id", "tokens", "want"}], "end": [ids]}.  An entry's tokens continue
its request; `want` lists the places among them whose logits go to OUT/n.f32 (little-endian f32, [wanted, vocab]).  'done n' is printed
after every step.  One request runs at a time: what an ended request held is given back before the next one starts.
"""
from __future__ import annotations

import argparse
import fcntl
import json
import os
import sys


def _ensure_built() -> None:
    """Compile the library these models run on, if it is missing or out of date (one process at a time)."""
    from . import build
    os.makedirs(build.OBJ, exist_ok=True)
    with open(os.path.join(build.OBJ, "build.lock"), "w") as lock:
        fcntl.flock(lock, fcntl.LOCK_EX)
        build.build_mixer()


class Replay:
    def __init__(self, model, out: str):
        self.model, self.out = model, out
        self.current = None                          # id of the live request

    def step(self, msg: dict) -> None:
        if len(msg["entries"]) > 1:
            raise ValueError("a step holds one entry: the model serves one sequence")
        for e in msg["entries"]:
            if e["id"] != self.current:
                if self.current is not None:
                    raise ValueError(f"request {e['id']} starts before {self.current} has ended")
                self.model.reset()
                self.current = e["id"]
            logits = self.model.step(e["tokens"], e["want"])
            if e["want"]:
                logits.cpu().numpy().astype("<f4").tofile(os.path.join(self.out, f"{msg['step']}.f32"))
        for name in msg.get("end", []):
            if name == self.current:
                self.model.reset()
                self.current = None


def main(argv=None) -> None:
    ap = argparse.ArgumentParser(prog="trace_run", description="replay a trace of token ids and write logits")
    ap.add_argument("--model", required=True, help="folder with config.json and model.safetensors")
    ap.add_argument("--dtype", choices=["bfloat16", "float32"], default="bfloat16")
    ap.add_argument("--out", required=True, help="folder for the <step>.f32 files")
    ap.add_argument("--max-tokens", type=int, required=True, help="the most tokens a request holds")
    a = ap.parse_args(argv)
    _ensure_built()
    from .registry import load_model
    replay = Replay(load_model(a.model, dtype=a.dtype, ctx=max(a.max_tokens, 1)), a.out)
    for line in sys.stdin:
        if line.strip():
            msg = json.loads(line)
            replay.step(msg)
            print(f"done {msg['step']}", flush=True)


if __name__ == "__main__":
    main()
