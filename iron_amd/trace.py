"""Replaying a trace: given token ids through a model, step by step, logits out; nothing is sampled.

``bin/trace_run --model DIR --dtype bfloat16|float32 --out DIR [--max-tokens N]`` reads steps from
standard input, one JSON object a line::

    {"step": 7, "entries": [{"id": "r1", "tokens": [210, 9, 31, 4], "want": [3]}], "end": ["r0"]}

``entries`` are the requests' next tokens, run as one batch after what each request holds; ``want`` the
places among them whose logits are wanted; ``end`` the requests that are over after this step.  A step
that wants logits writes ``DIR/<step>.f32``: float32, little-endian, ``[wanted, vocab]``, in the order of
the entries.  Every step ends with a line ``done <step>`` on standard output.
"""

from __future__ import annotations

import argparse
import json
import sys
from pathlib import Path

import numpy as np

REFUSED = 3   # exit code where the model cannot run in the asked-for type

# Positions a request is served where nothing says how many it will hold.
DEFAULT_TOKENS = 8192


def _fail(message: str, code: int = 2) -> int:
    print(f"trace_run: {message}", file=sys.stderr)
    return code


class Replay:
    """The model behind a trace, built for as many requests at once as the trace brings: a batch that is
    larger than any before it, on which nothing is live yet, has the model built again with more slots."""

    def __init__(self, folder, dtype: str, max_tokens: int):
        from .applications import model_class

        self.folder, self.max_tokens = folder, max_tokens
        self.cls = model_class(folder)
        self.options = {} if dtype == "bfloat16" else {"activations": np.float32}
        self.model = None

    def serve(self, requests: int):
        if self.model is not None and (self.model.config.slots >= requests or self.model.batch.slots):
            return self.model.batch
        if self.model is not None:
            self.model.release()
        self.model = self.cls.load(self.folder, slots=requests, max_seq_len=self.max_tokens, **self.options)
        return self.model.batch

    def step(self, step: dict) -> np.ndarray | None:
        from .lm.batched import Entry

        entries = [Entry(e["id"], e["tokens"], e.get("want") or ()) for e in step.get("entries", ())]
        rows = []
        if entries:
            batch = self.serve(len(entries))
            rows = [r for r in batch.step(entries) if len(r)]
        for key in step.get("end") or ():
            self.model.batch.end(key)
        return np.concatenate(rows) if rows else None


def main(argv=None) -> int:
    ap = argparse.ArgumentParser(prog="trace_run", description="Replay a trace of token ids and write the logits it asks for.")
    ap.add_argument("--model", required=True, help="a folder with config.json and model.safetensors")
    ap.add_argument("--dtype", required=True, choices=("bfloat16", "float32"), help="what activations are computed in")
    ap.add_argument("--out", required=True, help="folder the logits are written to")
    ap.add_argument("--max-tokens", type=int, default=DEFAULT_TOKENS, help="the most tokens live requests hold at any time")
    args = ap.parse_args(argv)

    from . import _lib
    from .build import build

    if not _lib.LIB_PATH.exists():
        build()
    from .lm.batched import BatchedLM

    out = Path(args.out)
    replay = Replay(args.model, args.dtype, args.max_tokens)
    if not issubclass(replay.cls, BatchedLM):
        return _fail(f"{replay.cls.__name__} serves one sequence at a time and gives the last token's logits only",
                     REFUSED if args.dtype == "float32" else 2)
    for line in sys.stdin:
        if not line.strip():
            continue
        step = json.loads(line)
        rows = replay.step(step)
        if rows is not None:
            np.ascontiguousarray(rows, dtype="<f4").tofile(out / f"{step['step']}.f32")
        print(f"done {step['step']}", flush=True)
    return 0
