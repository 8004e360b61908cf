"""A feed-forward of routed experts: Router chooses a row's, Experts is what they make of it."""

from __future__ import annotations

from typing import Any

import numpy as np

from ..bf16 import bfloat16
from ..common.declare import Built, In, Operator, Out, Scratch, param, per_call
from ..common.verify import Tolerance

F32 = np.float32


class Router(Operator):
    """The ``top`` experts with the largest ``weight h + bias`` (float32) of each row, and their shares: a softmax over the
    chosen logits alone.  ``scored``: those with the largest softmax score (over all logits) plus ``correction``, and their
    shares, the scores over their sum."""

    rows: int = param()
    cols: int = param()
    experts: int = param()
    top: int = param()
    scored: bool = param(default=False, repr=False)
    biased: bool = param(default=True, repr=False)
    corrected: bool = param(default=False, repr=False)
    dtype: Any = param(default=bfloat16, repr=False)
    h = In(rows, cols, dtype=dtype)
    weight = In(experts, cols)
    bias = In(experts, when=biased)
    correction = In(experts, when=corrected)
    ids = Out(rows, top, dtype=np.int32)
    shares = Out(rows, top, dtype=F32)
    valid = per_call(bounds=rows)

    @classmethod
    def infer(cls, shapes, **kw):
        return dict(rows=shapes["h"][0], cols=shapes["h"][1], experts=shapes["weight"][0], biased="bias" in shapes, corrected="correction" in shapes, **kw)

    def validate(self):
        if self.corrected and not self.scored:
            raise ValueError("Router: corrections are of scores")
        if not 1 <= self.top <= min(self.experts, 64) or self.experts > 1024:
            raise ValueError(f"Router: top ({self.top}) from 1 to the experts ({self.experts}), 64 at most of 1024")

    def tolerance(self):
        return Tolerance.relative(1e-3, 1e-4, note="float32")

    def build(self) -> Built:
        from .. import kernels

        kw = dict(rows=self.rows, cols=self.cols, experts=self.experts, top=self.top, scored=self.scored)

        def launch(t, words):
            kernels.router(t["h"], t["weight"], t.get("bias"), t["ids"], t["shares"], correction=t.get("correction"), valid=words.get("valid"), **kw)

        return Built("iron_router", launch)


class Experts(Operator):
    """``sum over a row's experts e of share * down_e (act(gate_e h) * (up_e h))``; the experts' matrices are stacked.
    ``identity``: that many ids behind the experts' last stand for ``h`` itself."""

    rows: int = param()
    cols: int = param()
    experts: int = param()
    top: int = param()
    ff: int = param()
    activation: str = param()
    identity: int = param(default=0)
    stacked: int = param(derive=lambda op: op.experts * op.ff, repr=False)
    tall: int = param(derive=lambda op: op.experts * op.cols, repr=False)
    dtype: Any = param(default=bfloat16, repr=False)
    h = In(rows, cols, dtype=dtype)
    gate = In(stacked, cols)
    up = In(stacked, cols)
    down = In(tall, ff)
    ids = In(rows, top, dtype=np.int32)
    shares = In(rows, top, dtype=F32)
    y = Out(rows, cols, dtype=dtype)
    workspace_words: int = param(derive=lambda op: op._workspace_words(), repr=False)
    workspace = Scratch(workspace_words, dtype=F32)
    valid = per_call(bounds=rows)

    def _workspace_words(self) -> int:
        from .._lib import lib

        return -(-int(lib().iron_experts_workspace_bytes(self.rows, self.cols, self.ff, self.experts, self.top,
                                                         int(self.dtype is not bfloat16))) // 4)

    @classmethod
    def infer(cls, shapes, **kw):
        rows, cols = shapes["h"]
        tall, ff = shapes["down"]
        return dict(rows=rows, cols=cols, experts=tall // cols, ff=ff, top=shapes["ids"][1], **kw)

    def validate(self):
        if self.identity < 0 or not 1 <= self.top <= self.experts + self.identity:
            raise ValueError(f"Experts: top ({self.top}) from 1 to {self.experts} experts and {self.identity} identities")

    def ops(self) -> int:
        return 6 * self.rows * self.top * self.cols * self.ff

    def tolerance(self):
        return Tolerance.relative(2e-2, 2e-2, note="float32 sums, products and result rounded")

    def build(self) -> Built:
        from .. import kernels

        kw = {n: getattr(self, n) for n in ("rows", "cols", "ff", "experts", "identity", "top", "activation")}

        def launch(t, words):
            kernels.experts(t["h"], t["gate"], t["up"], t["down"], t["ids"], t["shares"], t["y"], t["workspace"], valid=words.get("valid"), **kw)

        return Built("iron_experts", launch)
