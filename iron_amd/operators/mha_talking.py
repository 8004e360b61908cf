"""Attention within chunks whose heads' weights are mixed behind the softmax, over a batch of spans: TurnedHeads makes a packed
projection's rows ready, TalkingMHA attends them.
"""

from __future__ import annotations

from typing import Any

import numpy as np

from ..bf16 import bfloat16
from ..common.declare import Built, In, InOut, Operator, Out, Scratch, param, per_call
from ..common.verify import Tolerance

F32 = np.float32


class TurnedHeads(Operator):
    """Rows ``[q heads | k heads | v heads]``, biased: q and k RMS-normed a head, their first ``turned`` columns turned in
    neighbouring pairs by their position's row of ``angles`` (cos and sin side by side), q times ``scale * temp[head]``; v
    blended, with ``first``, to ``(1 - share) v + share first``, ``first``'s columns ``first_at ..``."""

    slots: int = param()
    rows: int = param()
    stride: int = param()
    heads: int = param()
    kv_heads: int = param()
    dim: int = param()
    vdim: int = param(derive=lambda op: (op.stride - (op.heads + op.kv_heads) * op.dim) // op.kv_heads, repr=False)
    turned: int = param(default=0)
    turns: bool = param(derive=lambda op: op.turned > 0, repr=False)
    angle_rows: int = param(default=1, array=True)
    mixed: bool = param(default=False, repr=False)
    first_stride: int = param(default=0)
    first_at: int = param(default=0, array=True)
    scale: float = param(array=True)
    epsilon: float = param(array=True)
    dtype: Any = param(default=bfloat16, repr=False)
    x = In(rows, stride, dtype=dtype)
    bias = In(stride)
    q_gain = In(dim)
    k_gain = In(dim)
    temp = In(heads)
    spans = In(slots, 4, dtype=np.int32)
    angles = In(angle_rows, turned, dtype=F32, when=turns)
    first = In(rows, first_stride, dtype=dtype, when=mixed)
    share = In(1, when=mixed)
    y = Out(rows, stride, dtype=dtype)
    valid = per_call(bounds=rows)

    @classmethod
    def infer(cls, shapes, **kw):
        out = dict(slots=shapes["spans"][0], rows=shapes["x"][0], stride=shapes["x"][1], heads=shapes["temp"][0], dim=shapes["q_gain"][0],
                   mixed="first" in shapes, **kw)
        if "angles" in shapes:
            out |= dict(angle_rows=shapes["angles"][0], turned=shapes["angles"][1])
        if "first" in shapes:
            out["first_stride"] = shapes["first"][1]
        return out

    def validate(self):
        if self.vdim < 1 or self.stride != (self.heads + self.kv_heads) * self.dim + self.kv_heads * self.vdim:
            raise ValueError(f"TurnedHeads: a row of {self.stride} is not {self.heads} + {self.kv_heads} heads of {self.dim} and values")
        if self.turned > self.dim or self.turned % 2:
            raise ValueError(f"TurnedHeads: {self.turned} of {self.dim} columns turn in pairs")
        if self.mixed and not 0 <= self.first_at <= self.first_stride - self.kv_heads * self.vdim:
            raise ValueError(f"TurnedHeads: {self.kv_heads * self.vdim} values from column {self.first_at} of a row of {self.first_stride}")

    def tolerance(self):
        return Tolerance.relative(1e-2, 1e-2, note="float32, rounded once")

    def build(self) -> Built:
        from .. import kernels

        kw = {n: getattr(self, n) for n in ("slots", "rows", "stride", "heads", "kv_heads", "dim", "vdim", "turned", "angle_rows",
                                            "first_stride", "first_at")}
        kw |= dict(scale=float(self.scale), eps=float(self.epsilon))

        def launch(t, words):
            kernels.turned_heads(t["x"], t["y"], t["bias"], t["q_gain"], t["k_gain"], t["temp"], t["spans"], angles=t.get("angles"),
                                 share=t.get("share"), first=t.get("first"), valid=words.get("valid"), **kw)

        return Built("iron_turned_heads", launch)


class TalkingMHA(Operator):
    """Rows ``x`` are ``[q heads | k heads | v heads]``, scores ready as ``q . k``.  Position i sees the ``j <= i`` with
    ``j // chunk == i // chunk``; softmax a head; head h's weights become ``sum_g talk[h, g] weight_g`` and weigh its own
    values.  Position p's key and value live in row ``p % chunk`` of the slot's ring.  ``single``: every span is one row at
    most (a decode step)."""

    slots: int = param()
    rows: int = param()
    stride: int = param()
    heads: int = param()
    kv_heads: int = param()
    dim: int = param()
    vdim: int = param()
    chunk: int = param()
    width: int = param(derive=lambda op: op.heads * op.vdim, repr=False)
    single: bool = param(default=False)
    dtype: Any = param(default=bfloat16, repr=False)
    x = In(rows, stride, dtype=dtype)
    talk = In(heads, heads)
    spans = In(slots, 4, dtype=np.int32)
    keys = InOut(slots, chunk, kv_heads, dim, dtype=dtype)
    values = InOut(slots, chunk, kv_heads, vdim, dtype=dtype)
    y = Out(rows, width, dtype=dtype)
    workspace_words: int = param(derive=lambda op: op._workspace_words(), repr=False)
    workspace = Scratch(workspace_words, dtype=F32)
    valid = per_call(bounds=rows)

    def _workspace_words(self) -> int:
        from .._lib import lib

        return int(lib().iron_mha_talking_workspace_bytes(self.slots, self.rows, self.heads, self.vdim, self.chunk, int(self.single))) // 4

    @classmethod
    def infer(cls, shapes, **kw):
        slots, chunk, kv_heads, dim = shapes["keys"]
        return dict(slots=slots, rows=shapes["x"][0], stride=shapes["x"][1], heads=shapes["talk"][0], kv_heads=kv_heads, dim=dim,
                    vdim=shapes["values"][3], chunk=chunk, **kw)

    def validate(self):
        if self.heads % self.kv_heads:
            raise ValueError(f"TalkingMHA: kv_heads ({self.kv_heads}) must divide heads ({self.heads})")

    def tolerance(self):
        return Tolerance.relative(4e-2, 4e-2, note="float32 scores and weights")

    def build(self) -> Built:
        from .. import kernels

        kw = {n: getattr(self, n) for n in ("slots", "rows", "stride", "heads", "kv_heads", "dim", "vdim", "chunk", "single")}
        kw["ring"] = self.chunk

        def launch(t, words):
            kernels.mha_talking(t["x"], t["keys"], t["values"], t["talk"], t["spans"], t["y"], t["workspace"], **kw)

        return Built("iron_mha_talking", launch)
