"""Causal attention over whole sequences, a batch of spans and a cache a slot: CachedHeads makes a packed projection's rows ready
and keeps their keys and values, GlobalMHA attends what is kept.
"""

from __future__ import annotations

from typing import Any

import numpy as np

from ..bf16 import bfloat16
from ..common.declare import Built, In, InOut, Operator, Out, Scratch, param, per_call
from ..common.verify import Tolerance

F32 = np.float32


class CachedHeads(Operator):
    """Rows ``[q heads | k heads | v heads | ..]``: q and k RMS-normed a head, columns ``i`` and ``i + turned / 2`` of their first
    ``turned`` turned together by their position's row of ``angles`` (cos and sin side by side, multiplied in as they are);
    ``value_norm``: v over its root mean square a head.  Position p's key and value go to row p of their head's cache."""

    slots: int = param()
    rows: int = param()
    stride: int = param()
    heads: int = param()
    kv_heads: int = param()
    dim: int = param()
    vdim: int = param()
    context: int = param()
    inner: int = param(derive=lambda op: op.heads * op.dim, repr=False)
    turned: int = param(default=0)
    turns: bool = param(derive=lambda op: op.turned > 0, repr=False)
    angle_rows: int = param(default=1, array=True)
    value_norm: bool = param(default=False)
    epsilon: float = param(array=True)
    dtype: Any = param(default=bfloat16, repr=False)
    x = In(rows, stride, dtype=dtype)
    q_gain = In(dim)
    k_gain = In(dim)
    spans = In(slots, 4, dtype=np.int32)
    keys = InOut(slots, kv_heads, context, dim, dtype=dtype)
    values = InOut(slots, kv_heads, context, vdim, dtype=dtype)
    angles = In(angle_rows, turned, dtype=F32, when=turns)
    q = Out(rows, inner, dtype=dtype)
    valid = per_call(bounds=rows)

    @classmethod
    def infer(cls, shapes, **kw):
        slots, kv_heads, context, dim = shapes["keys"]
        turn = dict(angle_rows=shapes["angles"][0], turned=shapes["angles"][1]) if "angles" in shapes else {}
        return dict(slots=slots, rows=shapes["x"][0], stride=shapes["x"][1], kv_heads=kv_heads, dim=dim, vdim=shapes["values"][3], context=context,
                    **turn, **kw)

    def validate(self):
        if (self.heads + self.kv_heads) * self.dim + self.kv_heads * self.vdim > self.stride:
            raise ValueError(f"CachedHeads: a row of {self.stride} holds no {self.heads} + {self.kv_heads} heads of {self.dim} and values of {self.vdim}")
        if self.turned > self.dim or self.turned % 2:
            raise ValueError(f"CachedHeads: {self.turned} of {self.dim} columns turn in pairs")

    def tolerance(self):
        return Tolerance.relative(1e-2, 1e-2, note="float32, rounded once")

    def build(self) -> Built:
        from .. import kernels

        kw = {n: getattr(self, n) for n in ("slots", "rows", "stride", "heads", "kv_heads", "dim", "vdim", "context", "turned", "angle_rows",
                                            "value_norm")}
        kw["eps"] = float(self.epsilon)

        def launch(t, words):
            kernels.cached_heads(t["x"], t["q"], t["keys"], t["values"], t["q_gain"], t["k_gain"], t["spans"], angles=t.get("angles"),
                                 valid=words.get("valid"), **kw)

        return Built("iron_cached_heads", launch)


class GlobalMHA(Operator):
    """Position i sees every ``j <= i`` of its slot's cache, its own row among them: score ``q . k * scale``, with ``cap`` above 0
    ``cap tanh(score / cap)``; softmax, with ``sink`` one more in its denominator.  The heads' values go to columns ``at ..`` of a
    row of ``width``.  ``single``: every span is one row at most (a decode step)."""

    slots: int = param()
    rows: int = param()
    heads: int = param()
    kv_heads: int = param()
    dim: int = param()
    vdim: int = param()
    context: int = param()
    inner: int = param(derive=lambda op: op.heads * op.dim, repr=False)
    width: int = param()
    at: int = param(default=0, array=True)
    scale: float = param(array=True)
    cap: float = param(default=0.0, array=True)
    sink: bool = param(default=False)
    single: bool = param(default=False)
    dtype: Any = param(default=bfloat16, repr=False)
    q = In(rows, inner, dtype=dtype)
    keys = In(slots, kv_heads, context, dim, dtype=dtype)
    values = In(slots, kv_heads, context, vdim, dtype=dtype)
    spans = In(slots, 4, dtype=np.int32)
    y = Out(rows, width, dtype=dtype)
    workspace_words: int = param(derive=lambda op: op._workspace_words(), repr=False)
    workspace = Scratch(workspace_words, dtype=F32, when=single)
    valid = per_call(bounds=rows)

    def _workspace_words(self) -> int:
        from .._lib import lib

        return max(1, int(lib().iron_mha_global_workspace_bytes(self.slots, self.heads, self.kv_heads, self.vdim, self.context, int(self.single))) // 4)

    @classmethod
    def infer(cls, shapes, **kw):
        slots, kv_heads, context, dim = shapes["keys"]
        heads, vdim = shapes["q"][1] // dim, shapes["values"][3]
        return {"slots": slots, "rows": shapes["q"][0], "heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "context": context,
                "width": heads * vdim, **kw}

    def validate(self):
        if self.heads % self.kv_heads:
            raise ValueError(f"GlobalMHA: kv_heads ({self.kv_heads}) must divide heads ({self.heads})")
        if not (1 <= self.dim <= 256 and 1 <= self.vdim <= 256):
            raise ValueError(f"GlobalMHA: dim ({self.dim}) and vdim ({self.vdim}) from 1 to 256")
        if self.cap < 0 or not 0 <= self.at <= self.width - self.heads * self.vdim:
            raise ValueError(f"GlobalMHA: a cap ({self.cap}) not negative, {self.heads * self.vdim} columns from {self.at} of a row of {self.width}")

    def ops(self) -> int:
        return self.heads * (self.dim + self.vdim) * self.rows * (self.rows + 1)

    def tolerance(self):
        return Tolerance.relative(4e-2, 4e-2, note="float32 scores and weights")

    def build(self) -> Built:
        from .. import kernels

        kw = {n: getattr(self, n) for n in ("slots", "rows", "heads", "kv_heads", "dim", "vdim", "context", "sink", "single")}
        kw |= dict(scale=float(self.scale), cap=float(self.cap), out_stride=self.width, out_at=self.at)

        def launch(t, words):
            kernels.mha_global(t["q"], t["keys"], t["values"], t["spans"], t["y"], workspace=t.get("workspace"), **kw)

        return Built("iron_mha_global", launch)
