"""Latent attention over a batch of spans: LatentRows leaves a position's normed latent (and its part of a
key that all heads share) in a ring a slot, LatentMHA attends them.
"""

from __future__ import annotations

from typing import Any

import numpy as np

from ..bf16 import bfloat16
from ..common.declare import Built, In, InOut, Operator, Out, Scratch, param, per_call
from ..common.verify import Tolerance

F32 = np.float32
EVERYTHING = 1 << 30   # a window that hides nothing


class LatentRows(Operator):
    """Rows ``[query latent | latent | shared key part | ..]`` of a packed projection: both latents RMS-normed,
    the first ``turned`` columns of the key part turned in neighbouring pairs by their position's row of
    ``angles`` (cos and sin side by side).  Position p's latent and key part go to row ``p % ring``."""

    slots: int = param()
    rows: int = param()
    stride: int = param()
    q_rank: int = param()
    rank: int = param()
    rot: int = param(default=0)
    shared: bool = param(derive=lambda op: op.rot > 0, repr=False)
    turned: int = param(default=0)
    turns: bool = param(derive=lambda op: op.turned > 0, repr=False)
    angle_rows: int = param(default=0, array=True)
    ring: int = param()
    epsilon: float = param(array=True)
    dtype: Any = param(default=bfloat16, repr=False)
    x = In(rows, stride, dtype=dtype)
    q_gain = In(q_rank)
    c_gain = In(rank)
    spans = In(slots, 4, dtype=np.int32)
    latents = InOut(slots, ring, rank, dtype=dtype)
    shared_keys = InOut(slots, ring, rot, dtype=dtype, when=shared)
    angles = In(angle_rows, turned, dtype=F32, when=turns)
    q = Out(rows, q_rank, dtype=dtype)
    valid = per_call(bounds=rows)

    @classmethod
    def infer(cls, shapes, **kw):
        out = dict(slots=shapes["spans"][0], rows=shapes["x"][0], stride=shapes["x"][1], q_rank=shapes["q_gain"][0],
                   rank=shapes["c_gain"][0], ring=shapes["latents"][1], **kw)
        if "shared_keys" in shapes:
            out["rot"] = shapes["shared_keys"][2]
        if "angles" in shapes:
            out |= dict(angle_rows=shapes["angles"][0], turned=shapes["angles"][1])
        return out

    def validate(self):
        if self.q_rank + self.rank + self.rot > self.stride:
            raise ValueError(f"LatentRows: a row of {self.stride} holds no {self.q_rank} + {self.rank} + {self.rot}")
        if self.turned > self.rot or self.turned % 2:
            raise ValueError(f"LatentRows: {self.turned} of {self.rot} columns turn in pairs")

    def tolerance(self):
        return Tolerance.relative(1e-2, 1e-2, note="float32, rounded once")

    def build(self) -> Built:
        from .. import kernels

        kw = {n: getattr(self, n) for n in ("slots", "rows", "stride", "q_rank", "rank", "rot", "turned", "angle_rows", "ring")}
        kw["eps"] = float(self.epsilon)

        def launch(t, words):
            kernels.latent_rows(t["x"], t["q_gain"], t["c_gain"], t["spans"], t["q"], t["latents"], angles=t.get("angles"),
                                shared_keys=t.get("shared_keys"), **kw)

        return Built("iron_latent_rows", launch)


class LatentMHA(Operator):
    """Attention of ``heads`` queries ``[dim | rot]`` a row over latents: with ``up`` = the heads' key rows (dim each)
    and then their value rows (vdim each), score = ``(q . U c + turned q . shared key) * scale`` over
    ``0 <= i - j < window``, softmax (with ``sink``: a term ``exp(sink[head])`` more in its denominator), and y the
    weighted sum of ``V c``.  The rows' own latents are in the ring already (LatentRows); it holds at least a window
    and a portion.  ``single``: every span is one row at most.  Otherwise the keys of the spans, each with what
    its window reaches before it, are ``cap`` at most."""

    slots: int = param()
    rows: int = param()
    heads: int = param()
    dim: int = param()
    rot: int = param(default=0)
    vdim: int = param()
    rank: int = param()
    q_width: int = param(derive=lambda op: op.heads * (op.dim + op.rot), repr=False)
    up_rows: int = param(derive=lambda op: op.heads * (op.dim + op.vdim), repr=False)
    width: int = param(derive=lambda op: op.heads * op.vdim, repr=False)
    shared: bool = param(derive=lambda op: op.rot > 0, repr=False)
    turned: int = param(default=0)
    turns: bool = param(derive=lambda op: op.turned > 0, repr=False)
    angle_rows: int = param(default=0, array=True)
    sunk: bool = param(default=False, repr=False)
    window: int = param(default=EVERYTHING)
    ring: int = param()
    cap: int = param(default=0)
    scale: float = param(array=True)
    single: bool = param(default=False)
    dtype: Any = param(default=bfloat16, repr=False)
    q = In(rows, q_width, dtype=dtype)
    latents = In(slots, ring, rank, dtype=dtype)
    up = In(up_rows, rank)
    spans = In(slots, 4, dtype=np.int32)
    shared_keys = In(slots, ring, rot, dtype=dtype, when=shared)
    angles = In(angle_rows, turned, dtype=F32, when=turns)
    sink = In(heads, when=sunk)
    y = Out(rows, width, dtype=dtype)
    workspace_words: int = param(derive=lambda op: op._workspace_words(), repr=False)
    workspace = Scratch(workspace_words, dtype=F32)
    valid = per_call(bounds=rows)

    def _workspace_words(self) -> int:
        from .._lib import lib

        return -(-int(lib().iron_mha_latent_workspace_bytes(
            self.slots, self.rows, self.heads, self.dim, self.rot, self.vdim, self.rank, self.window, self.ring, self.cap,
            int(self.single), int(self.dtype is not bfloat16))) // 4)

    @classmethod
    def infer(cls, shapes, **kw):
        slots, ring, rank = shapes["latents"]
        heads = kw["heads"]
        out = dict(slots=slots, ring=ring, rank=rank, rows=shapes["q"][0], sunk="sink" in shapes, **kw)
        if "shared_keys" in shapes:
            out["rot"] = shapes["shared_keys"][2]
        if "angles" in shapes:
            out |= dict(angle_rows=shapes["angles"][0], turned=shapes["angles"][1])
        out["dim"] = shapes["q"][1] // heads - out.get("rot", 0)
        out["vdim"] = shapes["up"][0] // heads - out["dim"]
        return out

    def validate(self):
        if self.dim + self.rot > 4096 or self.rank + self.rot > 2048 or self.vdim > 1024:
            raise ValueError(f"LatentMHA: keys ({self.dim} + {self.rot}) up to 4096, a latent ({self.rank} + {self.rot}) up to 2048, "
                             f"values ({self.vdim}) up to 1024")
        if self.window < 1:
            raise ValueError(f"LatentMHA: a window ({self.window}) of at least 1")
        if not self.single and self.cap < self.rows:
            raise ValueError(f"LatentMHA: room for {self.cap} keys of {self.rows} rows")

    def tolerance(self):
        return Tolerance.relative(4e-2, 4e-2, note="float32 scores and weights")

    def build(self) -> Built:
        from .. import kernels

        kw = {n: getattr(self, n) for n in ("slots", "rows", "heads", "dim", "rot", "vdim", "rank", "turned", "angle_rows", "window", "ring",
                                            "cap", "single")}
        kw["scale"] = float(self.scale)

        def launch(t, words):
            kernels.mha_latent(t["q"], t["latents"], t["up"], t["spans"], t["y"], t["workspace"], angles=t.get("angles"),
                               shared_keys=t.get("shared_keys"), sink=t.get("sink"), **kw)

        return Built("iron_mha_latent", launch)
