"""WindowMHA: sliding-window attention with a learned bias by distance, over a batch of spans and a ring
of keys and values a slot.
"""

from __future__ import annotations

from typing import Any

import numpy as np

from ..bf16 import bfloat16
from ..common.declare import Built, In, InOut, Operator, param, per_call
from ..common.verify import Tolerance


class WindowMHA(Operator):
    """Rows ``x`` are a packed projection ``[q heads | k heads | v heads]``.  Position i sees j with
    ``0 <= i - j < window``; score = ``q . k * scale + bias[head][i - j]``; ordinary softmax.  The heads'
    values, times ``out_scale``, go to columns ``at ..`` of ``y`` (whose other columns are left alone).
    Position p's key and value live in row ``p % ring`` of the slot's ring.  ``single``: every span is one
    row at most (a decode step)."""

    slots: int = param()
    rows: int = param()
    stride: int = param()
    heads: int = param()
    kv_heads: int = param()
    dim: int = param()
    vdim: int = param()
    window: int = param()
    ring: int = param()
    width: int = param()
    at: int = param(default=0, array=True)
    scale: float = param(array=True)
    out_scale: float = param(default=1.0, array=True)
    single: bool = param(default=False)
    dtype: Any = param(default=bfloat16, repr=False)
    x = In(rows, stride, dtype=dtype)
    bias = In(heads, window, dtype=np.float32)
    spans = In(slots, 4, dtype=np.int32)
    keys = InOut(slots, ring, kv_heads, dim, dtype=dtype)
    values = InOut(slots, ring, kv_heads, vdim, dtype=dtype)
    y = InOut(rows, width, dtype=dtype)
    valid = per_call(bounds=rows)

    @classmethod
    def infer(cls, shapes, **kw):
        heads, window = shapes["bias"]
        slots, ring, kv_heads, dim = shapes["keys"]
        return dict(slots=slots, rows=shapes["x"][0], stride=shapes["x"][1], heads=heads, kv_heads=kv_heads, dim=dim,
                    vdim=shapes["values"][3], window=window, ring=ring, width=shapes["y"][1], **kw)

    def validate(self):
        if self.heads % self.kv_heads:
            raise ValueError(f"WindowMHA: kv_heads ({self.kv_heads}) must divide heads ({self.heads})")
        if not (1 <= self.dim <= 256 and 1 <= self.vdim <= 256):
            raise ValueError(f"WindowMHA: dim ({self.dim}) and vdim ({self.vdim}) from 1 to 256")
        if not 1 <= self.window <= self.ring:
            raise ValueError(f"WindowMHA: a window ({self.window}) of at least 1 within the ring ({self.ring})")

    def ops(self) -> int:
        keys = np.minimum(np.arange(self.rows) + 1, self.window).sum()
        return int(2 * self.heads * (self.dim + self.vdim) * keys)

    def tolerance(self):
        return Tolerance.relative(4e-2, 4e-2, note="float32 scores and weights")

    def build(self) -> Built:
        from .. import kernels

        kw = {n: getattr(self, n) for n in ("slots", "rows", "stride", "heads", "kv_heads", "dim", "vdim", "window", "ring",
                                            "single")}
        kw |= dict(scale=float(self.scale), out_stride=self.width, out_at=self.at, out_scale=float(self.out_scale))

        def launch(t, words):
            kernels.mha_window(t["x"], t["keys"], t["values"], t["bias"], t["spans"], t["y"], **kw)

        return Built("iron_mha_window", launch)
