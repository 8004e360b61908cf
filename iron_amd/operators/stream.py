"""The float32 residual stream of a decoder: rows into it, rows or their norms out of it, blocks' outputs added to it,
averages over what it was behind earlier layers, a feed-forward's gated columns, and the head's scale and soft cap.  ``dtype`` is what the rows that leave the stream are rounded to: bf16, or
float32 in a model that runs in 32 bits throughout.  The stream is updated in place.
"""

from __future__ import annotations

import math
from typing import Any

import numpy as np

from ..bf16 import bfloat16
from ..common.declare import Built, In, InOut, Operator, Out, param, per_call
from ..common.verify import Tolerance

F32 = np.float32


class StreamEmbed(Operator):
    """``x[i] = scale * table[ids[i]]`` in float32: a decoder's embedding rows as its stream's first values.  ``twice``: into a
    second place as well."""

    rows: int = param()
    table_rows: int = param(array=True)
    cols: int = param()
    scale: float = param(default=1.0, array=True)
    twice: bool = param(default=False, repr=False)
    table = In(table_rows, cols)
    ids = In(rows, dtype=np.int32)
    x = Out(rows, cols, dtype=F32)
    also = Out(rows, cols, dtype=F32, when=twice)
    valid = per_call(bounds=rows)

    @classmethod
    def infer(cls, shapes, **kw):
        return dict(rows=math.prod(shapes["ids"]), table_rows=shapes["table"][0], cols=shapes["table"][1], **kw)

    def tolerance(self):
        return Tolerance.exact()

    def build(self) -> Built:
        from .. import kernels

        rows, table_rows, cols, scale = self.rows, self.table_rows, self.cols, float(self.scale)

        def launch(t, words):
            kernels.stream_embed(t["table"], t["ids"].reshape(-1), t["x"], rows=rows, table_rows=table_rows, cols=cols, scale=scale,
                                 also=t.get("also"), valid=words.get("valid"))

        return Built("iron_stream_embed", launch)


class StreamNorm(Operator):
    """``y = dtype(x / rms(x) * (unit + weight))`` of a float32 row: one rounding, where it leaves the stream.  ``groups``: each
    of a row's that many equal parts over its own root mean square."""

    rows: int = param()
    cols: int = param()
    groups: int = param(default=1)
    epsilon: float = param(array=True)
    unit: float = param(default=0.0, array=True)
    dtype: Any = param(default=bfloat16, repr=False)
    x = In(rows, cols, dtype=F32)
    weight = In(cols)
    y = Out(rows, cols, dtype=dtype)
    valid = per_call(bounds=rows)

    @classmethod
    def infer(cls, shapes, **kw):
        return dict(rows=shapes["x"][0], cols=shapes["x"][1], **kw)

    def validate(self):
        if self.groups < 1 or self.cols % self.groups:
            raise ValueError(f"StreamNorm: {self.cols} columns in {self.groups} equal groups")

    def tolerance(self):
        return Tolerance.relative(1e-2, 1e-2, note="float32, rounded once")

    def build(self) -> Built:
        from .. import kernels

        kw = dict(rows=self.rows, cols=self.cols, eps=float(self.epsilon), unit=float(self.unit))
        grouped = self.groups > 1

        def launch(t, words):
            given = dict(h=t["y"], gain=t["weight"], valid=words.get("valid"), **kw)
            if grouped:
                kernels.stream_groups(t["x"], groups=self.groups, **given)
            else:
                kernels.stream_rows(t["x"], **given)

        return Built("iron_stream_groups" if grouped else "iron_stream_rows", launch)


class StreamSum(Operator):
    """``x += y + also`` in float32: what blocks side by side made of one row joins the stream (``also`` may be missing)."""

    rows: int = param()
    cols: int = param()
    two: bool = param(default=False, repr=False)
    dtype: Any = param(default=bfloat16, repr=False)
    x = InOut(rows, cols, dtype=F32)
    y = In(rows, cols, dtype=dtype)
    also = In(rows, cols, dtype=dtype, when=two)
    valid = per_call(bounds=rows)

    @classmethod
    def infer(cls, shapes, **kw):
        return dict(rows=shapes["x"][0], cols=shapes["x"][1], two="also" in shapes, **kw)

    def tolerance(self):
        return Tolerance.relative(1e-5, 1e-5, note="float32")

    def build(self) -> Built:
        from .. import kernels

        kw = dict(rows=self.rows, cols=self.cols)

        def launch(t, words):
            kernels.stream_groups(t["x"], y=t["y"], y2=t.get("also"), valid=words.get("valid"), **kw)

        return Built("iron_stream_groups", launch)


class GatedColumns(Operator):
    """``act(gate) * up`` of columns ``gate_at ..`` and ``gate_at + cols ..`` of a projection's row, into columns ``at ..`` of
    ``y`` (whose other columns are left alone).  ``kind`` ``limited``: ``g sigmoid(1.702 g) (u + 1)``, g the gate held to at most
    ``limit``, u within it on both sides; else an activation's name."""

    rows: int = param()
    cols: int = param()
    stride: int = param()
    width: int = param()
    gate_at: int = param(default=0, array=True)
    at: int = param(default=0, array=True)
    kind: str = param()
    limit: float = param(default=0.0, array=True)
    dtype: Any = param(default=bfloat16, repr=False)
    x = In(rows, stride, dtype=dtype)
    y = InOut(rows, width, dtype=dtype)
    valid = per_call(bounds=rows)

    @classmethod
    def infer(cls, shapes, **kw):
        return dict(rows=shapes["x"][0], stride=shapes["x"][1], width=shapes["y"][1], **kw)

    def validate(self):
        if not (0 <= self.gate_at <= self.stride - 2 * self.cols and 0 <= self.at <= self.width - self.cols):
            raise ValueError(f"GatedColumns: twice {self.cols} columns from {self.gate_at} of {self.stride}, into those from {self.at} of {self.width}")
        if self.kind == "limited" and not self.limit > 0:
            raise ValueError(f"GatedColumns: a limit ({self.limit}) above 0")

    def tolerance(self):
        return Tolerance.relative(1e-2, 1e-2, note="float32, rounded once")

    def build(self) -> Built:
        from .. import kernels

        kw = {n: getattr(self, n) for n in ("rows", "cols", "stride", "gate_at", "width", "at", "kind")}
        kw["limit"] = float(self.limit)

        def launch(t, words):
            kernels.gated_columns(t["x"], t["y"], valid=words.get("valid"), **kw)

        return Built("iron_gated_columns", launch)


class StreamAdd(Operator):
    """``x += z / rms(z) * (unit + weight)`` in float32, ``z = y (+ y_bias)``: a block's output, normed, joins the stream."""

    rows: int = param()
    cols: int = param()
    epsilon: float = param(array=True)
    unit: float = param(default=0.0, array=True)
    biased: bool = param(default=False, repr=False)
    dtype: Any = param(default=bfloat16, repr=False)
    x = InOut(rows, cols, dtype=F32)
    y = In(rows, cols, dtype=dtype)
    weight = In(cols)
    y_bias = In(cols, when=biased)
    valid = per_call(bounds=rows)

    @classmethod
    def infer(cls, shapes, **kw):
        return dict(rows=shapes["x"][0], cols=shapes["x"][1], biased="y_bias" in shapes, **kw)

    def tolerance(self):
        return Tolerance.relative(1e-4, 1e-4, note="float32")

    def build(self) -> Built:
        from .. import kernels

        kw = dict(rows=self.rows, cols=self.cols, eps=float(self.epsilon), unit=float(self.unit))

        def launch(t, words):
            kernels.stream_rows(t["x"], y=t["y"], y_bias=t.get("y_bias"), back_gain=t["weight"], valid=words.get("valid"), **kw)

        return Built("iron_stream_rows", launch)


class DepthAverage(Operator):
    """``planes[index] = x``, then ``x = sum over j <= index of weights[j] * planes[j]``: a layer's result is kept, and a weighted
    sum of all there are so far takes its place.  ``planes`` may have more rows than ``x``."""

    rows: int = param()
    cols: int = param()
    depth: int = param()
    plane_rows: int = param()
    count: int = param()
    x = InOut(rows, cols, dtype=F32)
    planes = InOut(depth, plane_rows, cols, dtype=F32)
    weights = In(count)
    valid = per_call(bounds=rows)

    @classmethod
    def infer(cls, shapes, **kw):
        depth, plane_rows, cols = shapes["planes"]
        return dict(rows=shapes["x"][0], cols=cols, depth=depth, plane_rows=plane_rows, count=shapes["weights"][0], **kw)

    def validate(self):
        if not 1 <= self.count <= self.depth or self.rows > self.plane_rows:
            raise ValueError(f"DepthAverage: {self.count} weights, {self.rows} rows for {self.depth} planes of {self.plane_rows}")

    def tolerance(self):
        return Tolerance.relative(1e-4, 1e-4, note="float32")

    def build(self) -> Built:
        from .. import kernels

        kw = dict(rows=self.rows, cols=self.cols, plane_rows=self.plane_rows, index=self.count - 1)

        def launch(t, words):
            kernels.stream_depth_rows(t["x"], planes=t["planes"], weights=t["weights"], valid=words.get("valid"), **kw)

        return Built("iron_stream_depth_rows", launch)


class StreamCast(Operator):
    """``y = dtype(x)``: the stream's row as a block without a norm ahead of it reads it."""

    rows: int = param()
    cols: int = param()
    dtype: Any = param(default=bfloat16, repr=False)
    x = In(rows, cols, dtype=F32)
    y = Out(rows, cols, dtype=dtype)
    valid = per_call(bounds=rows)

    @classmethod
    def infer(cls, shapes, **kw):
        return dict(rows=shapes["x"][0], cols=shapes["x"][1], **kw)

    def tolerance(self):
        return Tolerance.relative(1e-2, 1e-2, note="rounded once")

    def build(self) -> Built:
        from .. import kernels

        rows, cols = self.rows, self.cols

        def launch(t, words):
            kernels.stream_depth_rows(t["x"], h=t["y"], rows=rows, cols=cols, valid=words.get("valid"))

        return Built("iron_stream_depth_rows", launch)


class StreamGatedAdd(Operator):
    """``x += (y + y_bias) * sigmoid(gate + gate_bias)`` in float32: a block's output joins the stream through
    a gate, columns ``gate_at ..`` of a projection's row."""

    rows: int = param()
    cols: int = param()
    gate_width: int = param()
    gate_at: int = param(default=0, array=True)
    biased: bool = param(default=False, repr=False)
    dtype: Any = param(default=bfloat16, repr=False)
    x = InOut(rows, cols, dtype=F32)
    y = In(rows, cols, dtype=dtype)
    gate = In(rows, gate_width, dtype=dtype)
    gate_bias = In(cols)
    y_bias = In(cols, when=biased)
    valid = per_call(bounds=rows)

    @classmethod
    def infer(cls, shapes, **kw):
        return dict(rows=shapes["x"][0], cols=shapes["x"][1], gate_width=shapes["gate"][1], biased="y_bias" in shapes, **kw)

    def validate(self):
        if not 0 <= self.gate_at <= self.gate_width - self.cols:
            raise ValueError(f"StreamGatedAdd: columns {self.gate_at} .. + {self.cols} of a row of {self.gate_width}")

    def tolerance(self):
        return Tolerance.relative(1e-4, 1e-4, note="float32")

    def build(self) -> Built:
        from .. import kernels

        kw = dict(rows=self.rows, cols=self.cols, gate_stride=self.gate_width, gate_at=self.gate_at)

        def launch(t, words):
            kernels.stream_gated_rows(t["x"], t["y"], t["gate"], t["gate_bias"], y_bias=t.get("y_bias"), valid=words.get("valid"), **kw)

        return Built("iron_stream_gated_rows", launch)


class PolyNorm(Operator):
    """``a N(z) + b N(z^2) + c N(z^3) + e``: an activation over the normed powers of a row, ``z`` columns
    ``at ..`` of a projection's row plus a bias, N a row over its root mean square; ``coefficients`` a, b, c, e."""

    rows: int = param()
    cols: int = param()
    stride: int = param()
    at: int = param(default=0, array=True)
    epsilon: float = param(array=True)
    biased: bool = param(default=False, repr=False)
    dtype: Any = param(default=bfloat16, repr=False)
    x = In(rows, stride, dtype=dtype)
    coefficients = In(4)
    bias = In(cols, when=biased)
    y = Out(rows, cols, dtype=dtype)
    valid = per_call(bounds=rows)

    @classmethod
    def infer(cls, shapes, **kw):
        given = {"cols": shapes["x"][1]} | ({"cols": shapes["bias"][0]} if "bias" in shapes else {})
        return {"rows": shapes["x"][0], "stride": shapes["x"][1], "biased": "bias" in shapes, **given, **kw}

    def validate(self):
        if not 0 <= self.at <= self.stride - self.cols:
            raise ValueError(f"PolyNorm: columns {self.at} .. + {self.cols} of a row of {self.stride}")

    def tolerance(self):
        return Tolerance.relative(1e-2, 1e-2, note="float32, rounded once")

    def build(self) -> Built:
        from .. import kernels

        kw = dict(rows=self.rows, cols=self.cols, stride=self.stride, at=self.at, eps=float(self.epsilon))

        def launch(t, words):
            kernels.poly_norm(t["x"], t["coefficients"], t["y"], bias=t.get("bias"), valid=words.get("valid"), **kw)

        return Built("iron_poly_norm", launch)


class SpanTails(Operator):
    """The stream's row of every slot's last token: what a prompt's portion hands its head."""

    slots: int = param()
    rows: int = param()
    cols: int = param()
    x = In(rows, cols, dtype=F32)
    spans = In(slots, 4, dtype=np.int32)
    y = Out(slots, cols, dtype=F32)

    @classmethod
    def infer(cls, shapes, **kw):
        return dict(slots=shapes["spans"][0], rows=shapes["x"][0], cols=shapes["x"][1])

    def output_valid(self, name, inputs):
        return {}

    def tolerance(self):
        return Tolerance.exact()

    def build(self) -> Built:
        from .. import kernels

        slots, rows, cols = self.slots, self.rows, self.cols

        def launch(t, words):
            kernels.span_tails(t["x"], t["spans"], t["y"], slots=slots, rows=rows, cols=cols)

        return Built("iron_span_tails", launch)


class Softcap(Operator):
    """``cap * tanh(scale * x / cap)`` of the head's rows (``cap`` 0: ``scale * x``), as float32 and, in rows
    padded to whole 16-byte pieces, as the bf16 the draw ranks."""

    rows: int = param()
    cols: int = param()
    cap: float = param(default=0.0, array=True)
    scale: float = param(default=1.0, array=True)
    dtype: Any = param(default=bfloat16, repr=False)
    stride: int = param(derive=lambda op: -(-op.cols // 8) * 8, repr=False)
    x = In(rows, cols, dtype=dtype)
    y = Out(rows, cols, dtype=F32)
    rounded = Out(rows, stride)

    @classmethod
    def infer(cls, shapes, **kw):
        return dict(rows=shapes["x"][0], cols=shapes["x"][1], **kw)

    def tolerance(self):
        return Tolerance.relative(1e-2, 1e-2, note="float32, the draw's copy rounded")

    def build(self) -> Built:
        from .. import kernels

        rows, cols, stride, cap, scale = self.rows, self.cols, self.stride, float(self.cap), float(self.scale)

        def launch(t, words):
            kernels.softcap(t["x"], t["y"], t["rounded"], rows=rows, cols=cols, stride=stride, cap=cap, scale=scale)

        return Built("iron_softcap", launch)


class GatedProduct(Operator):
    """``act(gate) * up`` in float32, the 32-bit model's step where a bf16 one records the two."""

    rows: int = param()
    cols: int = param()
    activation: str = param()
    gate = In(rows, cols, dtype=F32)
    up = In(rows, cols, dtype=F32)
    y = Out(rows, cols, dtype=F32)
    valid = per_call(bounds=rows)

    @classmethod
    def infer(cls, shapes, **kw):
        return dict(rows=shapes["gate"][0], cols=shapes["gate"][1], **kw)

    def tolerance(self):
        return Tolerance.relative(1e-5, 1e-6, note="float32")

    def build(self) -> Built:
        from .. import kernels

        rows, cols, kind = self.rows, self.cols, self.activation

        def launch(t, words):
            kernels.act_mul_f32(t["gate"], t["up"], t["y"], rows=rows, cols=cols, activation=kind, valid=words.get("valid"))

        return Built("iron_act_mul_f32", launch)


class Activation(Operator):
    """``act(x)`` of rows of either type, rounded once."""

    rows: int = param()
    cols: int = param()
    kind: str = param()
    dtype: Any = param(default=bfloat16, repr=False)
    x = In(rows, cols, dtype=dtype)
    y = Out(rows, cols, dtype=dtype)
    valid = per_call(bounds=rows)

    @classmethod
    def infer(cls, shapes, **kw):
        return dict(rows=shapes["x"][0], cols=shapes["x"][1], **kw)

    def tolerance(self):
        return Tolerance.relative(1e-2, 1e-2, note="float32, rounded once")

    def build(self) -> Built:
        from .. import kernels

        rows, cols, kind = self.rows, self.cols, self.kind

        def launch(t, words):
            kernels.activation(t["x"], t["y"], rows=rows, cols=cols, kind=kind, valid=words.get("valid"))

        return Built("iron_activation", launch)


class LinearAny(Operator):
    """``x @ weight.T`` on float32 products and sums, rows of either type and any length: the 32-bit
    model's projections (bf16 weights are float32 values), and a bf16 row of no whole 16-byte pieces."""

    rows: int = param()
    n: int = param()
    k: int = param()
    dtype: Any = param(default=bfloat16, repr=False)
    x = In(rows, k, dtype=dtype)
    weight = In(n, k)
    y = Out(rows, n, dtype=dtype)
    valid = per_call(bounds=rows)

    @classmethod
    def infer(cls, shapes, **kw):
        if shapes["x"][1] != shapes["weight"][1]:
            raise ValueError(f"x {shapes['x']} and the weight {shapes['weight']} disagree on their length")
        return dict(rows=shapes["x"][0], n=shapes["weight"][0], k=shapes["x"][1], **kw)

    def ops(self) -> int:
        return 2 * self.rows * self.n * self.k

    def tolerance(self):
        return Tolerance.relative(1e-2, 1e-2, note="float32 sums, rounded once if bf16")

    def build(self) -> Built:
        from .. import kernels

        rows, n, k = self.rows, self.n, self.k

        def launch(t, words):
            kernels.linear_any(t["x"], t["weight"], t["y"], rows=rows, n=n, k=k, valid=words.get("valid"))

        return Built("iron_linear_any", launch)
