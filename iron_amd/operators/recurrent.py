"""Layers that carry a state from token to token, over a batch of rows.

``spans`` (int32 ``(slots, 4)``) says which rows are which sequence's: ``{row0, rows, start, unused}`` per
slot; an idle slot has no rows.  A state is held a slot; a span that starts at position 0 reads none.
Everything that enters a recurrence is computed in float32; ``dtype`` is the projections' type, bf16 or
float32.
"""

from __future__ import annotations

from typing import Any

import numpy as np

from ..bf16 import bfloat16
from ..common.declare import Built, In, InOut, Operator, Out, Scratch, param, per_call
from ..common.verify import Tolerance

F32 = np.float32


class _Spanned(Operator):
    """An operator over a batch's rows told apart by spans."""

    # A portion of many rows runs its recurrence sixteen tokens at a time, a decode step's few token by token.
    CHUNKED_ROWS = 4   # rows a slot from which the chunks win

    def tolerance(self):
        return Tolerance.relative(1e-2, 1e-2, note="float32 inside, rounded once where it leaves")


class TokenShift(_Spanned):
    """``mixed[m] = h + (before - h) * mu[m]``: each of several projections reads its own blend of a token
    and the one before it (zeros ahead of the first).  ``carry`` keeps position
    p's row in row ``p % 2`` of its slot."""

    slots: int = param()
    rows: int = param()
    cols: int = param()
    mixes: int = param()
    dtype: Any = param(default=bfloat16, repr=False)
    h = In(rows, cols, dtype=dtype)
    mu = In(mixes, cols)
    carry = InOut(slots, 2, cols, dtype=dtype)
    spans = In(slots, 4, dtype=np.int32)
    mixed = Out(mixes, rows, cols, dtype=dtype)

    @classmethod
    def infer(cls, shapes, **kw):
        return dict(slots=shapes["spans"][0], rows=shapes["h"][0], cols=shapes["h"][1], mixes=shapes["mu"][0], **kw)

    def build(self) -> Built:
        from .. import kernels

        kw = dict(slots=self.slots, rows=self.rows, cols=self.cols, mixes=self.mixes)

        def launch(t, words):
            kernels.token_shift(t["h"], t["mu"], t["carry"], t["spans"], t["mixed"], **kw)

        return Built("iron_token_shift", launch)


class LowRankDecay(Operator):
    """``-exp(up tanh(z) + base)``: the logarithm of a decay per channel, from a narrow projection ``z``."""

    rows: int = param()
    n: int = param()
    rank: int = param()
    dtype: Any = param(default=bfloat16, repr=False)
    z = In(rows, rank, dtype=dtype)
    up = In(n, rank)
    base = In(n)
    y = Out(rows, n, dtype=F32)
    valid = per_call(bounds=rows)

    @classmethod
    def infer(cls, shapes, **kw):
        return dict(rows=shapes["z"][0], n=shapes["up"][0], rank=shapes["up"][1], **kw)

    def validate(self):
        if not 1 <= self.rank <= 512:
            raise ValueError(f"LowRankDecay: rank ({self.rank}) from 1 to 512")

    def tolerance(self):
        return Tolerance.relative(1e-4, 1e-5, note="float32")

    def build(self) -> Built:
        from .. import kernels

        rows, n, rank = self.rows, self.n, self.rank

        def launch(t, words):
            kernels.low_rank_decay(t["z"], t["up"], t["base"], t["y"], rows=rows, n=n, rank=rank, valid=words.get("valid"))

        return Built("iron_low_rank_decay", launch)


class TimeMix(_Spanned):
    """Per head ``o = (S + diag(u) k v^T)^T r``, then ``S <- diag(exp(log_decay)) S + k v^T``."""

    slots: int = param()
    rows: int = param()
    heads: int = param()
    dim: int = param()
    width: int = param(derive=lambda op: op.heads * op.dim, repr=False)
    dtype: Any = param(default=bfloat16, repr=False)
    r = In(rows, width, dtype=dtype)
    k = In(rows, width, dtype=dtype)
    v = In(rows, width, dtype=dtype)
    log_decay = In(rows, width, dtype=F32)
    u = In(heads, dim)
    state = InOut(slots, heads, dim, dim, dtype=F32)
    spans = In(slots, 4, dtype=np.int32)
    o = Out(rows, width, dtype=F32)
    chunked: bool = param(default=lambda op: op.rows > op.CHUNKED_ROWS * op.slots, array=True, repr=False)
    workspace_words: int = param(derive=lambda op: op._workspace_words(), repr=False)
    workspace = Scratch(workspace_words, dtype=np.float32, when=chunked)
    valid = per_call(bounds=rows)

    def _workspace_words(self) -> int:
        from .._lib import lib

        return int(lib().iron_time_mix_workspace_bytes(self.slots, self.rows, self.heads, self.dim)) // 4

    @classmethod
    def infer(cls, shapes, **kw):
        return dict(slots=shapes["spans"][0], rows=shapes["r"][0], heads=shapes["u"][0], dim=shapes["u"][1], **kw)

    def validate(self):
        if not 1 <= self.dim <= 256:
            raise ValueError(f"TimeMix: dim ({self.dim}) from 1 to 256")

    def build(self) -> Built:
        from .. import kernels

        kw = dict(slots=self.slots, rows=self.rows, heads=self.heads, dim=self.dim)

        def launch(t, words):
            kernels.time_mix(t["r"], t["k"], t["v"], t["log_decay"], t["u"], t["state"], t["spans"], t["o"],
                             workspace=t.get("workspace"), **kw)

        return Built("iron_time_mix", launch)


class MinGRU(_Spanned):
    """Per channel ``S <- (1 - z) S + z c; y = S silu(g)`` with ``z = sigmoid(zx + z_bias)`` and the candidate c,
    of ``u = ux + x_bias``, ``u + 1/2`` from 0 up and ``sigmoid(u)`` below; rows ``[zx | ux | g | ..]``.  The
    state behind position p is row ``p % 2`` of its slot."""

    slots: int = param()
    rows: int = param()
    stride: int = param()
    width: int = param()
    dtype: Any = param(default=bfloat16, repr=False)
    x = In(rows, stride, dtype=dtype)
    z_bias = In(width)
    x_bias = In(width)
    state = InOut(slots, 2, width, dtype=F32)
    spans = In(slots, 4, dtype=np.int32)
    y = Out(rows, width, dtype=dtype)
    chunked: bool = param(default=lambda op: op.rows > op.CHUNKED_ROWS * op.slots, array=True, repr=False)
    workspace_words: int = param(derive=lambda op: op._workspace_words(), repr=False)
    workspace = Scratch(workspace_words, dtype=np.float32, when=chunked)
    valid = per_call(bounds=rows)

    def _workspace_words(self) -> int:
        from .._lib import lib

        return int(lib().iron_min_gru_workspace_bytes(self.slots, self.rows, self.width)) // 4

    @classmethod
    def infer(cls, shapes, **kw):
        return dict(slots=shapes["spans"][0], rows=shapes["x"][0], stride=shapes["x"][1], width=shapes["z_bias"][0], **kw)

    def validate(self):
        if 3 * self.width > self.stride:
            raise ValueError(f"MinGRU: a row of {self.stride} holds no three projections of {self.width}")

    def build(self) -> Built:
        from .. import kernels

        kw = dict(slots=self.slots, rows=self.rows, stride=self.stride, width=self.width)

        def launch(t, words):
            kernels.min_gru(t["x"], t["z_bias"], t["x_bias"], t["state"], t["spans"], t["y"], workspace=t.get("workspace"), **kw)

        return Built("iron_min_gru", launch)


class _DeltaShape(_Spanned):
    """Sizes of a gated delta rule: ``kv_heads`` q/k heads of ``dim``, ``heads`` value heads of ``vdim``;
    the rows between its two steps are ``[unit q | unit k | v | log decay | beta]`` in float32."""

    slots: int = param()
    rows: int = param()
    heads: int = param()
    kv_heads: int = param()
    dim: int = param()
    vdim: int = param()
    channels: int = param(derive=lambda op: 2 * op.kv_heads * op.dim + op.heads * op.vdim, repr=False)
    wide: int = param(derive=lambda op: op.channels + 2 * op.heads, repr=False)

    def validate(self):
        if self.heads % self.kv_heads:
            raise ValueError(f"{type(self).__name__}: kv_heads ({self.kv_heads}) must divide heads ({self.heads})")
        if not (1 <= self.dim <= 256 and 1 <= self.vdim <= 256):
            raise ValueError(f"{type(self).__name__}: dim ({self.dim}) and vdim ({self.vdim}) from 1 to 256")


class ShortConv(_DeltaShape):
    """From a packed projection ``[q | k | v | .. b .. | .. a ..]``: a short causal convolution per channel
    and SiLU on q, k and v, unit q (times ``dim ** -0.5``) and k per head, and the step's log decay and
    write strength.  ``state`` keeps position p's inputs in row ``p % taps`` of its slot."""

    stride: int = param()
    taps: int = param()
    b_at: int = param(array=True)
    a_at: int = param(array=True)
    dtype: Any = param(default=bfloat16, repr=False)
    x = In(_DeltaShape.rows, stride, dtype=dtype)
    weight = In(_DeltaShape.channels, taps)
    a_log = In(_DeltaShape.heads)
    dt_bias = In(_DeltaShape.heads)
    state = InOut(_DeltaShape.slots, taps, _DeltaShape.channels, dtype=dtype)
    spans = In(_DeltaShape.slots, 4, dtype=np.int32)
    y = Out(_DeltaShape.rows, _DeltaShape.wide, dtype=F32)
    valid = per_call(bounds=_DeltaShape.rows)

    @classmethod
    def infer(cls, shapes, **kw):
        return dict(slots=shapes["spans"][0], rows=shapes["x"][0], stride=shapes["x"][1], taps=shapes["weight"][1],
                    heads=shapes["a_log"][0], **kw)

    def validate(self):
        super().validate()
        if not 1 <= self.taps <= 17:
            raise ValueError(f"ShortConv: taps ({self.taps}) from 1 to 17")

    def build(self) -> Built:
        from .. import kernels

        kw = {n: getattr(self, n) for n in ("slots", "rows", "stride", "heads", "kv_heads", "dim", "vdim", "taps", "b_at", "a_at")}

        def launch(t, words):
            kernels.short_conv(t["x"], t["weight"], t["a_log"], t["dt_bias"], t["state"], t["spans"], t["y"], **kw)

        return Built("iron_short_conv", launch)


class DeltaRule(_DeltaShape):
    """Per value head ``S <- g S; u = beta (v - S^T k); S <- S + k u^T; o = S^T q``."""

    width: int = param(derive=lambda op: op.heads * op.vdim, repr=False)
    x = In(_DeltaShape.rows, _DeltaShape.wide, dtype=F32)
    state = InOut(_DeltaShape.slots, _DeltaShape.heads, _DeltaShape.dim, _DeltaShape.vdim, dtype=F32)
    spans = In(_DeltaShape.slots, 4, dtype=np.int32)
    o = Out(_DeltaShape.rows, width, dtype=F32)
    chunked: bool = param(default=lambda op: op.rows > op.CHUNKED_ROWS * op.slots, array=True, repr=False)
    workspace_words: int = param(derive=lambda op: op._workspace_words(), repr=False)
    workspace = Scratch(workspace_words, dtype=np.float32, when=chunked)
    valid = per_call(bounds=_DeltaShape.rows)

    def _workspace_words(self) -> int:
        from .._lib import lib

        return int(lib().iron_delta_rule_workspace_bytes(self.slots, self.rows, self.heads)) // 4

    @classmethod
    def infer(cls, shapes, **kw):
        _, heads, dim, vdim = shapes["state"]
        return dict(slots=shapes["spans"][0], rows=shapes["x"][0], heads=heads, dim=dim, vdim=vdim, **kw)

    def build(self) -> Built:
        from .. import kernels

        kw = {n: getattr(self, n) for n in ("slots", "rows", "heads", "kv_heads", "dim", "vdim")}

        def launch(t, words):
            kernels.delta_rule(t["x"], t["state"], t["spans"], t["o"], workspace=t.get("workspace"), **kw)

        return Built("iron_delta_rule", launch)


class HeadGate(Operator):
    """``o / rms(o) * gain * silu(gate) * scale`` a head, into columns ``at ..`` of a row of ``width``.  The
    gate is columns ``gate_at ..`` of its row (not ``gated``: there is no such factor); ``gain`` is one head's (shared by
    all) or every column's."""

    rows: int = param()
    heads: int = param()
    dim: int = param()
    o_width: int = param(derive=lambda op: op.heads * op.dim, repr=False)
    gated: bool = param(default=True, repr=False)
    gate_width: int = param(default=0)
    gate_at: int = param(default=0, array=True)
    gains: int = param()
    width: int = param()
    at: int = param(default=0, array=True)
    epsilon: float = param(array=True)
    scale: float = param(default=1.0, array=True)
    dtype: Any = param(default=bfloat16, repr=False)
    o = In(rows, o_width, dtype=F32)
    gate = In(rows, gate_width, dtype=dtype, when=gated)
    gain = In(gains)
    y = Out(rows, width, dtype=dtype)
    valid = per_call(bounds=rows)

    @classmethod
    def infer(cls, shapes, **kw):
        dim = shapes["o"][1] // kw["heads"]
        gate = {"gate_width": shapes["gate"][1]} if "gate" in shapes else {"gated": False}
        return {"rows": shapes["o"][0], "dim": dim, "gains": shapes["gain"][0], "width": shapes["o"][1], **gate, **kw}

    def validate(self):
        if self.gains not in (self.dim, self.o_width):
            raise ValueError(f"HeadGate: {self.gains} gains for heads of {self.dim}")

    def tolerance(self):
        return Tolerance.relative(1e-2, 1e-2, note="float32, rounded once")

    def build(self) -> Built:
        from .. import kernels

        kw = dict(rows=self.rows, heads=self.heads, dim=self.dim, gate_stride=self.gate_width, gate_at=self.gate_at,
                  gain_shared=self.gains != self.o_width, out_stride=self.width, out_at=self.at,
                  eps=float(self.epsilon), scale=float(self.scale))

        def launch(t, words):
            kernels.head_gate(t["o"], t.get("gate"), t["gain"], t["y"], valid=words.get("valid"), **kw)

        return Built("iron_head_gate", launch)


class Hgrn2(_Spanned):
    """HGRN2: per head ``S <- diag(f) S + (1 - f) v^T``, then ``o = S^T silu(q)``, with the forget gate ``f = lower + (1 - lower)
    sigmoid(z + f_bias)`` a channel.  Rows ``[q | z | v | ..]``."""

    slots: int = param()
    rows: int = param()
    stride: int = param()
    heads: int = param()
    dim: int = param()
    vdim: int = param()
    channels: int = param(derive=lambda op: op.heads * op.dim, repr=False)
    width: int = param(derive=lambda op: op.heads * op.vdim, repr=False)
    dtype: Any = param(default=bfloat16, repr=False)
    x = In(rows, stride, dtype=dtype)
    f_bias = In(channels)
    lower = In(channels)
    state = InOut(slots, heads, dim, vdim, dtype=F32)
    spans = In(slots, 4, dtype=np.int32)
    o = Out(rows, width, dtype=F32)
    chunked: bool = param(default=lambda op: op.rows > op.CHUNKED_ROWS * op.slots, array=True, repr=False)
    workspace_words: int = param(derive=lambda op: op._workspace_words(), repr=False)
    workspace = Scratch(workspace_words, dtype=F32, when=chunked)
    valid = per_call(bounds=rows)

    def _workspace_words(self) -> int:
        from .._lib import lib

        return int(lib().iron_hgrn2_workspace_bytes(self.slots, self.rows, self.heads, self.dim)) // 4

    @classmethod
    def infer(cls, shapes, **kw):
        slots, heads, dim, vdim = shapes["state"]
        return dict(slots=slots, rows=shapes["x"][0], stride=shapes["x"][1], heads=heads, dim=dim, vdim=vdim, **kw)

    def validate(self):
        if not (1 <= self.dim <= 256 and self.heads * (2 * self.dim + self.vdim) <= self.stride):
            raise ValueError(f"Hgrn2: dim ({self.dim}) from 1 to 256; {self.heads} heads of {self.dim} and {self.vdim} in a row of {self.stride}")

    def build(self) -> Built:
        from .. import kernels

        kw = {n: getattr(self, n) for n in ("slots", "rows", "stride", "heads", "dim", "vdim")}

        def launch(t, words):
            kernels.hgrn2(t["x"], t["f_bias"], t["lower"], t["state"], t["spans"], t["o"], workspace=t.get("workspace"), **kw)

        return Built("iron_hgrn2", launch)


class MatrixMemory(_Spanned):
    """mLSTM: per head ``S <- keep S + write k v^T``, ``n <- keep n + write k`` with log gates i (capped) and f (the logarithm of a
    capped one's sigmoid), ``m' = max(f + m, i)``, ``keep = exp(f + m - m')``, ``write = exp(i - m')``.  Rows ``[q | k | v | ..]``,
    the gates at columns ``i_at`` and ``f_at``.  ``state`` is S with n behind its last column; ``tops`` holds m, position p's in row
    ``p % 2`` of its slot.  Output rows ``[S^T q | n . q | m]``, q times ``dim ** -0.5``."""

    slots: int = param()
    rows: int = param()
    stride: int = param()
    heads: int = param()
    dim: int = param()
    vdim: int = param()
    i_at: int = param(array=True)
    f_at: int = param(array=True)
    cap: float = param(array=True)
    columns: int = param(derive=lambda op: op.vdim + 1, repr=False)
    width: int = param(derive=lambda op: op.heads * (op.vdim + 2), repr=False)
    dtype: Any = param(default=bfloat16, repr=False)
    x = In(rows, stride, dtype=dtype)
    i_bias = In(heads)
    f_bias = In(heads)
    state = InOut(slots, heads, dim, columns, dtype=F32)
    tops = InOut(slots, 2, heads, dtype=F32)
    spans = In(slots, 4, dtype=np.int32)
    o = Out(rows, width, dtype=F32)
    chunked: bool = param(default=lambda op: op.rows > op.CHUNKED_ROWS * op.slots and op.dim <= 256, array=True, repr=False)
    workspace_words: int = param(derive=lambda op: op._workspace_words(), repr=False)
    workspace = Scratch(workspace_words, dtype=F32, when=chunked)
    valid = per_call(bounds=rows)

    def _workspace_words(self) -> int:
        from .._lib import lib

        return int(lib().iron_matrix_memory_workspace_bytes(self.slots, self.rows, self.heads, self.dim)) // 4

    @classmethod
    def infer(cls, shapes, **kw):
        slots, heads, dim, columns = shapes["state"]
        return dict(slots=slots, rows=shapes["x"][0], stride=shapes["x"][1], heads=heads, dim=dim, vdim=columns - 1, **kw)

    def validate(self):
        packed = self.heads * (2 * self.dim + self.vdim)
        if not (1 <= self.dim <= 512 and packed <= min(self.i_at, self.f_at) and max(self.i_at, self.f_at) + self.heads <= self.stride):
            raise ValueError(f"MatrixMemory: dim ({self.dim}) from 1 to 512; gates at {self.i_at}, {self.f_at} behind {packed} of {self.stride}")

    def build(self) -> Built:
        from .. import kernels

        kw = {n: getattr(self, n) for n in ("slots", "rows", "stride", "heads", "dim", "vdim", "i_at", "f_at")}
        kw["cap"] = float(self.cap)

        def launch(t, words):
            kernels.matrix_memory(t["x"], t["i_bias"], t["f_bias"], t["state"], t["tops"], t["spans"], t["o"],
                                  workspace=t.get("workspace"), **kw)

        return Built("iron_matrix_memory", launch)


class MemoryGate(Operator):
    """``o / (max(|n . q|, exp(-m)) + floor)`` of MatrixMemory's rows, RMS-normed a head, times ``gain`` and ``sigmoid(gate)``;
    the gate is columns ``gate_at ..`` of its row."""

    rows: int = param()
    heads: int = param()
    dim: int = param()
    inner: int = param(derive=lambda op: op.heads * op.dim, repr=False)
    wide: int = param(derive=lambda op: op.heads * (op.dim + 2), repr=False)
    gate_width: int = param()
    gate_at: int = param(default=0, array=True)
    floor: float = param(default=1e-6, array=True)
    epsilon: float = param(array=True)
    dtype: Any = param(default=bfloat16, repr=False)
    o = In(rows, wide, dtype=F32)
    gate = In(rows, gate_width, dtype=dtype)
    gain = In(inner)
    y = Out(rows, inner, dtype=dtype)
    valid = per_call(bounds=rows)

    @classmethod
    def infer(cls, shapes, **kw):
        return dict(rows=shapes["o"][0], dim=shapes["gain"][0] // kw["heads"], gate_width=shapes["gate"][1], **kw)

    def validate(self):
        if not 0 <= self.gate_at <= self.gate_width - self.inner:
            raise ValueError(f"MemoryGate: {self.inner} columns from {self.gate_at} of a row of {self.gate_width}")

    def tolerance(self):
        return Tolerance.relative(1e-2, 1e-2, note="float32, rounded once")

    def build(self) -> Built:
        from .. import kernels

        kw = dict(rows=self.rows, heads=self.heads, dim=self.dim, gate_stride=self.gate_width, gate_at=self.gate_at, floor=float(self.floor),
                  eps=float(self.epsilon))

        def launch(t, words):
            kernels.memory_gate(t["o"], t["gate"], t["gain"], t["y"], valid=words.get("valid"), **kw)

        return Built("iron_memory_gate", launch)
