"""Token mixers over a batch of rows told apart by spans, and the layer that runs them around a float32
residual stream: sliding-window attention with a learned distance bias, time mixing with a
data-dependent decay, both side by side, the gated delta rule, a gated recurrence element by element,
latent attention, attention within chunks whose heads mix their weights, a matrix memory, attention over everything before under
a soft cap and a sink, and a memory that fades by its one forget gate; feed-forwards that go with them.

A module holds weights; what a run of it carries from token to token is a ``states()`` mapping the
caller makes once per run, so that a layer run several times in a row has a state for each pass.
Constants and sizes are constructor arguments.  ``call`` is a ``batched.BatchCall``.
"""

from __future__ import annotations

import math

import numpy as np

from .. import functional as F
from ..common import graph as iron
from ..operators.experts import Experts, Router
from ..operators.mha_global import CachedHeads, GlobalMHA
from ..operators.mha_latent import EVERYTHING, LatentMHA, LatentRows
from ..operators.mha_talking import TalkingMHA, TurnedHeads
from ..operators.mha_window import WindowMHA
from ..operators.recurrent import (
    DeltaRule,
    HeadGate,
    Hgrn2,
    LowRankDecay,
    MatrixMemory,
    MemoryGate,
    MinGRU,
    ShortConv,
    TimeMix,
    TokenShift,
)
from ..operators.stream import (
    Activation,
    DepthAverage,
    GatedColumns,
    PolyNorm,
    StreamAdd,
    StreamCast,
    StreamGatedAdd,
    StreamNorm,
    StreamSum,
)
from .blocks import Linear


def as_rows(x, rows: int):
    """A projection's output as ``rows`` rows (a single row's product comes flat)."""
    return x if len(x.shape) == 2 else x.reshape(rows, x.elements // rows)


def distance_buckets(count: int, rows: int, bias_max: float) -> np.ndarray:
    """The row of a ``rows``-row distance-bias table that each of the distances ``0 .. count - 1`` reads:
    its own up to half the rows, then logarithmically spaced ones up to ``bias_max`` and the last row
    from there on.  In float32, as everything about positions."""
    half = np.float32(rows / 2)
    n = np.arange(count)
    far = n >= rows / 2
    ratio = np.maximum(n, 1).astype(np.float32) / half
    steps = np.log(ratio, dtype=np.float32) / np.float32(math.log(bias_max / (rows / 2))) * np.float32(rows - rows / 2)
    spaced = np.floor(half + np.floor(np.maximum(steps, 0)))
    return np.where(far, np.minimum(rows - 1, spaced), n).astype(np.int64)


class StreamRMSNorm(iron.Graph):
    """An RMS norm at the stream's edge: ``body`` takes a normed row out of it, ``add`` a block's output
    into it.  Gains are ``unit`` (0, or 1 where they are stored around zero) plus the weight.  ``groups``: the row is normed in
    that many equal parts, each by itself (out of the stream only)."""

    def __init__(self, width: int, eps: float, dtype, unit: float = 0.0, groups: int = 1):
        self.constants, self.groups = dict(epsilon=eps, unit=unit, dtype=dtype), groups
        self.weight = iron.param(width)

    def body(self, stream):
        return StreamNorm.step(stream, self.weight, groups=self.groups, **self.constants)

    def add(self, stream, y, y_bias=None):
        return StreamAdd.step(stream, y, self.weight, y_bias=y_bias, **self.constants)


class WindowAttention(iron.Graph):
    """Grouped-query sliding-window attention whose positions enter by a learned bias per distance bucket
    and head.  ``qkv`` is one packed projection (q heads, k heads, v heads).  Fills columns ``at ..`` of
    the mixer's row with the heads' outputs times ``out_scale``; the output projection is the mixer's."""

    def __init__(self, width, *, heads, kv_heads, dim, vdim, window, bias_rows, bias_max, scale, context, dtype, precision,
                 out_scale=1.0):
        self.heads, self.kv_heads, self.dim, self.vdim = heads, kv_heads, dim, vdim
        self.window = min(window, context)
        self.bias_max, self.scale, self.out_scale, self.dtype = bias_max, scale, out_scale, dtype
        self.qkv = Linear(width, heads * dim + kv_heads * (dim + vdim), precision=precision)
        self.rel = iron.param(bias_rows, heads)
        self.by_distance = None            # (heads, window) float32, spread from rel when the weights are loaded

    @property
    def out_width(self) -> int:
        return self.heads * self.vdim

    def loaded(self, as_float32) -> None:
        table = as_float32(self.rel.array)
        spread = table[distance_buckets(self.window, table.shape[0], self.bias_max)]
        self.by_distance = iron.Weight((self.heads, self.window), np.float32, np.ascontiguousarray(spread.T, dtype=np.float32))

    def states(self, slots: int) -> dict:
        # The ring holds just the window: a portion's own keys are read from its projection's rows.
        return {"keys": iron.state((slots, self.window, self.kv_heads, self.dim), self.dtype),
                "values": iron.state((slots, self.window, self.kv_heads, self.vdim), self.dtype)}

    def project(self, h):
        return as_rows(self.qkv(h), h.shape[0])

    def body(self, x, call, state, mixed, at=0):
        return WindowMHA.step(x, self.by_distance, call.spans, state["keys"], state["values"], mixed, scale=self.scale,
                              out_scale=self.out_scale, at=at, single=not call.prompt, dtype=self.dtype)[2]


class TimeMixing(iron.Graph):
    """Time mixing: r, k, v, a gate and a decay, each projected from its own blend of a token and the one
    before it, and a per-head outer-product state with a bonus for the current token.  Fills columns
    ``at ..`` of a ``width``-column mixer row."""

    BLENDS = "rkvgw"

    def __init__(self, width, *, heads, dim, rank, eps, dtype, precision, out_scale=1.0):
        self.width, self.heads, self.dim, self.eps, self.dtype, self.out_scale = width, heads, dim, eps, dtype, out_scale

        def dense(fan_out):
            return Linear(width, fan_out, precision=precision)

        inner = heads * dim
        self.mu = iron.param(len(self.BLENDS), width)
        self.r, self.k, self.v, self.g, self.w1 = dense(inner), dense(inner), dense(inner), dense(inner), dense(rank)
        self.w2 = iron.param(inner, rank)
        self.w0 = iron.param(inner)
        self.u = iron.param(heads, dim)
        self.norm = iron.param(inner)

    @property
    def out_width(self) -> int:
        return self.heads * self.dim

    def states(self, slots: int) -> dict:
        return {"before": iron.state((slots, 2, self.width), self.dtype),
                "memory": iron.state((slots, self.heads, self.dim, self.dim), np.float32)}

    def body(self, h, call, state, width, at=0):
        blends = TokenShift.step(h, self.mu, state["before"], call.spans, dtype=self.dtype)[1]
        r, k, v, g, z = (proj(call.bound(blends[i])) for i, proj in enumerate((self.r, self.k, self.v, self.g, self.w1)))
        r, k, v, g, z = (as_rows(x, h.shape[0]) for x in (r, k, v, g, z))
        decay = LowRankDecay.step(z, self.w2, self.w0, dtype=self.dtype)
        o = TimeMix.step(r, k, v, decay, self.u, state["memory"], call.spans, dtype=self.dtype)[1]
        return HeadGate.step(o, self.norm, gate=g, heads=self.heads, width=width, at=at, epsilon=self.eps, scale=self.out_scale,
                             dtype=self.dtype)


class ParallelMixer(iron.Graph):
    """Attention (``left``) and time mixing (``right``) of the same input, weighed and summed.  Their
    output projections are one product over the two outputs side by side, each scaled as it is made."""

    def __init__(self, width, left: WindowAttention, right: TimeMixing, *, precision):
        self.left, self.right = left, right
        self.out = Linear(left.out_width + right.out_width, width, precision=precision)

    def loaded(self, as_float32) -> None:
        self.left.loaded(as_float32)

    def states(self, slots: int) -> dict:
        return {**self.left.states(slots), **self.right.states(slots)}

    def body(self, h, call, state):
        # All projections of h, then both mixers: the runs a decode step launches as one each.
        x = self.left.project(h)
        mixed = self.right(h, call, state, self.out.in_features, at=self.left.out_width)
        return self.out(self.left(x, call, state, mixed))


class DeltaMixer(iron.Graph):
    """The gated delta rule: short convolutions over q, k and v, unit q and k, a write strength and a decay
    a head, a matrix state a value head, a gated norm a head.  ``proj`` is one packed projection
    (q, k, v, gate, b, a)."""

    def __init__(self, width, *, heads, kv_heads, dim, vdim, taps, eps, dtype, precision):
        self.heads, self.kv_heads, self.dim, self.vdim, self.taps = heads, kv_heads, dim, vdim, taps
        self.eps, self.dtype = eps, dtype
        self.channels = 2 * kv_heads * dim + heads * vdim
        inner = heads * vdim
        self.gate_at, self.b_at, self.a_at = self.channels, self.channels + inner, self.channels + inner + heads
        self.proj = Linear(width, self.a_at + heads, precision=precision)
        self.conv = iron.param(self.channels, taps)
        self.a_log = iron.param(heads)
        self.dt_bias = iron.param(heads)
        self.norm = iron.param(vdim)
        self.out = Linear(inner, width, precision=precision)

    def loaded(self, as_float32) -> None:
        pass

    def states(self, slots: int) -> dict:
        return {"inputs": iron.state((slots, self.taps, self.channels), self.dtype),
                "memory": iron.state((slots, self.heads, self.dim, self.vdim), np.float32)}

    def body(self, h, call, state):
        sizes = dict(kv_heads=self.kv_heads)
        x = as_rows(self.proj(h), h.shape[0])
        _, y = ShortConv.step(x, self.conv, self.a_log, self.dt_bias, state["inputs"], call.spans, dim=self.dim, vdim=self.vdim,
                              b_at=self.b_at, a_at=self.a_at, dtype=self.dtype, **sizes)
        _, o = DeltaRule.step(y, state["memory"], call.spans, **sizes)
        return self.out(HeadGate.step(o, self.norm, gate=x, heads=self.heads, gate_at=self.gate_at, epsilon=self.eps,
                                      dtype=self.dtype))


class StreamLayer(iron.Graph):
    """A sandwich layer around a float32 stream: the mixer, then the feed-forward (if any), each between a
    norm out of the stream and a norm back into it."""

    def __init__(self, width, mixer, mlp, *, eps, dtype):
        self.norm1, self.norm1b = StreamRMSNorm(width, eps, dtype), StreamRMSNorm(width, eps, dtype)
        self.mixer, self.mlp = mixer, mlp
        if mlp is not None:
            self.norm2, self.norm2b = StreamRMSNorm(width, eps, dtype), StreamRMSNorm(width, eps, dtype)
        self.rope = None

    def body(self, x, call, state):
        x = self.norm1b.add(x, as_rows(self.mixer(self.norm1(x), call, state), x.shape[0]))
        if self.mlp is not None:
            x = self.norm2b.add(x, as_rows(self.mlp(self.norm2(x)), x.shape[0]))
        return x


# ---- blocks whose packed projection carries, behind its own columns, a gate of ``gate`` columns for the layer


class GatedRecurrence(iron.Graph):
    """minGRU: a state a channel that a gate moves towards a candidate, read through a SiLU gate.  ``proj`` is one packed projection (z, x, g and the layer's gate)."""

    def __init__(self, width, *, inner, gate, dtype, precision):
        self.inner, self.dtype, self.own = inner, dtype, 3 * inner
        self.proj = Linear(width, self.own + gate, precision=precision)
        self.z_bias = iron.param(inner)
        self.x_bias = iron.param(inner)
        self.out = Linear(inner, width, precision=precision)

    def states(self, slots: int) -> dict:
        return {"memory": iron.state((slots, 2, self.inner), np.float32)}

    def body(self, x, call, state):
        return self.out(MinGRU.step(x, self.z_bias, self.x_bias, state["memory"], call.spans, dtype=self.dtype)[1])


class LatentAttention(iron.Graph):
    """Latent attention: queries through a normed latent of ``q_rank``; keys and values of every head from one
    of ``rank``, the only thing kept of a position beside ``rot`` key columns that all heads share, which turn with
    the position by ``angles``.  ``window`` None: everything before.  ``sink``: a learned term a head in the softmax's
    denominator.  ``proj`` is one packed projection (query latent, latent, shared key part and the layer's gate);
    ``room`` how many keys a prompt's portion may attend in all, ``portion`` its rows."""

    def __init__(self, width, *, heads, dim, vdim, q_rank, rank, scale, eps, gate, context, portion, room, dtype, precision, rot=0,
                 angles=None, window=None, sink=False):
        self.heads, self.rot, self.rank, self.scale, self.eps, self.dtype = heads, rot, rank, scale, eps, dtype
        self.own = q_rank + rank + rot
        self.window = EVERYTHING if window is None or window >= context else window
        self.context, self.portion, self.room = context, portion, room
        self.angles = angles
        self.proj = Linear(width, self.own + gate, precision=precision)
        self.q_norm = iron.param(q_rank)
        self.c_norm = iron.param(rank)
        self.query = Linear(q_rank, heads * (dim + rot), precision=precision)
        self.up = iron.param(heads * (dim + vdim), rank)
        self.sink = iron.param(heads) if sink else None
        self.out = Linear(heads * vdim, width, precision=precision)

    def states(self, slots: int) -> dict:
        # A portion's own rows are in the ring before they are attended: room for them beside the window.
        ring = min(self.context, self.window + self.portion)
        held = {"latents": iron.state((slots, ring, self.rank), self.dtype)}
        if self.rot:
            held["shared_keys"] = iron.state((slots, ring, self.rot), self.dtype)
        return held

    def keys(self, slots: int) -> int:
        """Keys a portion can attend here."""
        return min(self.room, slots * self.context, self.portion + slots * (self.window - 1))

    def body(self, x, call, state):
        beside = {"shared_keys": state.get("shared_keys"), "angles": self.angles}
        q = LatentRows.step(x, self.q_norm, self.c_norm, call.spans, state["latents"], epsilon=self.eps, dtype=self.dtype, **beside)[-1]
        q = as_rows(self.query(q), x.shape[0])
        y = LatentMHA.step(q, state["latents"], self.up, call.spans, heads=self.heads, scale=self.scale, window=self.window,
                           cap=self.keys(call.spans.shape[0]) if call.prompt else 0, single=not call.prompt, sink=self.sink,
                           dtype=self.dtype, **beside)
        return self.out(y)


class PolyNormMLP(iron.Graph):
    """A feed-forward of two biased projections around ``PolyNorm``.  ``proj`` is one packed projection (up and the
    layer's gate); the down projection's bias, ``out_bias``, is added where its product joins the stream."""

    def __init__(self, width, *, inner, gate, eps, dtype, precision):
        self.own, self.eps, self.dtype = inner, eps, dtype
        self.proj = Linear(width, inner + gate, precision=precision)
        self.bias = iron.param(inner)
        self.act = iron.param(4)
        self.out = Linear(inner, width, precision=precision)
        self.out_bias = iron.param(width)

    def body(self, x):
        return self.out(PolyNorm.step(x, self.act, bias=self.bias, cols=self.own, epsilon=self.eps, dtype=self.dtype))


class GatedStreamLayer(iron.Graph):
    """A pre-norm layer around a float32 stream: the mixer, then the feed-forward (if any), each joining the
    stream element by element through a sigmoid gate of what it was given."""

    def __init__(self, width, mixer, mlp, *, eps, dtype):
        self.dtype = dtype
        self.norm1, self.gate1_bias, self.mixer, self.mlp = StreamRMSNorm(width, eps, dtype), iron.param(width), mixer, mlp
        if mlp is not None:
            self.norm2, self.gate2_bias = StreamRMSNorm(width, eps, dtype), iron.param(width)
        self.rope = None

    def add(self, x, y, packed, block, bias):
        return StreamGatedAdd.step(x, as_rows(y, x.shape[0]), packed, bias, gate_at=block.own, dtype=self.dtype,
                                   y_bias=getattr(block, "out_bias", None))

    def body(self, x, call, state):
        packed = as_rows(self.mixer.proj(self.norm1(x)), x.shape[0])
        x = self.add(x, self.mixer(packed, call, state), packed, self.mixer, self.gate1_bias)
        if self.mlp is not None:
            packed = as_rows(self.mlp.proj(self.norm2(x)), x.shape[0])
            x = self.add(x, self.mlp(packed), packed, self.mlp, self.gate2_bias)
        return x


# ---- post-normed layers that read the stream itself, and average over what it was


class TalkingAttention(iron.Graph):
    """Grouped-query attention within chunks of ``chunk`` positions: biased projections, q and k normed a head and turned by
    ``angles``, scores times ``scale`` and the head's ``temp``, the heads' softmax weights mixed by ``talk``.  ``proj`` is one
    packed projection (q, k, v); ``out_bias`` is added where the output joins the stream.  ``mixes``: the values are blended
    with those of the call's first such layer by ``share``."""

    def __init__(self, width, *, heads, kv_heads, dim, vdim, chunk, scale, eps, context, dtype, precision, angles=None, mixes=False):
        self.heads, self.kv_heads, self.dim, self.vdim = heads, kv_heads, dim, vdim
        self.chunk = min(chunk, context)
        self.scale, self.eps, self.dtype, self.angles, self.mixes = scale, eps, dtype, angles, mixes
        packed = heads * dim + kv_heads * (dim + vdim)
        self.proj = Linear(width, packed, precision=precision)
        self.bias = iron.param(packed)
        self.q_norm = iron.param(dim)
        self.k_norm = iron.param(dim)
        self.temp = iron.param(heads)
        self.talk = iron.param(heads, heads)
        self.share = iron.param(1) if mixes else None
        self.out = Linear(heads * vdim, width, precision=precision)
        self.out_bias = iron.param(width)

    def states(self, slots: int) -> dict:
        # A position sees its own chunk only, so a ring of a chunk holds it in its first rows.
        return {"keys": iron.state((slots, self.chunk, self.kv_heads, self.dim), self.dtype),
                "values": iron.state((slots, self.chunk, self.kv_heads, self.vdim), self.dtype)}

    def body(self, h, call, state):
        beside, held = {"angles": self.angles}, call.kept.get("values") if self.mixes else None
        if held is not None:
            beside |= {"first": held[0], "share": self.share, "first_at": held[1]}
        x = TurnedHeads.step(as_rows(self.proj(h), h.shape[0]), self.bias, self.q_norm, self.k_norm, self.temp, call.spans,
                             kv_heads=self.kv_heads, scale=self.scale, epsilon=self.eps, dtype=self.dtype, **beside)
        if self.mixes and held is None:
            call.kept["values"] = x, (self.heads + self.kv_heads) * self.dim
        y = TalkingMHA.step(x, self.talk, call.spans, state["keys"], state["values"], single=not call.prompt, dtype=self.dtype)[2]
        return self.out(y)


class MatrixMemoryMixer(iron.Graph):
    """mLSTM: a matrix a head that keys and values are written into under exponential gates, read by queries, each head normed
    and gated.  ``proj`` is one packed projection (q, k, v, gate, input gate, forget gate)."""

    out_bias = None

    def __init__(self, width, *, heads, dim, vdim, cap, eps, dtype, precision):
        self.heads, self.dim, self.vdim, self.cap, self.eps, self.dtype = heads, dim, vdim, cap, eps, dtype
        self.gate_at = heads * (2 * dim + vdim)
        self.i_at = self.gate_at + heads * vdim
        self.proj = Linear(width, self.i_at + 2 * heads, precision=precision)
        self.i_bias = iron.param(heads)
        self.f_bias = iron.param(heads)
        self.norm = iron.param(heads * vdim)
        self.out = Linear(heads * vdim, width, precision=precision)

    def states(self, slots: int) -> dict:
        return {"memory": iron.state((slots, self.heads, self.dim, self.vdim + 1), np.float32),
                "tops": iron.state((slots, 2, self.heads), np.float32)}

    def body(self, h, call, state):
        x = as_rows(self.proj(h), h.shape[0])
        o = MatrixMemory.step(x, self.i_bias, self.f_bias, state["memory"], state["tops"], call.spans, i_at=self.i_at,
                              f_at=self.i_at + self.heads, cap=self.cap, dtype=self.dtype)[2]
        return self.out(MemoryGate.step(o, x, self.norm, heads=self.heads, gate_at=self.gate_at, epsilon=self.eps, dtype=self.dtype))


class ActivatedMLP(iron.Graph):
    """``down(act(up h))``."""

    def __init__(self, width, *, inner, activation, dtype, precision):
        self.kind, self.dtype = activation, dtype
        self.up = Linear(width, inner, precision=precision)
        self.down = Linear(inner, width, precision=precision)

    def body(self, h):
        return self.down(Activation.step(as_rows(self.up(h), h.shape[0]), kind=self.kind, dtype=self.dtype))


class ExpertsMLP(iron.Graph):
    """Gated feed-forwards of which a router chooses ``top`` a row.  The experts' matrices are stacked.  ``scored``: the choice and
    the shares are by the softmax over all of the router's logits, the choice by its scores plus corrections; else by biased
    logits and a softmax over the chosen.  ``identity``: the router's last ones, that many, hand on the row itself."""

    def __init__(self, width, *, inner, experts, top, activation, dtype, scored=False, identity=0):
        self.top, self.kind, self.dtype, self.scored, self.identity = top, activation, dtype, scored, identity
        self.router = iron.param(experts + identity, width)
        self.router_bias = None if scored else iron.param(experts)
        self.correction = iron.param(experts + identity) if scored else None
        self.gate = iron.param(experts * inner, width)
        self.up = iron.param(experts * inner, width)
        self.down = iron.param(experts * width, inner)

    def body(self, h):
        return self.apply(h, *self.choose(h))

    def choose(self, h):
        return Router.step(h, self.router, bias=self.router_bias, correction=self.correction, scored=self.scored, top=self.top, dtype=self.dtype)

    def apply(self, h, ids, shares):
        return Experts.step(h, self.gate, self.up, self.down, ids, shares, activation=self.kind, identity=self.identity, dtype=self.dtype)


class PostNormLayer(iron.Graph):
    """A layer around a float32 stream whose blocks read the stream itself and are normed where they join it.  Layer ``index``'s
    result is kept with those of the layers before it, and what goes on is the sum of all by ``depth``."""

    def __init__(self, width, mixer, mlp, *, index, eps, dtype, unit=0.0):
        self.dtype, self.mixer, self.mlp = dtype, mixer, mlp
        self.norm1 = StreamRMSNorm(width, eps, dtype, unit)
        if mlp is not None:
            self.norm2 = StreamRMSNorm(width, eps, dtype, unit)
        self.depth = iron.param(index + 2)
        self.rope = None

    def body(self, x, call, state):
        h = StreamCast.step(x, dtype=self.dtype)
        x = self.norm1.add(x, as_rows(self.mixer(h, call, state), x.shape[0]), self.mixer.out_bias)
        if self.mlp is not None:
            x = self.norm2.add(x, as_rows(self.mlp(StreamCast.step(x, dtype=self.dtype)), x.shape[0]))
        return DepthAverage.step(x, call.planes, self.depth)[0]


# ---- layers whose mixer and feed-forward read one norm of the stream side by side: one projection into both, one out of both


class GlobalAttention(iron.Graph):
    """Grouped-query attention over everything before: q and k normed a head, turned by ``angles`` in halves, values over their
    root mean square (``value_norm``), scores times ``scale`` under a soft ``cap`` (0: none), ``sink`` one more in the softmax's
    denominator.  Its columns of a packed projection's row are (q, k, v); fills the first ``out_width`` columns of a ``width``-column row."""

    def __init__(self, *, heads, kv_heads, dim, vdim, scale, eps, context, dtype, angles=None, cap=0.0, sink=False, value_norm=False):
        self.heads, self.kv_heads, self.dim, self.vdim = heads, kv_heads, dim, vdim
        self.scale, self.cap, self.sink, self.value_norm = scale, cap, sink, value_norm
        self.eps, self.context, self.dtype, self.angles = eps, context, dtype, angles
        self.own, self.out_width = heads * dim + kv_heads * (dim + vdim), heads * vdim
        self.q_norm = iron.param(dim)
        self.k_norm = iron.param(dim)

    def states(self, slots: int) -> dict:
        # A key head's positions one after the other: a step reads them as one run.
        return {"keys": iron.state((slots, self.kv_heads, self.context, self.dim), self.dtype),
                "values": iron.state((slots, self.kv_heads, self.context, self.vdim), self.dtype)}

    def body(self, x, call, state, width):
        keys, values, q = CachedHeads.step(x, self.q_norm, self.k_norm, call.spans, state["keys"], state["values"], angles=self.angles,
                                           heads=self.heads, value_norm=self.value_norm, epsilon=self.eps, dtype=self.dtype)
        return GlobalMHA.step(q, keys, values, call.spans, width=width, scale=self.scale, cap=self.cap, sink=self.sink,
                              single=not call.prompt, dtype=self.dtype)


class FadingMemory(iron.Graph):
    """HGRN2: a matrix a head that a forget gate a channel fades and, by what it leaves, writes, each head normed.  Its columns of
    a packed projection's row are (q, forget gate, v); fills the first ``out_width`` columns of a ``width``-column row."""

    def __init__(self, *, heads, dim, vdim, eps, dtype):
        self.heads, self.dim, self.vdim, self.eps, self.dtype = heads, dim, vdim, eps, dtype
        self.own, self.out_width = heads * (2 * dim + vdim), heads * vdim
        self.f_bias = iron.param(heads * dim)
        self.lower = iron.param(heads * dim)
        self.norm = iron.param(vdim)

    def states(self, slots: int) -> dict:
        return {"memory": iron.state((slots, self.heads, self.dim, self.vdim), np.float32)}

    def body(self, x, call, state, width):
        _, o = Hgrn2.step(x, self.f_bias, self.lower, state["memory"], call.spans, dtype=self.dtype)
        return HeadGate.step(o, self.norm, heads=self.heads, width=width, epsilon=self.eps, dtype=self.dtype)


class SideBySideLayer(iron.Graph):
    """``h = norm(x); x += mixer(h) + ff(h)`` around a float32 stream.  ``proj`` packs the mixer's columns and those of a gated
    feed-forward of ``inner`` (gate, up; ``kind`` and ``limit`` as GatedColumns has them); ``out`` is the output projections of
    both side by side; ``routed`` a feed-forward of experts beside them (or None)."""

    def __init__(self, width, mixer, *, inner=0, kind="silu", limit=0.0, routed=None, eps, groups, dtype, precision):
        self.mixer, self.routed, self.inner, self.kind, self.limit, self.dtype = mixer, routed, inner, kind, limit, dtype
        self.norm1 = StreamRMSNorm(width, eps, dtype, groups=groups)
        self.proj = Linear(width, mixer.own + 2 * inner, precision=precision)
        self.out = Linear(mixer.out_width + inner, width, precision=precision)
        self.rope = None

    def body(self, x, call, state):
        rows, h = x.shape[0], self.norm1(x)
        packed = as_rows(self.proj(h), rows)
        chosen = self.routed.choose(h) if self.routed is not None else None   # (what a decode step makes in one launch, side by side)
        made = self.mixer(packed, call, state, self.out.in_features)
        if self.inner:
            made = GatedColumns.step(packed, made, cols=self.inner, gate_at=self.mixer.own, at=self.mixer.out_width, kind=self.kind,
                                     limit=self.limit, dtype=self.dtype)
        beside = {"also": as_rows(self.routed.apply(h, *chosen), rows)} if chosen is not None else {}
        return StreamSum.step(x, as_rows(self.out(made), rows), dtype=self.dtype, **beside)
