"""Building blocks of a decoder; each is a small graph whose ``body`` records operator steps.

Module and parameter names are the Hugging Face ones the reference uses too (iron/lm/blocks.py:
``Linear`` :269, ``RMSNorm`` :321, ``Rope`` :394, ``KVCache`` :434, ``Attention`` :563, ``GatedMLP``
:676, ``DecoderLayer`` :702, ``SandwichLayer`` :748, ``PleLayer`` :770), because a checkpoint's
tensors are bound to them by dotted path.  What a body records, and in which order, is part of the
contract with ``common.fusion``: the runs it turns into single launches (norm -> q/k/v -> RoPE ->
cache rows; norm -> gate/up -> activation -> product; projection -> residual) are recognised by
their step sequence.
"""

from __future__ import annotations

import dataclasses
import functools

from .. import functional as F
from ..bf16 import bfloat16, round_bf16
from ..common import graph as iron
from ..common.declare import Precision
from ..operators.axpy import AXPY
from ..operators.copy import Copy
from ..operators.gelu import GELU
from ..operators.mha import MHA
from ..operators.stream import GatedProduct

# ``hidden_act`` as a config spells it -> what records it (iron/lm/blocks.py:246-266)
_ACTIVATIONS = {
    "silu": lambda: F.silu,
    "gelu_pytorch_tanh": lambda: functools.partial(GELU.step, approximate="tanh"),
    "gelu": lambda: functools.partial(GELU.step, approximate="none"),
    "relu": lambda: F.relu,
}
# the names a gated product in 32 bits has for them
_FLOAT_GATES = {"silu": "silu", "gelu_pytorch_tanh": "gelu_tanh", "relu": "relu"}


def activation(name: str):
    """The recorder for a config's ``hidden_act``.

    Raises:
        ValueError: an activation no operator here implements.
    """
    if name not in _ACTIVATIONS:
        raise ValueError(f"hidden_act {name!r}: no operator here computes it")
    return _ACTIVATIONS[name]()


class Linear(iron.Graph):
    """A dense layer stored the PyTorch way: ``weight`` is ``(out_features, in_features)`` and the
    body computes ``x @ weight.T`` (+ ``bias``).  One row becomes a GEMV, several a GEMM."""

    def __init__(self, in_features: int, out_features: int, bias: bool = False, *, precision: Precision):
        self.in_features = in_features
        self.out_features = out_features
        self.precision = precision
        self.weight = iron.param(out_features, in_features)
        self.bias = iron.param(out_features) if bias else None

    def body(self, x):
        return F.linear(x, self.weight, self.bias, precision=self.precision)


class Embedding(iron.Graph):
    """A table of ``num_embeddings`` rows of width ``embedding_dim``; the body gathers rows by id."""

    def __init__(self, num_embeddings: int, embedding_dim: int):
        self.num_embeddings = num_embeddings
        self.embedding_dim = embedding_dim
        self.weight = iron.param(num_embeddings, embedding_dim)

    def body(self, ids):
        table = iron.weight(self.weight)
        return Copy.step(table[ids])


class RMSNorm(iron.Graph):
    """Root-mean-square normalisation of the trailing axis with a learned gain ``weight``."""

    def __init__(self, normalized_shape, eps: float | None = None):
        shape = (normalized_shape,) if isinstance(normalized_shape, int) else tuple(normalized_shape)
        self.normalized_shape = shape
        self.eps = eps
        self.weight = iron.param(*shape)

    def body(self, x):
        return F.rms_norm(x, self.normalized_shape, self.weight, self.eps)


def residual_add(x, y, residual: float = 1.0):
    """``x + residual * y`` shaped like ``x``: a plain sum when the weight is 1, else one AXPY step
    (iron/lm/blocks.py:386-391).  Either way the fused projections take it into their epilogue."""
    if y.shape != x.shape:
        y = y.reshape(x.shape)
    return x + y if residual == 1 else AXPY.step(y, x, scalar_factor=residual)


class Rope(iron.Graph):
    """The rotary table of a decoder, bf16, a row of interleaved (cos, sin) per position.

    A call copies the rows it needs out of the table once and every layer rotates by that copy: a
    prompt chunk takes ``chunk`` rows from its start (bounded by the rows it really has), a decode
    step the single row at its position."""

    def __init__(self, c):
        self.table = iron.weight(round_bf16(c.angles()))
        self.chunk = c.prefill_chunk
        self.width = c.rope_width

    def rows(self, call) -> tuple:
        """``(angles for q, angles for k)`` of this call -- one copy serves both."""
        if call.prompt:
            window = self.table[call.start : call.start + self.chunk]
            picked = Copy.step(window[: call.rows])
        else:
            picked = Copy.step(self.table[call.position]).reshape(1, self.width)
        return picked, picked


class KVCache(iron.Graph):
    """Keys and values of one layer (or of several layers sharing them), laid out
    ``(rows, kv_heads, head_dim)`` so that one position is one contiguous row, plus the attention
    over them (iron/lm/blocks.py:434-529).

    Two layouts.  *Linear*: one row per position up to ``max_seq_len``.  *Ring*, for a sliding
    ``window`` much shorter than the context: ``R`` = ``window + prefill_chunk`` rounded up to a
    power of two; the buffer has ``2R`` rows and position ``p`` is written twice, at ``p % R`` and
    ``R`` rows further on.  Thanks to the mirror, the window ending at any position is ONE contiguous
    run of rows, and attention reads it in place (``iron_mha_*_at_bf16`` take the first row from a
    device word) instead of staging a copy.  A ring is used only when three of them would fit the
    context; otherwise it saves nothing worth its complication.

    Args:
        window: how many earlier positions a query sees besides its own; None = all of them.

    Raises:
        ValueError: a ring is called for but the chunk length is not a power of two.
    """

    def __init__(self, c, window: int | None = None):
        heads, width = c.num_key_value_heads, c.head_dim
        self.chunk, self.window = c.prefill_chunk, window
        self.ring = None
        rows = c.max_seq_len
        if window is not None:
            ring = 1 << (window + self.chunk - 1).bit_length()
            if 3 * ring < rows:
                if self.chunk & (self.chunk - 1):
                    raise ValueError(f"KVCache: a {self.chunk}-position chunk is no power of two")
                self.ring, rows = ring, 2 * ring
        self.keys = iron.state((rows, heads, width))
        self.values = iron.state((rows, heads, width))

    def restart(self, held: int, ran: int) -> int:
        """The position a run must begin at to redo everything from ``held`` on, given that ``ran``
        positions have been through the cache.  A linear cache can resume anywhere.  A ring resumes
        at the chunk boundary at or below ``held`` provided the window in front of that boundary has
        not been overwritten yet; if it has, only a run from position 0 is sound."""
        if self.ring is None:
            return held
        boundary = held - held % self.chunk
        oldest_needed = boundary - self.window
        return boundary if ran - oldest_needed <= self.ring else 0

    def attend(self, call, q, k, v, scale: float | None = None):
        """Store this call's ``k`` / ``v`` (``(rows, kv_heads, head_dim)``; None when another layer
        owns the cache and has stored them already), then attend ``q`` (``(rows, heads, head_dim)``)
        causally over everything up to the call's position.  Returns ``(rows, heads * head_dim)``."""
        rows, heads, width = q.shape
        if self.ring is None:
            self._store_linear(call, k, v)
            upto = call.position + 1
            keys, values = self.keys[:upto], self.values[:upto]
        else:
            keys, values, q = self._ring(call, q, k, v)
        out = MHA.step(q, keys, values, heads_interleaved=True, kv_interleaved=True, window=self.window,
                       scale=scale)
        if self.ring is not None and call.prompt:
            out = out[: call.rows]     # the ring's chunk ran unbounded; keep the call's own rows
        return out.reshape(rows, heads * width)

    def _store_linear(self, call, k, v) -> None:
        _, kv_heads, width = self.keys.shape
        for new, cache in ((k, self.keys), (v, self.values)):
            if new is None:
                continue
            if call.prompt:
                cache[call.start : call.start + self.chunk][: call.rows] = new
            else:
                cache[call.position] = new.reshape(kv_heads, width)

    def _ring(self, call, q, k, v):
        """Store into the ring (both copies) and pick the run of rows to attend over.

        Prompt chunk: the keys are the last ``R`` positions ending with the chunk's last slot; all
        ``chunk`` query rows attend (rows past the call's bound compute garbage that ``attend``
        drops), so the queries lose their bound here.  Decode step: the window plus the position
        itself, ``W + 1`` rows."""
        R, W, C = self.ring, self.window, self.chunk
        if call.prompt:
            slot, span = call.start % R, C
            first = iron.clamp(call.start + C - R, lo=0) % R
            length, count = R, iron.clamp(call.start + C, hi=R)
            q = dataclasses.replace(q, valid={})
        else:
            slot, span = call.position % R, None
            first = iron.clamp(call.position - W, lo=0) % R
            length, count = W + 1, iron.clamp(call.position + 1, hi=W + 1)
        for new, ring in ((k, self.keys), (v, self.values)):
            if new is None:
                continue
            for row in (slot, slot + R):                  # the slot and its mirror
                if span is None:
                    ring[row] = new.reshape(ring.shape[1:])
                else:
                    ring[row : row + span][: call.rows] = new
        keys = self.keys[first : first + length][:count]
        values = self.values[first : first + length][:count]
        return keys, values, q


class Attention(iron.Graph):
    """Grouped-query self-attention of layer ``i`` (iron/lm/blocks.py:563-660): project, optionally
    RMS-norm each head (``norms`` lists which of q, k, v: q and k with learned gains ``q_norm`` /
    ``k_norm``, v without), rotate q and k, attend over the layer's ``KVCache``, project back.

    A layer that reads another layer's cache has no use for k and v: the caller sets its
    ``k_proj`` / ``v_proj`` / ``k_norm`` to None after construction.

    Raises:
        ValueError: ``norms`` contains a letter other than q, k, v.
    """

    def __init__(self, c, i: int, norms: str = ""):
        stray = set(norms) - {"q", "k", "v"}
        if stray:
            raise ValueError(f"Attention: norms {norms!r} names other than q, k and v")
        self.heads, self.groups, self.head_dim = c.num_attention_heads, c.num_key_value_heads, c.head_dim
        hidden, q_width, kv_width = c.hidden_size, self.heads * self.head_dim, self.groups * self.head_dim

        def dense(fan_in, fan_out):
            return Linear(fan_in, fan_out, bias=c.attention_bias, precision=c.precision)

        self.q_proj = dense(hidden, q_width)
        self.k_proj = dense(hidden, kv_width)
        self.v_proj = dense(hidden, kv_width)
        self.o_proj = dense(q_width, hidden)
        self.q_norm = RMSNorm(self.head_dim, c.eps) if "q" in norms else None
        self.k_norm = RMSNorm(self.head_dim, c.eps) if "k" in norms else None
        self.v_norm = "v" in norms
        self.eps = c.eps
        self.scaling: float | None = None      # None: 1/sqrt(head_dim)

    def project(self, x, **gemv) -> list:
        """``[q, k, v]`` of ``x`` (None where the projection is absent); ``gemv`` are tunables a
        single-row projection carries."""
        out = []
        for proj in (self.q_proj, self.k_proj, self.v_proj):
            out.append(None if proj is None else
                       F.linear(x, proj.weight, proj.bias, precision=proj.precision, **gemv))
        return out

    def rotate(self, x, angles):
        """RoPE on ``x`` ``(rows, head_dim)``.  Under partial rotary (``config.rotary_dim``) the table
        is narrower than a head: one ``RoPE`` step turns the leading columns it covers and passes the
        rest through, where the reference copies them out and back (iron/lm/blocks.py:612-620)."""
        return F.rope(x, angles)

    def body(self, x, cache, call, angles=None):
        rows, H, G, D = x.shape[0], self.heads, self.groups, self.head_dim
        # The reference's decode GEMVs tile half a head per output tile; carried for its profiles.
        q, k, v = self.project(x, **({"tile_size_output": D // 2} if rows == 1 else {}))
        own_kv = k is not None
        q = q.reshape(rows * H, D)
        if self.q_norm is not None:
            q = self.q_norm(q)
        if own_kv:
            k, v = k.reshape(rows * G, D), v.reshape(rows * G, D)
            if self.k_norm is not None:
                k = self.k_norm(k)
            if self.v_norm:
                v = F.rms_norm(v, (D,), eps=self.eps)
        if angles is not None:
            q_angles, k_angles = angles
            q = self.rotate(q, q_angles)
            if own_kv:
                k = self.rotate(k, k_angles)
        if own_kv:
            k, v = k.reshape(rows, G, D), v.reshape(rows, G, D)
        mixed = cache.attend(call, q.reshape(rows, H, D), k, v, scale=self.scaling)
        return self.o_proj(mixed)


class GatedMLP(iron.Graph):
    """The gated feed-forward ``down_proj(act(gate_proj(x)) * up_proj(x))``."""

    def __init__(self, c):
        hidden, inner = c.hidden_size, c.intermediate_size

        def dense(fan_in, fan_out):
            return Linear(fan_in, fan_out, bias=c.mlp_bias, precision=c.precision)

        self.gate_proj = dense(hidden, inner)
        self.up_proj = dense(hidden, inner)
        self.down_proj = dense(inner, hidden)
        self.act = activation(c.hidden_act)
        self.hidden_act = c.hidden_act

    def body(self, x):
        gate = self.gate_proj(x)
        up = self.up_proj(x)
        if gate.dtype is not bfloat16:   # a model that runs in 32 bits throughout
            return self.down_proj(GatedProduct.step(gate, up, activation=_FLOAT_GATES[self.hidden_act]))
        return self.down_proj(self.act(gate) * up)


class DecoderLayer(iron.Graph):
    """Pre-norm decoder layer ``i``: ``x += attn(norm(x))`` then ``x += mlp(norm(x))``, both sums
    weighted by ``residual_multiplier``.  ``self_attn``, ``mlp`` and ``cache`` may be handed in (a
    model with its own flavour of them); ``rope`` is set by the model to the table this layer
    rotates by."""

    def __init__(self, c, i: int, self_attn=None, mlp=None, cache=None):
        self.input_layernorm = RMSNorm(c.hidden_size, c.eps)
        self.self_attn = self_attn if self_attn is not None else Attention(c, i)
        self.post_attention_layernorm = RMSNorm(c.hidden_size, c.eps)
        self.mlp = mlp if mlp is not None else GatedMLP(c)
        self.cache = cache if cache is not None else KVCache(c, c.window)
        self.rope = None
        self.residual_multiplier = 1.0

    def mix(self, h, call):
        """The attention block on normed input ``h``."""
        angles = call.ropes[id(self.rope)] if self.rope is not None else None
        return self.self_attn(h, self.cache, call, angles)

    def body(self, x, call):
        weight = self.residual_multiplier
        x = residual_add(x, self.mix(self.input_layernorm(x), call), weight)
        return residual_add(x, self.mlp(self.post_attention_layernorm(x)), weight)


class SandwichLayer(DecoderLayer):
    """Gemma's layer (iron/lm/blocks.py:748-767): norms on both sides of each block.  Attention is
    normed before (``input_layernorm``) and after (``post_attention_layernorm``), the feed-forward
    before (``pre_feedforward_layernorm``) and after (``post_feedforward_layernorm``); the residual
    takes the post-normed output."""

    def __init__(self, c, i: int, self_attn=None, mlp=None, cache=None):
        super().__init__(c, i, self_attn, mlp, cache)
        self.pre_feedforward_layernorm = RMSNorm(c.hidden_size, c.eps)
        self.post_feedforward_layernorm = RMSNorm(c.hidden_size, c.eps)

    def body(self, x, call):
        weight = self.residual_multiplier
        attended = self.mix(self.input_layernorm(x), call)
        x = residual_add(x, self.post_attention_layernorm(attended), weight)
        fed = self.mlp(self.pre_feedforward_layernorm(x))
        return residual_add(x, self.post_feedforward_layernorm(fed), weight)


class PleLayer(SandwichLayer):
    """Gemma 4's layer (iron/lm/blocks.py:770-800): a sandwich layer followed by the per-layer
    input.  ``ple`` (``(rows, ple_dim)``) gates a down-projection of the hidden state
    (``per_layer_input_gate``), is projected back up (``per_layer_projection``), normed
    (``post_per_layer_input_norm``) and added; finally everything is multiplied by the layer's
    scalar, held as a constant row ``scale`` the model fills from ``layer_scalar``."""

    def __init__(self, c, i: int, self_attn=None, mlp=None, cache=None):
        super().__init__(c, i, self_attn, mlp, cache)
        hidden, narrow = c.hidden_size, c.ple_dim
        self.per_layer_input_gate = Linear(hidden, narrow, False, precision=c.precision)
        self.per_layer_projection = Linear(narrow, hidden, False, precision=c.precision)
        self.post_per_layer_input_norm = RMSNorm(hidden, c.eps)
        self.layer_scalar = iron.param(1)

    def body(self, x, call, ple):
        x = super().body(x, call)
        gated = self.mlp.act(self.per_layer_input_gate(x)) * ple
        extra = self.post_per_layer_input_norm(self.per_layer_projection(gated))
        return residual_add(x, extra, self.residual_multiplier) * self.scale
