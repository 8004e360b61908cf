"""The operators' ``reference()`` methods, restated on ``oracle.ops`` -- TEST INFRASTRUCTURE.

``install()`` registers one function per operator class into
``iron_amd.common.declare.REFERENCES``; each takes the constructed operator and its
inputs as numpy arrays, as the reference's methods do (file:line cited per function).
"""

from __future__ import annotations

import numpy as np

from iron_amd.bf16 import bfloat16, round_bf16

from . import ops


def gemm(op, A, B):
    """iron/operators/gemm.py:696-702."""
    return ops.gemm(A, B, b_col_maj=op.b_col_maj, c_col_maj=op.c_col_maj, valid_k=op.valid_k)


def gemv(op, A, B):
    """iron/operators/gemv.py:408-417."""
    return ops.gemv(A, B, repeat=op.repeat)


def rms_norm(op, x, weight=None):
    """iron/common/elementwise.py:676-682 over norm.rms_norm_eps."""
    return ops.rms_norm(np.asarray(x).reshape(op.rows, op.tile_size), weight, epsilon=op.epsilon)


def silu(op, x):
    return ops.silu(x)


def mul(op, a, b):
    return ops.mul(a, np.asarray(b).reshape(np.shape(a)))


def add(op, a, b):
    return ops.add(a, np.asarray(b).reshape(np.shape(a)))


def gelu(op, x):
    """iron/operators/gelu.py:13-40."""
    return ops.gelu(x, op.approximate)


def relu(op, x):
    return ops.relu(x)


def sigmoid(op, x):
    return ops.sigmoid(x)


def tanh(op, x):
    return ops.tanh(x)


def clamp(op, x):
    """iron/operators/clamp.py:14-63."""
    return ops.clamp(x, op.low, op.high)


def axpy(op, a, b):
    """iron/operators/axpy.py:13-31: ``scalar_factor * a + b``."""
    return ops.axpy(op.scalar_factor, a, np.asarray(b).reshape(np.shape(a)))


def layer_norm(op, x, weight=None):
    """iron/common/elementwise.py:676-682 over norm.layer_norm_eps."""
    return ops.layer_norm(np.asarray(x).reshape(op.rows, op.tile_size), weight, epsilon=op.epsilon)


def softmax(op, x, addend=None):
    """iron/operators/softmax.py:523-545; a bounded call's ``length`` read off the operator."""
    length = vars(op).get("_extents", {}).get("length")
    return ops.softmax(np.asarray(x).reshape(op.rows, op.cols),
                       None if addend is None else np.asarray(addend).reshape(op.rows, op.cols),
                       soft_cap=op.soft_cap, length=length)


def rowwise_add(op, x, row):
    """iron/common/elementwise.py:797-867 over eltwise.add_sized: every row plus the one row."""
    x = np.asarray(x).reshape(op.rows, op.tile_size)
    return ops.add(x, np.broadcast_to(np.asarray(row).reshape(1, -1), x.shape))


def rowwise_mul(op, x, row):
    """iron/common/elementwise.py:797-867 over eltwise.mul_sized."""
    x = np.asarray(x).reshape(op.rows, op.tile_size)
    return ops.mul(x, np.broadcast_to(np.asarray(row).reshape(1, -1), x.shape))


def rope(op, x, angles):
    """iron/operators/rope.py:167-184; with a row wider than the table, the first columns turn and the
    rest pass through (the reference's Attention.rotate, iron/lm/blocks.py:612-620)."""
    x = np.asarray(x)
    if op.row == op.cols:
        return ops.rope(x, angles, two_halves=op.two_halves)
    y = np.array(x, dtype=np.float32).reshape(op.rows, op.row)
    y[:, : op.cols] = ops.rope(y[:, : op.cols], angles, two_halves=op.two_halves)
    return y


def mha(op, Q, K, V):
    """iron/operators/mha.py:1073-1116; a bounded call's extents read off the operator."""
    ext = vars(op).get("_extents", {})
    return ops.mha(Q, K, V, num_heads=op.num_heads, num_KV_heads=op.num_KV_heads, seq_len=op.seq_len,
                   kv_len=op.kv_len, d=op.d, causal=op.causal, window=op.window, scale=op.scale,
                   heads_interleaved=op.heads_interleaved, kv_interleaved=op.kv_interleaved,
                   valid=ext.get("valid"), kv_valid=ext.get("kv_valid"))


def copy(op, src):
    """iron/operators/copy.py:839-902: exact."""
    return np.array(src).reshape(op.shape)


def gather(op, table, control, *, valid_rows=None):
    """iron/operators/copy.py:72-378: the rows of ``table`` the first ``rows`` control words name;
    rows past ``valid_rows`` are not written (zeros here)."""
    ids = np.asarray(control).reshape(-1)[: op.rows].astype(np.int64)
    n = op.rows if valid_rows is None else int(valid_rows)
    y = np.zeros((op.rows, op.row), np.asarray(table).dtype)
    y[:n] = np.asarray(table).reshape(op.table_rows, op.row)[ids[:n]]
    return y


def gather_words(op, ids, *, valid_rows=None, base_lo=0, base_hi=0):
    """iron/operators/copy.py:380-470 as this build defines it: the ids themselves, first in ``control``."""
    control = np.zeros(op.words, np.int32)
    n = op.rows if valid_rows is None else int(valid_rows)
    control[:n] = np.asarray(ids).reshape(-1)[:n]
    return control


def sample(op, logits, draws, tokens, *, row=0, at=0):
    """iron/operators/sample.py:72-79,324-333: the draw at ``draws`` word ``row``, recorded at ``at``."""
    words = np.asarray(draws).reshape(-1)[row : row + 4]
    temperature, top_k, n53 = ops.draw_words(words)
    token = ops.sample_ref(np.asarray(logits).reshape(-1)[: op.drawable], temperature, top_k, n53, op.k_max)
    tokens = np.array(tokens, dtype=np.int32).reshape(-1)
    tokens[at] = token
    return tokens, np.array([token], dtype=np.int32)


# ---- the float32 stream and the layers that carry a state.  ``_out`` rounds to the operator's dtype.


def _out(op, x):
    x = np.asarray(x, np.float32)
    return round_bf16(x) if op.dtype is bfloat16 else x


def _spans(spans):
    """(slot, first row, rows, first position) of every slot that has rows."""
    return [(s, int(r), int(n), int(p)) for s, (r, n, p, _) in enumerate(np.asarray(spans)) if n]


def stream_embed(op, table, ids):
    rows = np.asarray(table, np.float32)[np.clip(np.asarray(ids).reshape(-1), 0, op.table_rows - 1)] * np.float32(op.scale)
    return (rows, rows) if op.twice else rows


def _unit_rms(x, eps):
    x = np.asarray(x, np.float64)
    return x / np.sqrt((x * x).mean(-1, keepdims=True) + eps)


def stream_norm(op, x, weight):
    x = np.reshape(x, (op.rows, op.cols))
    parts = _unit_rms(np.reshape(x, (op.rows, op.groups, -1)), op.epsilon).reshape(x.shape)
    return _out(op, parts * (op.unit + np.asarray(weight, np.float64)))


def stream_add(op, x, y, weight, *, y_bias=None):
    z = np.asarray(y, np.float64) + (0 if y_bias is None else y_bias)
    return np.asarray(x + _unit_rms(z, op.epsilon) * (op.unit + np.asarray(weight, np.float64)), np.float32)


def depth_average(op, x, planes, weights):
    planes = np.array(planes)
    planes[op.count - 1, : op.rows] = np.reshape(x, (op.rows, op.cols))
    return np.einsum("j,jrc->rc", np.asarray(weights, np.float64), planes[: op.count, : op.rows].astype(np.float64)).astype(np.float32), planes


def stream_cast(op, x):
    return _out(op, x)


def _sigmoid(z):
    return 1 / (1 + np.exp(-np.asarray(z, np.float64)))


def stream_gated_add(op, x, y, gate, gate_bias, *, y_bias=None):
    y = np.asarray(y, np.float64) + (0 if y_bias is None else y_bias)
    z = np.asarray(gate, np.float64)[:, op.gate_at : op.gate_at + op.cols] + gate_bias
    return np.asarray(x + y * _sigmoid(z), np.float32)


def poly_norm(op, x, coefficients, *, bias=None):
    z = np.asarray(x, np.float64)[:, op.at : op.at + op.cols] + (0 if bias is None else bias)
    a, b, c, e = np.asarray(coefficients, np.float64)
    return _out(op, a * _unit_rms(z, op.epsilon) + b * _unit_rms(z**2, op.epsilon) + c * _unit_rms(z**3, op.epsilon) + e)


def min_gru(op, x, z_bias, x_bias, state, spans):
    W, state, y = op.width, np.array(state), np.zeros((op.rows, op.width), np.float32)
    x = np.asarray(x, np.float64)
    z, u, g = _sigmoid(x[:, :W] + z_bias), x[:, W : 2 * W] + x_bias, x[:, 2 * W : 3 * W]
    c = np.where(u >= 0, u + 0.5, _sigmoid(u))
    for s, row, n, start in _spans(spans):
        S = np.asarray(state[s, (start - 1) % 2], np.float64) if start else np.zeros(W)
        for t in range(row, row + n):
            S = (1 - z[t]) * S + z[t] * c[t]
            y[t] = S * g[t] * _sigmoid(g[t])
        state[s, (start + n - 1) % 2] = S
    return state, _out(op, y)


def _turn(x, angles, turned):
    """The first ``turned`` of x's trailing columns turned, pair by pair, by rows of (cos, sin)."""
    x = np.array(x, np.float64)
    c, s = np.asarray(angles, np.float64)[..., 0::2], np.asarray(angles, np.float64)[..., 1::2]
    u, v = x[..., 0:turned:2].copy(), x[..., 1:turned:2].copy()
    x[..., 0:turned:2], x[..., 1:turned:2] = u * c - v * s, v * c + u * s
    return x


def latent_rows(op, x, q_gain, c_gain, spans, latents, *, shared_keys=None, angles=None):
    x, latents, q = np.asarray(x, np.float64), np.array(latents), np.zeros((op.rows, op.q_rank), np.float32)
    keys = None if shared_keys is None else np.array(shared_keys)
    for s, row, n, start in _spans(spans):
        own, at = x[row : row + n], np.arange(start, start + n)
        q[row : row + n] = _unit_rms(own[:, : op.q_rank], op.epsilon) * q_gain
        latents[s, at % op.ring] = _out(op, _unit_rms(own[:, op.q_rank : op.q_rank + op.rank], op.epsilon) * c_gain)
        if keys is not None:
            rest = own[:, op.q_rank + op.rank : op.q_rank + op.rank + op.rot]
            keys[s, at % op.ring] = _out(op, rest if angles is None else _turn(rest, angles[at], op.turned))
    return (latents, _out(op, q)) if keys is None else (latents, keys, _out(op, q))


def latent_mha(op, q, latents, up, spans, *, shared_keys=None, angles=None, sink=None):
    H, D, V, R = op.heads, op.dim, op.vdim, op.rank
    y = np.zeros((op.rows, H, V), np.float32)
    q, up = np.asarray(q, np.float64).reshape(op.rows, H, D + op.rot), np.asarray(up, np.float64)
    for s, row, n, start in _spans(spans):
        first = max(0, start - op.window + 1)
        at = np.arange(first, start + n) % op.ring
        c = np.asarray(latents[s, at], np.float64)
        k, v = (c @ up[: H * D].T).reshape(-1, H, D), (c @ up[H * D :].T).reshape(-1, H, V)
        for i in range(n):
            lo, hi, query = max(0, start + i - op.window + 1) - first, start + i + 1 - first, q[row + i]
            if op.turned:
                query = np.concatenate([query[:, :D], _turn(query[:, D:], angles[start + i], op.turned)], axis=1)
            score = np.einsum("jhd,hd->hj", k[lo:hi], query[:, :D])
            if shared_keys is not None:
                score = score + query[:, D:] @ np.asarray(shared_keys[s, at[lo:hi]], np.float64).T
            score = score * op.scale
            top = score.max(1) if sink is None else np.maximum(score.max(1), sink)
            p = np.exp(score - top[:, None])
            total = p.sum(1) + (0 if sink is None else np.exp(sink - top))
            y[row + i] = np.einsum("hj,jhv->hv", p / total[:, None], v[lo:hi])
    return _out(op, y.reshape(op.rows, -1))


def turned_heads(op, x, bias, q_gain, k_gain, temp, spans, *, angles=None, first=None, share=None):
    H, G, D = op.heads, op.kv_heads, op.dim
    y = np.zeros((op.rows, op.stride), np.float32)
    for s, row, n, start in _spans(spans):
        own = np.asarray(x, np.float64)[row : row + n] + bias
        parts = []
        for heads, gain in ((own[:, : H * D].reshape(n, H, D), q_gain), (own[:, H * D : (H + G) * D].reshape(n, G, D), k_gain)):
            heads = _unit_rms(heads, op.epsilon) * gain
            if op.turned:
                heads = _turn(heads, np.asarray(angles)[start : start + n, None], op.turned)
            parts.append(heads)
        parts[0] = parts[0] * (op.scale * np.asarray(temp, np.float64))[:, None]
        v = own[:, (H + G) * D :]
        if op.mixed:
            share = float(np.reshape(share, -1)[0])
            v = (1 - share) * v + share * np.asarray(first, np.float64)[row : row + n, op.first_at : op.first_at + v.shape[1]]
        y[row : row + n] = np.concatenate([parts[0].reshape(n, -1), parts[1].reshape(n, -1), v], axis=1)
    return _out(op, y)


def talking_mha(op, x, talk, spans, keys, values):
    H, G, D, V, C = op.heads, op.kv_heads, op.dim, op.vdim, op.chunk
    keys, values, y = np.array(keys), np.array(values), np.zeros((op.rows, H, V), np.float32)
    group, talk = np.arange(H) // (H // G), np.asarray(talk, np.float64)
    for s, row, n, start in _spans(spans):
        own = np.asarray(x, np.float64)[row : row + n]
        q, k, v = own[:, : H * D].reshape(n, H, D), own[:, H * D : (H + G) * D].reshape(n, G, D), own[:, (H + G) * D :].reshape(n, G, V)
        for i in range(n):
            p = start + i
            keys[s, p % C], values[s, p % C] = k[i], v[i]
            seen = p % C + 1
            score = np.einsum("hd,jhd->hj", q[i], np.asarray(keys[s, :seen], np.float64)[:, group])
            w = np.exp(score - score.max(1, keepdims=True))
            w = talk @ (w / w.sum(1, keepdims=True))
            y[row + i] = np.einsum("hj,jhv->hv", w, np.asarray(values[s, :seen], np.float64)[:, group])
    return keys, values, _out(op, y.reshape(op.rows, -1))


def matrix_memory(op, x, i_bias, f_bias, state, tops, spans):
    H, D, V = op.heads, op.dim, op.vdim
    state, tops, o = np.array(state), np.array(tops), np.zeros((op.rows, op.width), np.float32)
    x = np.asarray(x, np.float64)
    q, k, v = x[:, : H * D].reshape(-1, H, D) * D**-0.5, x[:, H * D : 2 * H * D].reshape(-1, H, D), x[:, 2 * H * D : H * (2 * D + V)].reshape(-1, H, V)
    v = np.concatenate([v, np.ones((len(v), H, 1))], axis=2)
    i = op.cap * np.tanh((x[:, op.i_at : op.i_at + H] + i_bias) / op.cap)
    f = -np.logaddexp(0, -op.cap * np.tanh((x[:, op.f_at : op.f_at + H] + f_bias) / op.cap))
    for s, row, n, start in _spans(spans):
        S = np.asarray(state[s], np.float64) if start else np.zeros((H, D, V + 1))
        m = np.asarray(tops[s, (start - 1) % 2], np.float64) if start else np.zeros(H)
        for t in range(row, row + n):
            top = np.maximum(f[t] + m, i[t])
            S = np.exp(f[t] + m - top)[:, None, None] * S + np.exp(i[t] - top)[:, None, None] * k[t][:, :, None] * v[t][:, None]
            m = top
            read = np.einsum("hdv,hd->hv", S, q[t])
            o[t] = np.concatenate([read[:, :V].reshape(-1), read[:, V], m])
        state[s], tops[s, (start + n - 1) % 2] = S, m
    return state, tops, o


def memory_gate(op, o, gate, gain):
    H, D = op.heads, op.dim
    o = np.asarray(o, np.float64)
    under = np.maximum(np.abs(o[:, H * D : H * D + H]), np.exp(-o[:, H * D + H :])) + op.floor
    y = _unit_rms(o[:, : H * D].reshape(-1, H, D) / under[:, :, None], op.epsilon).reshape(op.rows, -1)
    return _out(op, y * gain * _sigmoid(np.asarray(gate, np.float64)[:, op.gate_at : op.gate_at + H * D]))


def activation(op, x):
    return _out(op, _act_of(op.kind, np.asarray(x, np.float64)))


def router(op, h, weight, *, bias=None, correction=None):
    z = np.asarray(h, np.float64) @ np.asarray(weight, np.float64).T + (0 if bias is None else bias)
    if op.scored:
        e = np.exp(z - z.max(1, keepdims=True))
        e = e / e.sum(1, keepdims=True)
        by = e + (0 if correction is None else np.asarray(correction, np.float64))
        ids = np.argsort(-by, axis=1, kind="stable")[:, : op.top]
        e = np.take_along_axis(e, ids, 1)
        return ids.astype(np.int32), (e / (e.sum(1, keepdims=True) + 1e-20)).astype(np.float32)
    ids = np.argsort(-z, axis=1, kind="stable")[:, : op.top]
    chosen = np.take_along_axis(z, ids, 1)
    e = np.exp(chosen - chosen.max(1, keepdims=True))
    return ids.astype(np.int32), (e / e.sum(1, keepdims=True)).astype(np.float32)


def experts(op, h, gate, up, down, ids, shares):
    h, y = np.asarray(h, np.float64), np.zeros((op.rows, op.cols))
    gate, up = (np.reshape(np.asarray(w, np.float64), (op.experts, op.ff, op.cols)) for w in (gate, up))
    down = np.reshape(np.asarray(down, np.float64), (op.experts, op.cols, op.ff))
    for r in range(op.rows):
        for e, share in zip(np.asarray(ids)[r], np.asarray(shares, np.float64)[r]):
            if e >= op.experts:   # an identity
                y[r] += share * h[r]
                continue
            a = _out(op, _act_of(op.activation, gate[e] @ h[r]) * (up[e] @ h[r]))
            y[r] += share * (down[e] @ np.asarray(a, np.float64))
    return _out(op, y)


def stream_sum(op, x, y, *, also=None):
    return np.asarray(np.asarray(x, np.float64) + y + (0 if also is None else np.asarray(also, np.float64)), np.float32)


def gated_columns(op, x, y):
    y = np.array(y)
    g, u = (np.asarray(x, np.float64)[:, at : at + op.cols] for at in (op.gate_at, op.gate_at + op.cols))
    if op.kind == "limited":
        g, u = np.minimum(g, op.limit), np.clip(u, -op.limit, op.limit)
        made = g * _sigmoid(1.702 * g) * (u + 1)
    else:
        made = _act_of(op.kind, g) * u
    y[:, op.at : op.at + op.cols] = made
    return _out(op, y)


def hgrn2(op, x, f_bias, lower, state, spans):
    H, D, V = op.heads, op.dim, op.vdim
    state, o = np.array(state), np.zeros((op.rows, H, V), np.float32)
    x, lower = np.asarray(x, np.float64), np.asarray(lower, np.float64)
    q = (x[:, : H * D] * _sigmoid(x[:, : H * D])).reshape(-1, H, D)
    f = (lower + (1 - lower) * _sigmoid(x[:, H * D : 2 * H * D] + f_bias)).reshape(-1, H, D)
    v = x[:, 2 * H * D : H * (2 * D + V)].reshape(-1, H, V)
    for s, row, n, start in _spans(spans):
        S = np.asarray(state[s], np.float64) if start else np.zeros((H, D, V))
        for t in range(row, row + n):
            S = f[t][:, :, None] * S + (1 - f[t])[:, :, None] * v[t][:, None, :]
            o[t] = np.einsum("hdv,hd->hv", S, q[t])
        state[s] = S
    return state, o.reshape(op.rows, -1)


def _turn_halves(x, angles, n):
    """Columns i and i + n / 2 of x (..., width) turned together by a row of cosines and sines side by side."""
    x = np.array(x)
    u, v, c, s = x[..., : n // 2].copy(), x[..., n // 2 : n].copy(), angles[..., 0:n:2], angles[..., 1:n:2]
    x[..., : n // 2], x[..., n // 2 : n] = u * c - v * s, v * c + u * s
    return x


def cached_heads(op, x, q_gain, k_gain, spans, keys, values, *, angles=None):
    H, G, D, V = op.heads, op.kv_heads, op.dim, op.vdim
    keys, values, q = np.array(keys), np.array(values), np.zeros((op.rows, op.inner), np.float32)
    for s, row, n, start in _spans(spans):
        own, at = np.asarray(x, np.float64)[row : row + n], np.arange(start, start + n)
        made = []
        for heads, gain in ((own[:, : H * D].reshape(n, H, D), q_gain), (own[:, H * D : (H + G) * D].reshape(n, G, D), k_gain)):
            heads = _unit_rms(heads, op.epsilon) * gain
            if op.turned:
                heads = _turn_halves(heads, np.asarray(angles, np.float64)[start : start + n, None], op.turned)
            made.append(heads)
        v = own[:, (H + G) * D : (H + G) * D + G * V].reshape(n, G, V)
        v = _unit_rms(v, op.epsilon) if op.value_norm else v
        q[row : row + n] = made[0].reshape(n, -1)
        keys[s][:, at], values[s][:, at] = _out(op, made[1]).swapaxes(0, 1), _out(op, v).swapaxes(0, 1)
    return keys, values, _out(op, q)


def global_mha(op, q, keys, values, spans):
    H, G, D, V = op.heads, op.kv_heads, op.dim, op.vdim
    y, group = np.zeros((op.rows, op.width), np.float32), np.arange(H) // (H // G)
    q = np.asarray(q, np.float64).reshape(op.rows, H, D)
    for s, row, n, start in _spans(spans):
        for i in range(n):
            k, v = (np.asarray(c[s][:, : start + i + 1], np.float64)[group] for c in (keys, values))
            score = np.einsum("hd,hjd->hj", q[row + i], k) * op.scale
            if op.cap:
                score = op.cap * np.tanh(score / op.cap)
            top = np.maximum(score.max(1, keepdims=True), 0)
            e = np.exp(score - top)
            p = e / (e.sum(1, keepdims=True) + (np.exp(-top) if op.sink else 0))
            y[row + i, op.at : op.at + H * V] = np.einsum("hj,hjv->hv", p, v).reshape(-1)
    return _out(op, y)


def span_tails(op, x, spans):
    y = np.zeros((op.slots, op.cols), np.float32)
    for s, row, n, _ in _spans(spans):
        y[s] = x[row + n - 1]
    return y


def softcap(op, x):
    y = np.asarray(x, np.float64)
    y = y * op.scale
    y = np.asarray(op.cap * np.tanh(y / op.cap) if op.cap else y, np.float32)
    rounded = np.zeros((op.rows, op.stride), np.float32)
    rounded[:, : op.cols] = round_bf16(y)
    return y, rounded


def _act_of(kind, z):
    return {"relu": lambda z: np.maximum(z, 0), "silu": lambda z: z / (1 + np.exp(-z)),
            "gelu_tanh": lambda z: 0.5 * z * (1 + np.tanh(np.sqrt(2 / np.pi) * (z + 0.044715 * z**3)))}[kind](z)


def gated_product(op, gate, up):
    return np.asarray(_act_of(op.activation, np.asarray(gate, np.float64)) * up, np.float32)


def linear_any(op, x, weight):
    return _out(op, np.asarray(x, np.float64) @ np.asarray(weight, np.float64).T)


def token_shift(op, h, mu, carry, spans):
    carry, mixed = np.array(carry), np.zeros((op.mixes, op.rows, op.cols), np.float32)
    for s, row, n, start in _spans(spans):
        own = np.asarray(h[row : row + n], np.float64)
        before = np.concatenate([carry[s, (start - 1) % 2][None] if start else np.zeros((1, op.cols)), own[:-1]])
        mixed[:, row : row + n] = own + (before - own) * np.asarray(mu, np.float64)[:, None]
        carry[s, (start + n - 1) % 2] = h[row + n - 1]
    return carry, _out(op, mixed)


def low_rank_decay(op, z, up, base):
    return np.asarray(-np.exp(np.tanh(np.asarray(z, np.float64)) @ np.asarray(up, np.float64).T + base), np.float32)


def time_mix(op, r, k, v, log_decay, u, state, spans):
    H, D = op.heads, op.dim
    state, o = np.array(state), np.zeros((op.rows, H, D), np.float32)
    r, k, v, w = (np.asarray(x, np.float64).reshape(op.rows, H, D) for x in (r, k, v, log_decay))
    for s, row, n, start in _spans(spans):
        S = np.asarray(state[s], np.float64) if start else np.zeros((H, D, D))
        for t in range(row, row + n):
            kv = k[t][:, :, None] * v[t][:, None, :]
            o[t] = np.einsum("hi,hij->hj", r[t], S + np.asarray(u, np.float64)[:, :, None] * kv)
            S = np.exp(w[t])[:, :, None] * S + kv
        state[s] = S
    return state, o.reshape(op.rows, -1)


def short_conv(op, x, weight, a_log, dt_bias, state, spans):
    G, H, D, V, C = op.kv_heads, op.heads, op.dim, op.vdim, op.channels
    state, y = np.array(state), np.zeros((op.rows, op.wide), np.float32)
    for s, row, n, start in _spans(spans):
        rows = np.asarray(x[row : row + n], np.float64)
        past = [state[s, p % op.taps] if p >= 0 else np.zeros(C) for p in range(start - op.taps + 1, start)]
        fed = np.concatenate([np.reshape(past, (-1, C)), rows[:, :C]])
        conv = sum(fed[i : i + n] * np.asarray(weight, np.float64)[:, i] for i in range(op.taps))
        conv = conv / (1 + np.exp(-conv))
        qk = conv[:, : 2 * G * D].reshape(n, 2, G, D)
        qk = qk / np.sqrt((qk * qk).sum(-1, keepdims=True) + 1e-6)
        qk[:, 0] *= D**-0.5
        decay = -np.exp(np.asarray(a_log, np.float64)) * np.logaddexp(0, rows[:, op.a_at : op.a_at + H] + dt_bias)
        beta = 1 / (1 + np.exp(-rows[:, op.b_at : op.b_at + H]))
        y[row : row + n] = np.concatenate([qk.reshape(n, -1), conv[:, 2 * G * D :], decay, beta], axis=1)
        for p in range(max(start, start + n - op.taps + 1), start + n):
            state[s, p % op.taps] = x[row + p - start][:C]
    return state, y


def delta_rule(op, x, state, spans):
    G, H, D, V, C = op.kv_heads, op.heads, op.dim, op.vdim, op.channels
    x, state, o = np.asarray(x, np.float64), np.array(state), np.zeros((op.rows, H, V), np.float32)
    group = np.arange(H) // (H // G)
    q, k = x[:, : G * D].reshape(-1, G, D)[:, group], x[:, G * D : 2 * G * D].reshape(-1, G, D)[:, group]
    v, g, beta = x[:, 2 * G * D : C].reshape(-1, H, V), np.exp(x[:, C : C + H]), x[:, C + H :]
    for s, row, n, start in _spans(spans):
        S = np.asarray(state[s], np.float64) if start else np.zeros((H, D, V))
        for t in range(row, row + n):
            S = g[t][:, None, None] * S
            u = beta[t][:, None] * (v[t] - np.einsum("hij,hi->hj", S, k[t]))
            S = S + k[t][:, :, None] * u[:, None, :]
            o[t] = np.einsum("hij,hi->hj", S, q[t])
        state[s] = S
    return state, o.reshape(op.rows, -1)


def head_gate(op, o, gain, *, gate=None):
    H, D = op.heads, op.dim
    z = None if gate is None else np.asarray(gate, np.float64)[:, op.gate_at : op.gate_at + H * D]
    gains = np.asarray(gain, np.float64) if op.gains == op.o_width else np.tile(np.asarray(gain, np.float64), H)
    y = np.zeros((op.rows, op.width), np.float32)
    y[:, op.at : op.at + H * D] = (_unit_rms(np.reshape(o, (-1, H, D)), op.epsilon).reshape(op.rows, -1) * gains
                                   * (1 if z is None else z / (1 + np.exp(-z))) * op.scale)
    return _out(op, y)


def window_mha(op, x, bias, spans, keys, values, y):
    H, G, D, V = op.heads, op.kv_heads, op.dim, op.vdim
    keys, values, y = np.array(keys), np.array(values), np.array(y)
    for s, row, n, start in _spans(spans):
        rows = np.asarray(x[row : row + n], np.float64)
        q, k, v = rows[:, : H * D].reshape(n, H, D), rows[:, H * D : (H + G) * D].reshape(n, G, D), \
            rows[:, (H + G) * D : (H + G) * D + G * V].reshape(n, G, V)
        first = max(0, start - op.window + 1)
        old = [p % op.ring for p in range(first, start)]
        allk = np.concatenate([np.asarray(keys[s][old], np.float64), k])
        allv = np.concatenate([np.asarray(values[s][old], np.float64), v])
        for i in range(n):
            lo = max(0, start + i - op.window + 1)
            a, b = lo - first, start + i + 1 - first
            for h in range(H):
                score = allk[a:b, h // (H // G)] @ q[i, h] * op.scale + bias[h][: b - a][::-1]
                p = np.exp(score - score.max())
                y[row + i, op.at + h * V : op.at + (h + 1) * V] = p / p.sum() @ allv[a:b, h // (H // G)] * op.out_scale
        for i in range(max(0, n - op.ring), n):
            keys[s, (start + i) % op.ring], values[s, (start + i) % op.ring] = k[i], v[i]
    return keys, values, _out(op, y)


def sample_slots(op, logits, draws, spans, token, tokens):
    spans, token, tokens = np.array(spans), np.array(token), np.array(tokens)
    for s, _, n, start in _spans(spans):
        at = start + n - 1
        temperature, top_k, n53 = ops.draw_words(np.asarray(draws)[s, at])
        token[s] = tokens[s, at] = ops.sample_ref(np.asarray(logits)[s, : op.vocab], temperature, top_k, n53, op.k_max)
        spans[s] = s, 1, at + 1, 0
    return spans, token, tokens


def install() -> None:
    from iron_amd.common.declare import REFERENCES

    REFERENCES.update(
        GEMM=gemm, GEMV=gemv, RMSNorm=rms_norm, SiLU=silu, ElementwiseMul=mul, ElementwiseAdd=add,
        RoPE=rope, MHA=mha, Copy=copy, Gather=gather, GatherWords=gather_words, Sample=sample, RowwiseAdd=rowwise_add, RowwiseMul=rowwise_mul,
        GELU=gelu, ReLU=relu, Sigmoid=sigmoid, Tanh=tanh, Clamp=clamp, AXPY=axpy, LayerNorm=layer_norm,
        Softmax=softmax, StreamEmbed=stream_embed, StreamNorm=stream_norm, StreamAdd=stream_add, SpanTails=span_tails,
        Softcap=softcap, GatedProduct=gated_product, LinearAny=linear_any, TokenShift=token_shift, LowRankDecay=low_rank_decay,
        TimeMix=time_mix, ShortConv=short_conv, DeltaRule=delta_rule, HeadGate=head_gate, WindowMHA=window_mha,
        SampleSlots=sample_slots, StreamGatedAdd=stream_gated_add, PolyNorm=poly_norm, MinGRU=min_gru, LatentRows=latent_rows,
        LatentMHA=latent_mha, DepthAverage=depth_average, StreamCast=stream_cast, TurnedHeads=turned_heads, TalkingMHA=talking_mha,
        MatrixMemory=matrix_memory, MemoryGate=memory_gate, Activation=activation, Router=router, Experts=experts,
        StreamSum=stream_sum, GatedColumns=gated_columns, Hgrn2=hgrn2, CachedHeads=cached_heads, GlobalMHA=global_mha,
        # The host's draw, for iron_amd.lm.generation.Sampler's checks.
        sample_ref=ops.sample_ref, sample_weights=ops.sample_weights,
    )
