"""Pegilix written out plainly in float64: one function per mechanism, a sequence at a time, every
attention over explicit pairs and every recurrence token by token.  TEST INFRASTRUCTURE: slow on
purpose, and it shares nothing with the package but the names in a checkpoint.

``weights`` maps a checkpoint's tensor names to arrays, ``config`` is the parsed ``config.json``.
"""

from __future__ import annotations

import math

import numpy as np


def f64(x):
    return np.asarray(x, dtype=np.float64)


def rms(x, eps):
    """x over its root mean square along the last axis."""
    x = f64(x)
    return x / np.sqrt((x * x).mean(axis=-1, keepdims=True) + eps)


def rms_norm(x, gain, eps):
    return rms(x, eps) * f64(gain)


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-f64(z)))


def silu(z):
    return f64(z) * sigmoid(z)


def softplus(z):
    return np.logaddexp(0.0, f64(z))


def distance_bucket(n: int, rows: int, bias_max: float) -> int:
    """The row of a distance-bias table with ``rows`` rows that ``n`` tokens back reads."""
    exact = rows // 2
    if n < rows / 2:
        return n
    share = math.log(n / (rows / 2)) / math.log(bias_max / (rows / 2))
    return min(rows - 1, int(exact + math.floor(share * (rows - rows / 2))))


def window_attention(q, k, v, bias, *, window, bias_max, scale):
    """q (T, H, dim), k (T, G, dim), v (T, G, vdim), bias (B, H): each query over itself and the
    ``window - 1`` tokens before it."""
    T, H, _ = q.shape
    G = k.shape[1]
    out = np.zeros((T, H, v.shape[-1]))
    for i in range(T):
        lo = max(0, i - window + 1)
        rows = [distance_bucket(i - j, bias.shape[0], bias_max) for j in range(lo, i + 1)]
        for h in range(H):
            g = h // (H // G)
            s = k[lo : i + 1, g] @ q[i, h] * scale + bias[rows, h]
            p = np.exp(s - s.max())
            out[i, h] = (p / p.sum()) @ v[lo : i + 1, g]
    return out


def shifted(h):
    """The previous token's row (zeros before the first)."""
    return np.concatenate([np.zeros_like(h[:1]), h[:-1]])


def time_mix(r, k, v, w, u):
    """The bonus-then-decay recurrence.  r, k, v, w (T, H, D), u (H, D): (T, H, D)."""
    T, H, D = r.shape
    state = np.zeros((H, D, D))
    out = np.zeros((T, H, D))
    for t in range(T):
        kv = k[t][:, :, None] * v[t][:, None, :]
        out[t] = np.einsum("hij,hi->hj", state + u[:, :, None] * kv, r[t])
        state = w[t][:, :, None] * state + kv
    return out


def causal_conv(x, taps):
    """x (T, C), taps (C, n), the last tap the current token's."""
    n = taps.shape[1]
    padded = np.concatenate([np.zeros((n - 1, x.shape[1])), x])
    return sum(padded[i : i + len(x)] * taps[:, i] for i in range(n))


def unit(x):
    return x / np.sqrt((x * x).sum(axis=-1, keepdims=True) + 1e-6)


def delta_rule(q, k, v, g, beta):
    """The gated delta rule.  q, k (T, H, D), v (T, H, V), g, beta (T, H): (T, H, V)."""
    T, H, D = q.shape
    state = np.zeros((H, D, v.shape[-1]))
    out = np.zeros(v.shape)
    for t in range(T):
        state = g[t][:, None, None] * state
        read = np.einsum("hij,hi->hj", state, k[t])
        state = state + k[t][:, :, None] * (beta[t][:, None] * (v[t] - read))[:, None, :]
        out[t] = np.einsum("hij,hi->hj", state, q[t])
    return out


class Plain:
    def __init__(self, config, weights):
        self.c = config
        self.w = {n: f64(a) for n, a in weights.items()}
        self.eps = config["norm"]["eps"]

    def left(self, name, h, m):
        w, (T, _) = self.w, h.shape
        H, G = m["heads"], m["kv_heads"]
        q = (h @ w[name + "q"].T).reshape(T, H, m["dim"])
        k = (h @ w[name + "k"].T).reshape(T, G, m["dim"])
        v = (h @ w[name + "v"].T).reshape(T, G, m["vdim"])
        out = window_attention(q, k, v, w[name + "rel"], window=m["mask"]["size"], bias_max=m["bias_max"],
                               scale=m["scale"])
        return out.reshape(T, -1) @ w[name + "o"].T

    def right(self, name, h, m):
        w, (T, _) = self.w, h.shape
        H, D = m["heads"], m["dim"]
        before = shifted(h)
        mix = {s: h + (before - h) * w[f"{name}mu.{s}"] for s in "rkvgw"}
        r, k, v = ((mix[s] @ w[name + s].T).reshape(T, H, D) for s in "rkv")
        gate = silu(mix["g"] @ w[name + "g"].T)
        decay = np.exp(-np.exp(np.tanh(mix["w"] @ w[name + "w1"].T) @ w[name + "w2"].T + w[name + "w0"]))
        o = rms(time_mix(r, k, v, decay.reshape(T, H, D), w[name + "u"]), self.eps)
        return (o.reshape(T, -1) * w[name + "norm"] * gate) @ w[name + "o"].T

    def parallel(self, name, h, m):
        return (m["left_scale"] * self.left(name + "left.", h, m["left"])
                + m["right_scale"] * self.right(name + "right.", h, m["right"]))

    def delta(self, name, h, m):
        w, (T, _) = self.w, h.shape
        H, G, D, V = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
        q, k, v = (silu(causal_conv(h @ w[name + s].T, w[f"{name}{s}.conv"])) for s in "qkv")
        group = np.arange(H) // (H // G)
        q = unit(q.reshape(T, G, D))[:, group] * D**-0.5
        k = unit(k.reshape(T, G, D))[:, group]
        beta = sigmoid(h @ w[name + "b"].T)
        g = np.exp(-np.exp(w[name + "A_log"]) * softplus(h @ w[name + "a"].T + w[name + "dt_bias"]))
        o = rms(delta_rule(q, k, v.reshape(T, H, V), g, beta), self.eps) * w[name + "norm"]
        return (o.reshape(T, -1) * silu(h @ w[name + "g"].T)) @ w[name + "o"].T

    def mlp(self, name, h):
        w = self.w
        return (np.maximum(h @ w[name + "gate"].T, 0) * (h @ w[name + "up"].T)) @ w[name + "down"].T

    def layer(self, i, x):
        w, spec, name = self.w, self.c["layers"][i], f"l{i}."
        mixed = getattr(self, spec["type"])(name + "mix.", rms_norm(x, w[name + "norm1"], self.eps), spec["mixer"])
        x = x + rms_norm(mixed, w[name + "norm1b"], self.eps)
        if spec["mlp"] is not None:
            fed = self.mlp(name + "mlp.", rms_norm(x, w[name + "norm2"], self.eps))
            x = x + rms_norm(fed, w[name + "norm2b"], self.eps)
        return x

    def order(self):
        layers, loop = list(range(len(self.c["layers"]))), self.c.get("loop")
        if loop is None:
            return layers
        a, b = loop["start"], loop["stop"]
        return layers[:a] + layers[a:b] * loop["times"] + layers[b:]

    def __call__(self, tokens, trace=None):
        """Logits at every position, (T, vocab); ``trace`` collects the stream after every layer run."""
        x = self.w["embed"][np.asarray(tokens)]
        for i in self.order():
            x = self.layer(i, x)
            if trace is not None:
                trace.append(x)
        logits = rms_norm(x, self.w["final.norm"], self.eps) @ self.w["head"].T
        cap = self.c.get("logit_softcap")
        return logits if cap is None else cap * np.tanh(logits / cap)
