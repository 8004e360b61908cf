"""Pufuzen written out plainly in float64: one function per mechanism, a sequence at a time, every
attention over explicit pairs of expanded keys and values, the recurrence token by token.  TEST
INFRASTRUCTURE: slow on purpose, and it shares nothing with the package but the names in a checkpoint.

``weights`` maps a checkpoint's tensor names to arrays, ``config`` is the parsed ``config.json``.
"""

from __future__ import annotations

import numpy as np


def f64(x):
    return np.asarray(x, dtype=np.float64)


def over_rms(x, eps):
    """x over its root mean square along the last axis."""
    x = f64(x)
    return x / np.sqrt((x * x).mean(axis=-1, keepdims=True) + eps)


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-f64(z)))


def min_gru(z, u, state=None):
    """z, u (T, W): a state that moves by the share sigmoid(z) towards u + 1/2, or sigmoid(u) below zero.
    The states, (T, W)."""
    z, u = sigmoid(z), f64(u)
    candidate = np.where(u >= 0, u + 0.5, sigmoid(u))
    s = np.zeros(z.shape[1]) if state is None else f64(state)
    out = np.empty_like(z)
    for t in range(len(z)):
        s = (1 - z[t]) * s + z[t] * candidate[t]
        out[t] = s
    return out


def turned(x, base, dims, start=0):
    """x (T, ..., n): neighbouring pairs of the first ``dims`` values turned by position times
    ``base ** (-2 i / dims)``."""
    x = np.array(f64(x))
    place = np.arange(start, start + len(x))
    angle = place[:, None] * f64(base) ** (-2.0 * np.arange(dims // 2) / dims)
    angle = angle.reshape(len(x), *[1] * (x.ndim - 2), dims // 2)
    u, v = x[..., 0:dims:2].copy(), x[..., 1:dims:2].copy()
    x[..., 0:dims:2], x[..., 1:dims:2] = u * np.cos(angle) - v * np.sin(angle), v * np.cos(angle) + u * np.sin(angle)
    return x


def attention(q, k, v, *, scale, window=None, sink=None):
    """q, k (T, H, D), v (T, H, V): each query over itself and what is before it (``window``: the window - 1
    tokens before it), ``sink`` (H,) one more term of each head's denominator."""
    T, H, _ = q.shape
    out = np.zeros((T, H, v.shape[-1]))
    for i in range(T):
        lo = 0 if window is None else max(0, i - window + 1)
        for h in range(H):
            s = k[lo : i + 1, h] @ q[i, h] * scale
            top = s.max() if sink is None else max(s.max(), sink[h])
            p = np.exp(s - top)
            out[i, h] = p @ v[lo : i + 1, h] / (p.sum() + (0.0 if sink is None else np.exp(sink[h] - top)))
    return out


def poly_norm(z, coefficients, eps):
    a, b, c, e = f64(coefficients)
    z = f64(z)
    return a * over_rms(z, eps) + b * over_rms(z**2, eps) + c * over_rms(z**3, eps) + e


class Plain:
    def __init__(self, config, weights):
        self.c = config
        self.w = {n: f64(a) for n, a in weights.items()}
        self.eps = config["norm"]["eps"]

    def norm(self, x, name):
        return over_rms(x, self.eps) * self.w[name]

    def mingru(self, name, h, m):
        w = self.w
        s = min_gru(h @ w[name + "z"].T + w[name + "z.b"], h @ w[name + "x"].T + w[name + "x.b"])
        gate = h @ w[name + "g"].T
        return (s * gate * sigmoid(gate)) @ w[name + "o"].T

    def latent(self, name, h, m, rot_dim=0):
        w, (T, _) = self.w, h.shape
        H, D, V, R = m["heads"], m["dim"], m["vdim"], m["kv_rank"]
        q = (self.norm(h @ w[name + "dq"].T, name + "dq.norm") @ w[name + "uq"].T).reshape(T, H, D + rot_dim)
        down = h @ w[name + "dkv"].T
        c = self.norm(down[:, :R], name + "dkv.norm")
        k, v = (c @ w[name + "uk"].T).reshape(T, H, D), (c @ w[name + "uv"].T).reshape(T, H, V)
        if rot_dim:
            turn = dict(base=m["rot"]["base"], dims=m["rot"]["dims"])
            shared = turned(down[:, R:], **turn)
            q = np.concatenate([q[..., :D], turned(q[..., D:], **turn)], axis=-1)
            k = np.concatenate([k, np.repeat(shared[:, None], H, axis=1)], axis=-1)
        out = attention(q, k, v, scale=m["scale"], window=m["mask"]["size"] if "mask" in m else None,
                        sink=w.get(name + "sink"))
        return out.reshape(T, -1) @ w[name + "o"].T

    def latent_attention(self, name, h, m):
        return self.latent(name, h, m)

    def latent_attention_2(self, name, h, m):
        return self.latent(name, h, m, m["rot_dim"])

    def mlp(self, name, h):
        w = self.w
        z = h @ w[name + "up"].T + w[name + "up.b"]
        return poly_norm(z, w[name + "act"], self.eps) @ w[name + "down"].T + w[name + "down.b"]

    def gate(self, name, h):
        return sigmoid(h @ self.w[name].T + self.w[name + ".b"])

    def layer(self, i, x):
        spec, name = self.c["layers"][i], f"l{i}."
        h = self.norm(x, name + "norm1")
        x = x + self.gate(name + "rg1", h) * getattr(self, spec["type"])(name + "mix.", h, spec["mixer"])
        if spec["mlp"] is not None:
            h = self.norm(x, name + "norm2")
            x = x + self.gate(name + "rg2", h) * self.mlp(name + "mlp.", h)
        return x

    def __call__(self, tokens, trace=None):
        """Logits at every position, (T, vocab); ``trace`` collects the stream after every layer."""
        x = self.w["embed"][np.asarray(tokens)]
        for i in range(len(self.c["layers"])):
            x = self.layer(i, x)
            if trace is not None:
                trace.append(x)
        return self.norm(x, "final.norm") @ self.w["head"].T * self.c["logit_scale"]
