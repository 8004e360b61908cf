"""Pudinex written out plainly in float64: one function per mechanism, a sequence at a time, every attention over
explicit pairs, the gated memory token by token, every token's experts one by one.  TEST INFRASTRUCTURE: slow on
purpose, and it shares nothing with the package but the names in a checkpoint.

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


def group_norm(x, gain, groups, eps):
    """Each of ``groups`` equal runs of a row over its own root mean square; the row times ``gain``."""
    x = f64(x)
    parts = x.reshape(*x.shape[:-1], groups, x.shape[-1] // groups)
    return over_rms(parts, eps).reshape(x.shape) * gain


def sigmoid(z):
    return 0.5 * (1.0 + np.tanh(0.5 * f64(z)))


def silu(z):
    return f64(z) * sigmoid(z)


def clamped_gate(g, u, limit):
    """min(g, limit) through a steep SiLU, times one more than u held within the limit."""
    g, u = np.minimum(f64(g), limit), np.clip(f64(u), -limit, limit)
    return g * sigmoid(1.702 * g) * (u + 1.0)


def frequencies(dims, base, scaling=None):
    """What position 1 turns each of ``dims / 2`` pairs by, and what cosines and sines are multiplied by: under YaRN the
    pairs that turn slowly over the original length are slowed by ``factor``, quick ones are left, between them a ramp."""
    i = np.arange(dims // 2)
    f = f64(base) ** (-2.0 * i / dims)
    if not scaling:
        return f, 1.0
    def place(turns):
        return dims * np.log(scaling["original"] / (2 * np.pi * turns)) / (2 * np.log(base))
    lo, hi = max(np.floor(place(scaling["fast"])), 0), min(np.ceil(place(scaling["slow"])), dims - 1)
    ramp = np.clip((i - lo) / max(hi - lo, 0.001), 0, 1)
    return f / scaling["factor"] * ramp + f * (1 - ramp), 0.1 * np.log(scaling["factor"]) + 1.0


def turned(x, dims, f, by=1.0, start=0):
    """x (T, ..., n): dimensions i and i + dims / 2 turned together by position times ``f[i]``, times ``by``."""
    x = np.array(f64(x))
    angle = (np.arange(start, start + len(x))[:, None] * f).reshape(len(x), *[1] * (x.ndim - 2), dims // 2)
    u, v = x[..., : dims // 2].copy(), x[..., dims // 2 : dims].copy()
    c, s = by * np.cos(angle), by * np.sin(angle)
    x[..., : dims // 2], x[..., dims // 2 : dims] = u * c - v * s, v * c + u * s
    return x


def sunk_weights(q, k, scale, softcap=None):
    """q (T, H, D), k (T, G, D): each query's weights of itself and everything before it under a denominator with one more
    in it, (H, T, T), zeros elsewhere."""
    T, H, _ = q.shape
    G = k.shape[1]
    p = np.zeros((H, T, T))
    for i in range(T):
        for h in range(H):
            s = k[: i + 1, h // (H // G)] @ q[i, h] * scale
            if softcap:
                s = softcap * np.tanh(s / softcap)
            top = max(s.max(), 0.0)
            e = np.exp(s - top)
            p[h, i, : i + 1] = e / (np.exp(-top) + e.sum())
    return p


def hgrn2(q, v, f, state=None):
    """q, f (T, H, D), v (T, H, V): a matrix a head whose rows fade by f and are written 1 - f of v, read by q behind that.
    The readings (T, H, V), and the state behind them."""
    S = np.zeros((q.shape[1], q.shape[2], v.shape[2])) if state is None else state
    out = np.zeros(v.shape)
    for t in range(len(q)):
        S = f[t][:, :, None] * S + (1.0 - f[t])[:, :, None] * v[t][:, None, :]
        out[t] = np.einsum("hdv,hd->hv", S, q[t])
    return out, S


def routed(z, correction, top):
    """z (E,): the experts of the ``top`` largest softmax scores plus corrections, and their shares of the scores without."""
    s = np.exp(f64(z) - np.max(z))
    s = s / s.sum()
    chosen = np.argsort(-(s + correction), kind="stable")[:top]
    return chosen, s[chosen] / (s[chosen].sum() + 1e-20)


class Plain:
    def __init__(self, config, weights):
        self.c = config
        self.w = {n: f64(a) for n, a in weights.items()}
        self.eps, self.groups = config["norm"]["eps"], config["norm"]["groups"]

    def norm(self, x, name):
        return group_norm(x, self.w[name], self.groups, self.eps)

    def attention(self, name, h, m):
        w, T = self.w, len(h)
        H, G, D, V = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
        q, k, v = ((h @ w[name + n].T).reshape(T, heads, width) for n, heads, width in (("q", H, D), ("k", G, D), ("v", G, V)))
        q, k = over_rms(q, self.eps) * w[name + "q.norm"], over_rms(k, self.eps) * w[name + "k.norm"]
        f, by = frequencies(m["rot"]["dims"], m["rot"]["base"], m["rot"].get("scaling"))
        q, k = (turned(x, m["rot"]["dims"], f, by) for x in (q, k))
        v = over_rms(v, self.eps)
        p = sunk_weights(q, k, m["scale"], m.get("softcap"))
        out = np.stack([p[j] @ v[:, j // (H // G)] for j in range(H)], axis=1)
        return out.reshape(T, -1) @ w[name + "o"].T

    def hgrn2(self, name, h, m):
        w, T = self.w, len(h)
        H, D, V = m["heads"], m["dim"], m["vdim"]
        q, v = silu(h @ w[name + "q"].T).reshape(T, H, D), (h @ w[name + "v"].T).reshape(T, H, V)
        low = w[name + "lower"]
        f = (low + (1 - low) * sigmoid(h @ w[name + "f"].T + w[name + "f.b"])).reshape(T, H, D)
        o, _ = hgrn2(q, v, f)
        return (over_rms(o, self.eps) * w[name + "norm"]).reshape(T, -1) @ w[name + "o"].T

    def dense(self, name, h, spec):
        w = self.w
        return clamped_gate(h @ w[name + "gate"].T, h @ w[name + "up"].T, spec["limit"]) @ w[name + "down"].T

    def expert(self, name, h):
        w = self.w
        return (silu(h @ w[name + "gate"].T) * (h @ w[name + "up"].T)) @ w[name + "down"].T

    def moe(self, name, h, spec):
        y = self.expert(name + "shared.", h) if spec.get("shared") else np.zeros_like(h)
        z, real = h @ self.w[name + "router"].T, spec["router"]["experts"]
        for t in range(len(h)):
            for e, share in zip(*routed(z[t], self.w[name + "correction"], spec["router"]["top"])):
                y[t] += share * (self.expert(f"{name}e{e}.", h[t]) if e < real else h[t])
        return y

    def layer(self, i, x):
        spec, name = self.c["layers"][i], f"l{i}."
        h = self.norm(x, name + "norm1")
        y = getattr(self, spec["type"])(name + "mix.", h, spec["mixer"])
        mlp = spec.get("mlp")
        return x + (y if mlp is None else y + getattr(self, mlp["kind"])(name + "mlp.", h, mlp))

    def __call__(self, tokens, trace=None):
        """Logits at every position, (T, vocab); ``trace`` collects the stream after every layer."""
        x = self.w["embed"][np.asarray(tokens)] * self.c["embedding"]["scale"]
        for i in range(len(self.c["layers"])):
            x = self.layer(i, x)
            if trace is not None:
                trace.append(x)
        return self.norm(x, "final.norm") @ self.w["head"].T
