"""Tilarax written out plainly in float64: one function per mechanism, a sequence at a time, every attention over
explicit pairs, the matrix memory token by token, every token's experts one by one.  TEST INFRASTRUCTURE: slow on
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


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-f64(z)))


def gelu_tanh(z):
    z = f64(z)
    return 0.5 * z * (1.0 + np.tanh(np.sqrt(2.0 / np.pi) * (z + 0.044715 * z**3)))


def silu(z):
    return f64(z) * sigmoid(z)


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


def chunk_weights(q, k, scale, chunk):
    """q (T, H, D), k (T, G, D), scale (H,): each query's softmax over itself and what is before it in its chunk,
    (H, T, T), zeros elsewhere."""
    T, H, _ = q.shape
    G = k.shape[1]
    p = np.zeros((H, T, T))
    for i in range(T):
        lo = i // chunk * chunk
        for h in range(H):
            s = k[lo : i + 1, h // (H // G)] @ q[i, h] * scale[h]
            e = np.exp(s - s.max())
            p[h, i, lo : i + 1] = e / e.sum()
    return p


def talked(p, talk):
    """The heads' weights mixed: row h of ``talk`` says what head h takes of each."""
    return np.einsum("hg,gij->hij", f64(talk), p)


def mlstm(q, k, v, i, f, state=None):
    """q, k (T, H, D), v (T, H, V), log gates i, f (T, H): a matrix of decayed outer products k v^T and the sum of
    their keys, both kept relative to the largest exponent so far (0 at first).  The readings (T, H, V), and the
    state behind them."""
    T, H, D = q.shape
    S, n, m = (np.zeros((H, D, v.shape[-1])), np.zeros((H, D)), np.zeros(H)) if state is None else state
    out = np.zeros(v.shape)
    for t in range(T):
        top = np.maximum(f[t] + m, i[t])
        keep, write = np.exp(f[t] + m - top), np.exp(i[t] - top)
        S = keep[:, None, None] * S + write[:, None, None] * k[t][:, :, None] * v[t][:, None, :]
        n = keep[:, None] * n + write[:, None] * k[t]
        m = top
        for h in range(H):
            out[t, h] = S[h].T @ q[t, h] / (max(abs(n[h] @ q[t, h]), np.exp(-m[h])) + 1e-6)
    return out, (S, n, m)


def log_gates(i, f, cap):
    """The capped input gate, and the logarithm of the capped forget gate's sigmoid."""
    return cap * np.tanh(f64(i) / cap), -np.logaddexp(0.0, -cap * np.tanh(f64(f) / cap))


def routed(z, top):
    """z (E,): the ``top`` largest logits' experts, and their softmax among themselves."""
    chosen = np.argsort(-f64(z), kind="stable")[:top]
    e = np.exp(z[chosen] - z[chosen].max())
    return chosen, e / e.sum()


class Plain:
    def __init__(self, config, weights):
        self.c = config
        self.w = {n: f64(a) for n, a in weights.items()}
        self.eps = config["norm"]["eps"]
        mixing = [i for i, s in enumerate(config["layers"]) if s["type"] == "attention" and s["mixer"].get("v_mix")]
        self.first_values = mixing[0] if mixing else None

    def norm(self, x, name):
        return over_rms(x, self.eps) * (1.0 + self.w[name])

    def attention(self, i, h, m):
        w, T, name = self.w, len(h), f"l{i}.mix."
        H, G, D, V = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
        q, k, v = ((h @ w[name + n].T + w[name + n + ".b"]).reshape(T, heads, width) for n, heads, width in (("q", H, D), ("k", G, D), ("v", G, V)))
        q, k = over_rms(q, self.eps) * w[name + "q.norm"], over_rms(k, self.eps) * w[name + "k.norm"]
        q, k = (turned(x, m["rot"]["base"], m["rot"]["dims"]) for x in (q, k))
        if m.get("v_mix"):
            if i == self.first_values:
                self.values = v
            else:
                share = w[name + "vmix"]
                v = (1 - share) * v + share * self.values
        p = talked(chunk_weights(q, k, m["scale"] * w[name + "temp"], m["mask"]["size"]), w[name + "talk"])
        out = np.stack([p[j] @ v[:, j // (H // G)] for j in range(H)], axis=1)
        return out.reshape(T, -1) @ w[name + "o"].T + w[name + "o.b"]

    def mlstm(self, i, h, m):
        w, T, name = self.w, len(h), f"l{i}.mix."
        H, D, V = m["heads"], m["dim"], m["vdim"]
        q, k, v = ((h @ w[name + n].T).reshape(T, H, width) for n, width in (("q", D), ("k", D), ("v", V)))
        gates = log_gates(h @ w[name + "i"].T + w[name + "i.b"], h @ w[name + "f"].T + w[name + "f.b"], m["gate_cap"])
        o, _ = mlstm(q * D**-0.5, k, v, *gates)
        y = over_rms(o, self.eps).reshape(T, -1) * w[name + "norm"] * sigmoid(h @ w[name + "g"].T)
        return y @ w[name + "o"].T

    def dense(self, name, h, spec):
        return gelu_tanh(h @ self.w[name + "up"].T) @ self.w[name + "down"].T

    def moe(self, name, h, spec):
        w, y = self.w, np.zeros_like(h)
        z = h @ w[name + "router"].T + w[name + "router.b"]
        for t in range(len(h)):
            for e, share in zip(*routed(z[t], spec["router"]["top"])):
                at = f"{name}e{e}."
                y[t] += share * ((silu(h[t] @ w[at + "gate"].T) * (h[t] @ w[at + "up"].T)) @ w[at + "down"].T)
        return y

    def layer(self, i, x):
        spec, name = self.c["layers"][i], f"l{i}."
        x = x + self.norm(getattr(self, spec["type"])(i, x, spec["mixer"]), name + "norm1")
        mlp = spec.get("mlp")
        if mlp is not None:
            x = x + self.norm(getattr(self, mlp["kind"])(name + "mlp.", x, mlp), name + "norm2")
        return x

    def __call__(self, tokens, trace=None):
        """Logits at every position, (T, vocab); ``trace`` collects the stream after every layer."""
        x = self.w["embed"][np.asarray(tokens)]
        results = [x]
        for i in range(len(self.c["layers"])):
            results.append(self.layer(i, x))
            x = sum(share * r for share, r in zip(self.w[f"l{i}.dwa"], results))
            if trace is not None:
                trace.append(x)
        return self.norm(x, "final.norm") @ self.w["embed"].T
