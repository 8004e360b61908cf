"""Running one operator's launch on arrays, beside its oracle; spans tables and random bf16 values."""

from __future__ import annotations

import numpy as np
import torch

from iron_amd.bf16 import bfloat16, from_torch, round_bf16, to_torch

F32 = np.float32


def device(array, dtype):
    return to_torch(array).cuda() if dtype is bfloat16 else torch.from_numpy(np.ascontiguousarray(array, dtype=dtype)).cuda()


def ran(op, workspace=None, **inputs):
    """The operator's launch on these arrays: what it wrote, by name."""
    tensors = {}
    for b in op.buffers:
        given = inputs.get(b.name)
        assert given is not None or not b.fills, b.name
        start = np.full(b.shape, 7.0, F32) if given is None else np.reshape(given, b.shape)
        tensors[b.name] = device(start, b.dtype)
    if workspace is not None:
        tensors["workspace"] = torch.full((op.workspace_words,), float("nan"), device="cuda") if workspace else None
    op.compile().launch(tensors, {})
    torch.cuda.synchronize()
    return {b.name: from_torch(tensors[b.name]).reshape(b.shape) for b in op.outputs}


# outputs a slot each, whatever the batch's rows
STATES = ("state", "carry", "keys", "values", "latents", "shared_keys", "tops", "planes")


def agrees(op, inputs, tol, rows=None, **kw):
    """The launch against the operator's oracle: every output (of rows ``rows`` where it has the batch's) within
    ``tol`` of the largest magnitude."""
    want = op._call_reference(inputs)
    got = ran(op, **kw, **inputs)
    for name, w in want.items():
        g, w = np.asarray(got[name], np.float64), np.asarray(w, np.float64).reshape(np.shape(got[name]))
        if rows is not None and len(w) == op.rows and name not in STATES:
            g, w = g[rows], w[rows]
        assert np.isfinite(g).all(), name
        assert np.abs(g - w).max() <= tol * max(np.abs(w).max(), 1e-3), (name, np.abs(g - w).max(), np.abs(w).max())
    return got


def tolerance(dtype):
    return 2e-5 if dtype is F32 else 1e-2


def table(*spans, slots=None):
    """A spans table: (slot, row0, rows, start) each."""
    out = np.zeros((slots or max(s[0] for s in spans) + 1, 4), np.int32)
    for slot, *rest in spans:
        out[slot, :3] = rest
    return out


def rows_of(spans):
    return np.concatenate([np.arange(r, r + n) for r, n, _, _ in np.asarray(spans) if n])


def bf(rng, *shape, scale=1.0):
    return round_bf16((rng.standard_normal(shape) * scale).astype(F32))
