"""Pudinex's mechanisms and models on the GPU against the oracle and the plain implementation: each kernel
alone, prompts, portions, batches, slots used again, far keys, long decoding, generation."""

import json
import subprocess
import sys
from pathlib import Path

import numpy as np
import pytest
import torch

import oracle
from iron_amd import kernels as K
from iron_amd.applications import Pudinex, PudinexConfig
from iron_amd.bf16 import bfloat16, from_torch, round_bf16
from iron_amd.lm import Sampler, rope_angles, write_safetensors
from iron_amd.lm.batched import Entry
from iron_amd.operators.experts import Experts, Router
from iron_amd.operators.mha_global import CachedHeads, GlobalMHA
from iron_amd.operators.recurrent import HeadGate, Hgrn2
from iron_amd.operators.stream import GatedColumns, StreamEmbed, StreamNorm, StreamSum
from tests.operator_support import agrees, bf, device, ran, rows_of, table
from tests.pudinex_plain import hgrn2, over_rms, sigmoid, sunk_weights
from tests.pudinex_support import MODELS, built, far_off, weights_of

pytestmark = pytest.mark.gpu
oracle.install()
F32, BF16 = np.float32, bfloat16
BOTH = pytest.mark.parametrize("dtype", [F32, BF16], ids=["f32", "bf16"])
ids_of = lambda p: "x".join(map(str, p))  # noqa: E731


# ---------------------------------------------------------------- the stream


@BOTH
@pytest.mark.parametrize("rows,cols,groups", [(5, 128, 4), (3, 60, 5), (2, 2048, 1), (3, 4096, 2), (1, 1303, 1), (7, 96, 3), (1, 12288, 3), (1, 16384, 256)])
def test_sums_join_the_stream_and_it_is_normed_in_groups(cuda, dtype, rows, cols, groups):
    rng = np.random.default_rng(cols)
    x, y, also, gain = rng.standard_normal((rows, cols)).astype(F32) * 3, bf(rng, rows, cols), bf(rng, rows, cols), bf(rng, cols)
    x[:, : cols // groups] *= 50.0   # a group by itself
    kw = dict(rows=rows, cols=cols)
    limit = 3e-6 if dtype is F32 else 5e-3
    agrees(StreamNorm(epsilon=1e-3, groups=groups, unit=1.0, dtype=dtype, **kw), dict(x=x, weight=gain), limit)
    agrees(StreamSum(dtype=dtype, **kw), dict(x=x, y=y), 2e-6)
    added = agrees(StreamSum(two=True, dtype=dtype, **kw), dict(x=x, y=y, also=also), 2e-6)["x"]
    normed = ran(StreamNorm(epsilon=1e-3, groups=groups, dtype=dtype, **kw), x=added, weight=gain)["y"]
    # both in one launch: bit for bit where the norm alone is made the same way
    xd, hd = device(x, F32), torch.empty((rows, cols), dtype=torch.bfloat16 if dtype is BF16 else torch.float32, device="cuda")
    K.stream_groups(xd, y=device(y, dtype), y2=device(also, dtype), h=hd, gain=device(gain, BF16), groups=groups, eps=1e-3, **kw)
    torch.cuda.synchronize()
    assert np.array_equal(from_torch(xd), added)
    assert np.abs(from_torch(hd) - normed).max() <= (1e-6 if dtype is F32 else 8e-3) * np.abs(normed).max()
    if groups > 1:
        assert np.array_equal(from_torch(hd), normed)


@pytest.mark.parametrize("cols", [64, 61])
def test_embedding_rows_are_scaled(cuda, cols):
    rng = np.random.default_rng(cols)
    t, ids = bf(rng, 30, cols), rng.integers(0, 30, 9)
    assert np.array_equal(ran(StreamEmbed(rows=9, table_rows=30, cols=cols, scale=12.5), table=t, ids=ids)["x"], t[ids] * F32(12.5))


@BOTH
@pytest.mark.parametrize("kind", ["limited", "silu", "gelu_tanh", "relu"])
@pytest.mark.parametrize("cols,gate_at,at", [(64, 24, 8), (37, 5, 3), (2048, 0, 0)])
def test_gated_columns(cuda, dtype, kind, cols, gate_at, at):
    rng = np.random.default_rng(cols)
    op = GatedColumns(rows=6, cols=cols, stride=2 * cols + 32, width=cols + 16, gate_at=gate_at, at=at, kind=kind, limit=0.75, dtype=dtype)
    x, y = bf(rng, 6, 2 * cols + 32, scale=2), bf(rng, 6, cols + 16)
    got = agrees(op, dict(x=x, y=y), 3e-6 if dtype is F32 else 5e-3)["y"]
    assert np.array_equal(got[:, :at], y[:, :at]) and np.array_equal(got[:, at + cols :], y[:, at + cols :])


@pytest.mark.parametrize("K_,M,groups,logits", [(128, 96, 4, 0), (2048, 300, 4, 18), (4096, 64, 2, 1), (192, 8200, 3, 7), (8, 5, 1, 3), (16384, 10, 8, 0),
                                                (1024, 40, 128, 66)])
def test_a_normed_row_s_product_and_logits(cuda, K_, M, groups, logits):
    rng = np.random.default_rng(K_)
    x, gain, W = rng.standard_normal((1, K_)).astype(F32) * 2, bf(rng, K_), bf(rng, M, K_, scale=K_**-0.5)
    router = bf(rng, max(logits, 1), K_, scale=K_**-0.5)
    x[0, : K_ // groups] *= 30.0
    h = ran(StreamNorm(rows=1, cols=K_, groups=groups, epsilon=1e-4), x=x, weight=gain)["y"]
    y, made = torch.zeros(M, dtype=torch.bfloat16, device="cuda"), torch.zeros(K_, dtype=torch.bfloat16, device="cuda")
    z = torch.zeros(max(logits, 1), device="cuda")
    more = dict(router=device(router, BF16), z=z, logits=logits) if logits else {}
    K.norm_product(device(x, F32).reshape(-1), device(gain, BF16), device(W, BF16), y, M=M, K=K_, groups=groups, eps=1e-4, h=made, **more)
    torch.cuda.synchronize()
    assert np.abs(from_torch(made) - h[0]).max() <= 8e-3 * np.abs(h).max()   # (the sums in another order)
    want = W.astype(np.float64) @ from_torch(made)
    assert np.abs(from_torch(y) - want).max() <= 6e-3 * np.abs(want).max()
    if logits:
        want = router.astype(np.float64) @ from_torch(made)
        assert np.abs(from_torch(z) - want).max() <= 2e-6 * max(np.abs(want).max(), 1)


@pytest.mark.parametrize("two", [False, True])
@pytest.mark.parametrize("K_,M", [(384, 100), (2048, 2049), (10240, 33), (16384, 7), (18432, 50), (32768, 3)])
def test_a_product_joins_the_stream(cuda, K_, M, two):
    rng = np.random.default_rng(M)
    x, W, stream, also = bf(rng, K_), bf(rng, M, K_, scale=K_**-0.5), rng.standard_normal(M).astype(F32), bf(rng, M)
    at = device(stream, F32)
    K.product_sum(device(x, BF16), device(W, BF16), at, M=M, K=K_, also=device(also, BF16) if two else None)
    torch.cuda.synchronize()
    product = W.astype(np.float64) @ x
    got = from_torch(at) - stream.astype(np.float64) - (also if two else 0)
    assert np.abs(got - product).max() <= 5e-3 * np.abs(product).max()


# ---------------------------------------------------------------- the rows of attention


@BOTH
@pytest.mark.parametrize("H,G,D,V,turned", [(6, 2, 32, 48, 16), (3, 1, 11, 7, 6), (2, 2, 128, 64, 128), (6, 2, 88, 200, 0), (8, 4, 8, 16, 2), (2, 1, 40, 24, 24),
                                            (32, 8, 256, 128, 64)])
def test_heads_into_their_caches(cuda, dtype, H, G, D, V, turned):
    rng = np.random.default_rng(D)
    stride, context = (H + G) * D + G * V + 16, 70
    spans = table((0, 30, 40, 60 - 40), (1, 3, 1, 7), (3, 4, 26, 0), slots=4)
    given = dict(x=bf(rng, 72, stride), q_gain=bf(rng, D), k_gain=bf(rng, D), spans=spans, keys=bf(rng, 4, G, context, D), values=bf(rng, 4, G, context, V))
    given |= {"angles": rope_angles(turned, 128, 400.0) * F32(1.3)} if turned else {}
    for value_norm in (True, False):
        op = CachedHeads(slots=4, rows=72, stride=stride, heads=H, kv_heads=G, dim=D, vdim=V, context=context, turned=turned,
                         angle_rows=128 if turned else 1, value_norm=value_norm, epsilon=1e-3, dtype=dtype)
        agrees(op, given, 4e-6 if dtype is F32 else 5e-3, rows_of(spans))


@pytest.mark.parametrize("H,G,D,V,turned,cols,logits", [(6, 2, 32, 48, 16, 56, 0), (8, 1, 64, 64, 32, 0, 9), (4, 4, 128, 256, 128, 300, 66)])
def test_a_step_s_heads_with_columns_and_a_choice_beside(cuda, H, G, D, V, turned, cols, logits):
    rng = np.random.default_rng(V)
    slots, context, own = (1 if logits else 3), 40, (H + G) * D + G * V
    stride, width = own + 2 * cols, H * V + cols
    spans = table(*[(i, i, 1, 7 + 9 * i) for i in range(slots)], slots=slots)
    x, q_gain, k_gain, angles = bf(rng, slots, stride), bf(rng, D), bf(rng, D), rope_angles(turned, 64, 400.0)
    keys, values = bf(rng, slots, G, context, D), bf(rng, slots, G, context, V)
    op = CachedHeads(slots=slots, rows=slots, stride=stride, heads=H, kv_heads=G, dim=D, vdim=V, context=context, turned=turned, angle_rows=64,
                     value_norm=True, epsilon=1e-3)
    want = ran(op, x=x, q_gain=q_gain, k_gain=k_gain, spans=spans, keys=keys, values=values, angles=angles)
    t = {n: device(v, BF16) for n, v in dict(x=x, q_gain=q_gain, k_gain=k_gain, keys=keys, values=values, q=np.zeros((slots, H * D)),
                                             out=np.full((slots, width), 7.0)).items()}
    t |= dict(spans=device(spans, np.int32), angles=device(angles, F32))
    kw = {n: getattr(op, n) for n in ("slots", "rows", "stride", "heads", "kv_heads", "dim", "vdim", "context", "turned", "angle_rows", "value_norm")}
    if cols:
        kw |= dict(out_stride=width, cols=cols, gate_at=own, gated_at=H * V, kind="limited", limit=0.6)
    choice = {}
    if logits:
        z, correction = rng.standard_normal(logits).astype(F32), bf(rng, logits, scale=0.2)
        choice = dict(z=device(z, F32), correction=device(correction, BF16), logits=logits, top=3, ids=device(np.zeros(3), np.int32),
                      shares=device(np.zeros(3), F32))
    K.decode_heads_global(**t, **kw, eps=1e-3, **choice)
    torch.cuda.synchronize()
    for name in ("q", "keys", "values"):
        assert np.array_equal(from_torch(t[name]).reshape(want[name].shape), want[name]), name
    out = from_torch(t["out"])
    assert (out[:, : H * V] == 7).all()
    if cols:
        assert np.array_equal(out, ran(GatedColumns(rows=slots, cols=cols, stride=stride, width=width, gate_at=own, at=H * V, kind="limited", limit=0.6),
                                       x=x, y=np.full((slots, width), 7.0))["y"])
    if logits:
        check_choice(z, correction, 3, choice["ids"].cpu().numpy(), from_torch(choice["shares"]))


def check_choice(z, correction, top, ids, shares):
    s = np.exp(z.astype(np.float64) - z.max())
    s /= s.sum()
    want = np.argsort(-(s + correction), kind="stable")[:top]
    assert np.array_equal(ids, want) and np.abs(shares - s[want] / s[want].sum()).max() < 1e-5


# ---------------------------------------------------------------- attention over everything before

# heads, key/value heads, dim, vdim
SIZES = [(6, 2, 32, 48), (4, 4, 64, 24), (3, 1, 11, 7), (1, 1, 12, 7), (16, 4, 64, 64), (18, 1, 32, 64), (2, 2, 40, 48), (8, 2, 128, 128), (34, 2, 88, 104),
         (4, 2, 256, 256), (4, 1, 64, 200), (2, 2, 136, 16), (8, 8, 8, 8), (32, 8, 64, 64)]
CAPS = pytest.mark.parametrize("cap", [0.0, 6.0, 55.0], ids=["plain", "fixed", "capped"])   # (the last: beyond what bounds exponentials)


def global_case(rng, H, G, D, V, T, quiet=False):
    """A sequence's rows in which chosen queries meet a key that stands out far back -- the first position's, one just ahead of a
    tile's edge, one just behind -- or, ``quiet``, no key that does and scores far below the sink's."""
    q, k, v = bf(rng, T, H, D, scale=0.5 if quiet else 0.25), bf(rng, T, G, D, scale=1.0 if quiet else 0.4), bf(rng, T, G, V)
    if quiet:
        k = -np.abs(k)
        q = np.abs(q)
    for i in range(0 if quiet else T):
        if i > 2 and i % 5 == 0:
            h = i % H
            far = (0, max(0, i // 64 * 64 - 1), i // 64 * 64, i // 3)[i // 5 % 4]
            k[far, h // (H // G)] = 14 * q[i, h] / max(float(np.linalg.norm(q[i, h])), 1e-3)
    return q, round_bf16(k.astype(F32)), v


def plain_global(q, k, v, cap, sink=True):
    H, G = q.shape[1], k.shape[1]
    p = sunk_weights(q.astype(np.float64), k.astype(np.float64), 1.0, cap)
    if not sink:
        p = p / p.sum(-1, keepdims=True)
    return np.stack([p[h] @ v[:, h // (H // G)] for h in range(H)], axis=1).reshape(len(q), -1)


@BOTH
@CAPS
@pytest.mark.parametrize("case", SIZES, ids=ids_of)
def test_global_attention_in_portions_and_steps(cuda, dtype, case, cap):
    H, G, D, V = case
    rng = np.random.default_rng(D + H)
    T, context, pad = 190, 200, 8
    for quiet in (False, True):
        q, k, v = global_case(rng, *case, T, quiet)
        scale = 1.0 if not quiet else 0.5
        sink = not (quiet and H % 3 == 0)
        want = plain_global(q * scale, k, v, cap, sink)
        limit = (3e-5 if dtype is F32 else 2e-2) * np.abs(want).max()
        keys, values = np.full((2, G, context, D), np.nan, F32), np.full((2, G, context, V), np.nan, F32)   # what a slot held before is nobody's
        keys[1, :, :T], values[1, :, :T] = k.swapaxes(0, 1), v.swapaxes(0, 1)
        for sizes in ([T], [64, 1, 1, 2, T - 68], [T // 2] + [1] * 20):
            got, at = [], 0
            for n in sizes:
                op = GlobalMHA(slots=2, rows=n + 3, heads=H, kv_heads=G, dim=D, vdim=V, context=context, width=H * V + 2 * pad, at=pad, scale=scale,
                               cap=cap, sink=sink, single=n == 1, dtype=dtype)
                held_k, held_v = keys.copy(), values.copy()
                held_k[1, :, at + n :], held_v[1, :, at + n :] = np.nan, np.nan   # what is not yet there is nothing
                out = ran(op, q=np.concatenate([np.full((3, H * D), 9.0), q[at : at + n].reshape(n, -1)]), spans=table((1, 3, n, at), slots=2),
                          keys=held_k, values=held_v, workspace=True if n == 1 else None)
                assert (out["y"][:3] == 7).all() and (out["y"][:, :pad] == 7).all() and (out["y"][:, H * V + pad :] == 7).all()
                got.append(out["y"][3:, pad : H * V + pad])
                at += n
            got = np.concatenate(got)
            assert np.isfinite(got).all() and np.abs(got - want[:at]).max() <= limit, (quiet, sizes, np.abs(got - want[:at]).max(), limit)


@BOTH
@pytest.mark.parametrize("single", [False, True], ids=["portion", "step"])
@pytest.mark.parametrize("case", [SIZES[0], SIZES[2], SIZES[4], SIZES[5], SIZES[7]], ids=ids_of)
def test_global_attention_over_several_requests(cuda, dtype, case, single):
    """Rows out of slot order, requests of unequal lengths, one that begins."""
    H, G, D, V = case
    rng = np.random.default_rng(3)
    parts = [(0, 4, 1, 300), (2, 0, 1, 127), (3, 2, 1, 128), (5, 3, 1, 0)] if single else [(0, 60, 130, 0), (2, 2, 1, 64), (3, 3, 57, 250), (4, 191, 2, 63)]
    rows, context = 6 if single else 200, 320
    keys, values, q = np.full((6, G, context, D), np.nan, F32), np.full((6, G, context, V), np.nan, F32), np.full((rows, H * D), 3.0, F32)
    want = {}
    for slot, row, n, start in parts:
        a, k, v = global_case(rng, *case, start + n)
        want[slot] = plain_global(a, k, v, 30.0)[start:]
        keys[slot, :, : start + n], values[slot, :, : start + n] = k.swapaxes(0, 1), v.swapaxes(0, 1)
        q[row : row + n] = a[start:].reshape(n, -1)
    op = GlobalMHA(slots=6, rows=rows, heads=H, kv_heads=G, dim=D, vdim=V, context=context, width=H * V, scale=1.0, cap=30.0, sink=True, single=single,
                   dtype=dtype)
    y = ran(op, q=q, spans=table(*parts, slots=6), keys=keys, values=values, workspace=True if single else None)["y"]
    for slot, row, n, _ in parts:
        assert np.abs(y[row : row + n] - want[slot]).max() <= (3e-5 if dtype is F32 else 2e-2) * np.abs(want[slot]).max(), slot
    idle = np.setdiff1d(np.arange(rows), np.concatenate([np.arange(r, r + n) for _, r, n, _ in parts]))
    assert (y[idle] == 7).all()


@pytest.mark.parametrize("case", [(8, 2, 64, 64), (4, 1, 128, 64)], ids=ids_of)
@pytest.mark.parametrize("cap", [0.0, 30.0, 55.0])
def test_a_step_deep_in_a_long_context(cuda, case, cap):
    """Many runs of keys, several tiles each; a key that stands out in the first, at runs' edges and in the last."""
    H, G, D, V = case
    rng, count, context = np.random.default_rng(5), 9000, 70000
    q, k, v = bf(rng, H, D, scale=0.3), bf(rng, count, G, D, scale=0.3), bf(rng, count, G, V)
    for far in (0, 127, 128, 4095, count - 1):
        k[far] = 0.0
        for h in range(0, H, max(1, H // G)):
            k[far, h // (H // G)] = 12 * q[h] / np.linalg.norm(q[h])
    k = round_bf16(k.astype(F32))
    s = np.einsum("hd,jhd->hj", q.astype(np.float64), k[:, np.arange(H) // (H // G)].astype(np.float64))
    s = cap * np.tanh(s / cap) if cap else s
    e = np.exp(s - s.max(1, keepdims=True))
    p = e / (e.sum(1, keepdims=True) + np.exp(-s.max(1, keepdims=True)))
    want = np.einsum("hj,jhv->hv", p, v[:, np.arange(H) // (H // G)].astype(np.float64)).reshape(-1)
    keys, values = np.full((1, G, context, D), np.nan, F32), np.full((1, G, context, V), np.nan, F32)
    keys[0, :, :count], values[0, :, :count] = k.swapaxes(0, 1), v.swapaxes(0, 1)
    op = GlobalMHA(slots=1, rows=1, heads=H, kv_heads=G, dim=D, vdim=V, context=context, width=H * V, scale=1.0, cap=cap, sink=True, single=True)
    y = ran(op, q=q.reshape(1, -1), spans=table((0, 0, 1, count - 1)), keys=keys, values=values, workspace=True)["y"][0]
    assert np.abs(y - want).max() <= 2e-2 * np.abs(want).max()


# ---------------------------------------------------------------- the fading memory


def fading_inputs(rng, op, spans):
    x = bf(rng, op.rows, op.stride)
    x[:, op.channels : 2 * op.channels] = bf(rng, op.rows, op.channels, scale=3)
    lower = round_bf16((rng.uniform(0, 0.98, op.channels) * (rng.random(op.channels) > 0.3)).astype(F32))
    return dict(x=x, f_bias=round_bf16(rng.uniform(-2, 6, op.channels).astype(F32)), lower=lower,
                state=rng.standard_normal((op.slots, op.heads, op.dim, op.vdim)).astype(F32), spans=spans)


def fading_op(slots, rows, H, D, V, dtype, more=0):
    return Hgrn2(slots=slots, rows=rows, stride=H * (2 * D + V) + more, heads=H, dim=D, vdim=V, dtype=dtype)


TOKENS = pytest.mark.parametrize("chunked", [False, True], ids=["tokens", "chunks"])


@BOTH
@TOKENS
@pytest.mark.parametrize("H,D,V", [(2, 24, 40), (3, 5, 9), (1, 33, 3), (4, 16, 16), (2, 64, 128), (2, 128, 64), (2, 128, 256), (1, 256, 160), (1, 200, 33)])
def test_a_fading_memory(cuda, dtype, chunked, H, D, V):
    rng = np.random.default_rng(D)
    # lengths around a chunk's, rows out of slot order, slots that go on and ones that start over
    spans = table((0, 130, 33, 9), (1, 0, 32, 0), (2, 32, 1, 3), (4, 33, 97, 0), (5, 163, 2, 40), slots=6)
    op = fading_op(6, 170, H, D, V, dtype, more=24)
    agrees(op, fading_inputs(rng, op, spans), 2e-5, rows_of(spans), workspace=chunked)


@TOKENS
def test_a_fading_memory_goes_on_where_a_portion_ends(cuda, chunked):
    rng = np.random.default_rng(7)
    H, D, V, T = 2, 40, 48, 200
    whole = fading_inputs(rng, fading_op(1, T, H, D, V, F32), table((0, 0, T, 0)))
    whole["x"][90, H * D] = 1000.0     # a gate that keeps all, and one that closes altogether under no bound
    whole["x"][120, H * D : 2 * H * D] = -1000.0
    x = whole["x"].astype(np.float64)
    q, v = (x[:, : H * D] * sigmoid(x[:, : H * D])).reshape(T, H, D), x[:, 2 * H * D :].reshape(T, H, V)
    f = (whole["lower"] + (1 - whole["lower"]) * sigmoid(x[:, H * D : 2 * H * D] + whole["f_bias"])).reshape(T, H, D)
    want, _ = hgrn2(q, v, f)
    for sizes in ([T], [2, 31, 1, 70, 33, 2, 61], [16] * 12 + [8], [1] * 40):
        state, at = whole["state"], 0
        for n in sizes:
            got = ran(fading_op(1, n, H, D, V, F32), workspace=chunked, **{**whole, "x": whole["x"][at : at + n], "state": state, "spans": table((0, 0, n, at))})
            assert np.abs(got["o"].reshape(n, H, V) - want[at : at + n]).max() <= 2e-5 * np.abs(want).max(), (sizes[:3], at)
            state, at = got["state"], at + n


@BOTH
@pytest.mark.parametrize("H,V", [(2, 40), (3, 9), (4, 256), (1, 200)])
def test_heads_normed_without_a_gate(cuda, dtype, H, V):
    rng = np.random.default_rng(V)
    op = HeadGate(rows=7, heads=H, dim=V, gated=False, gains=V, width=H * V + 24, at=8, epsilon=1e-3, dtype=dtype)
    agrees_at = dict(o=rng.standard_normal((7, H * V)).astype(F32), gain=bf(rng, V))
    got, want = ran(op, **agrees_at)["y"][:, 8 : 8 + H * V], op._call_reference(agrees_at)["y"][:, 8 : 8 + H * V]
    assert np.abs(got - want).max() <= (3e-6 if dtype is F32 else 5e-3) * np.abs(want).max()


@pytest.mark.parametrize("H,D,V,cols,logits", [(2, 24, 16, 40, 0), (3, 128, 128, 0, 5), (4, 256, 64, 1100, 66), (1, 40, 256, 24, 18)])
def test_a_step_s_memory_with_columns_and_a_choice_beside(cuda, H, D, V, cols, logits):
    rng = np.random.default_rng(D + V)
    slots, own = (1 if logits else 4), H * (2 * D + V)
    spans = table(*[(i, slots - 1 - i, 1, (5, 0, 3, 9)[i]) for i in range(slots) if i != 2], slots=slots)
    op = fading_op(slots, slots, H, D, V, BF16, more=2 * cols)
    given, gain, width, at = fading_inputs(rng, op, spans), bf(rng, V), H * V + cols + 8, 8
    want = op._call_reference(given)
    t = {n: device(given[n], BF16) for n in ("x", "f_bias", "lower")}
    t |= dict(state=device(given["state"], F32), spans=device(spans, np.int32), norm=device(gain, BF16), out=device(np.full((slots, width), 7.0), BF16))
    kw = dict(slots=slots, rows=slots, stride=op.stride, heads=H, dim=D, vdim=V, out_stride=width, out_at=at, eps=1e-3)
    if cols:
        kw |= dict(cols=cols, gate_at=own, gated_at=H * V + at, kind="silu")
    choice = {}
    if logits:
        z, correction = rng.standard_normal(logits).astype(F32), bf(rng, logits, scale=0.2)
        choice = dict(z=device(z, F32), correction=device(correction, BF16), logits=logits, top=3, ids=device(np.zeros(3), np.int32),
                      shares=device(np.zeros(3), F32))
    K.decode_hgrn2(**t, **kw, **choice)
    torch.cuda.synchronize()
    rows = rows_of(spans)
    y = over_rms(want["o"].reshape(slots, H, V), 1e-3) * gain
    got, state = from_torch(t["out"])[rows], from_torch(t["state"])
    assert np.abs(got[:, at : at + H * V] - y.reshape(slots, -1)[rows]).max() <= 6e-3 * np.abs(y).max() and (got[:, :at] == 7).all()
    assert np.abs(state - want["state"]).max() <= 1e-5 * np.abs(want["state"]).max()
    if cols:
        whole = ran(GatedColumns(rows=slots, cols=cols, stride=op.stride, width=width, gate_at=own, at=H * V + at, kind="silu"), x=given["x"],
                    y=np.full((slots, width), 7.0))["y"][rows]
        assert np.array_equal(got[:, H * V + at :], whole[:, H * V + at :])
    if logits:
        check_choice(z, correction, 3, choice["ids"].cpu().numpy(), from_torch(choice["shares"]))


# ---------------------------------------------------------------- experts


@BOTH
@pytest.mark.parametrize("rows,cols,experts,top", [(5, 128, 13, 3), (300, 96, 7, 7), (1, 60, 1, 1), (9, 37, 130, 11), (4, 2048, 66, 8), (8, 512, 18, 4)])
def test_a_scored_router(cuda, dtype, rows, cols, experts, top):
    rng = np.random.default_rng(cols)
    given = dict(h=bf(rng, rows, cols), weight=bf(rng, experts, cols, scale=2 / np.sqrt(cols)), correction=bf(rng, experts, scale=0.3))
    op = Router(rows=rows, cols=cols, experts=experts, top=top, scored=True, biased=False, corrected=True, dtype=dtype)
    want, got = op._call_reference(given), ran(op, **given)
    assert np.array_equal(got["ids"], want["ids"]) and np.abs(got["shares"] - want["shares"]).max() < 1e-5
    # equal scores: the first ones; without corrections
    plain = Router(rows=rows, cols=cols, experts=experts, top=top, scored=True, biased=False, dtype=dtype)
    got = ran(plain, h=given["h"], weight=np.zeros((experts, cols), F32))
    assert np.array_equal(got["ids"], np.tile(np.arange(top), (rows, 1))) and np.allclose(got["shares"], 1 / top)


@BOTH
@pytest.mark.parametrize("rows,cols,ff,experts,identity,top", [(5, 128, 80, 11, 2, 2), (300, 96, 64, 7, 1, 2), (1, 60, 21, 1, 3, 2), (9, 37, 10, 5, 2, 7),
                                                               (200, 256, 128, 16, 4, 4), (130, 256, 104, 40, 1, 3), (700, 192, 320, 3, 2, 1), (1, 2048, 256, 16, 2, 4)])
def test_routed_feed_forwards_and_identities(cuda, dtype, rows, cols, ff, experts, identity, top):
    rng = np.random.default_rng(ff)
    ids = np.stack([rng.permutation(experts + identity)[:top] for _ in range(rows)]).astype(np.int32)
    ids[0, 0] = experts + identity - 1 if experts + identity - 1 not in ids[0, 1:] else ids[0, 0]
    shares = rng.dirichlet(np.ones(top), rows).astype(F32)
    given = dict(h=bf(rng, rows, cols), gate=bf(rng, experts * ff, cols, scale=1 / np.sqrt(cols)), up=bf(rng, experts * ff, cols, scale=1 / np.sqrt(cols)),
                 down=bf(rng, experts * cols, ff, scale=1 / np.sqrt(ff)), ids=ids, shares=shares)
    op = Experts(rows=rows, cols=cols, experts=experts, identity=identity, top=top, ff=ff, activation="silu", dtype=dtype)
    agrees(op, given, 5e-6 if dtype is F32 else 1e-2, workspace=True)


@pytest.mark.parametrize("cols,ff,inner,experts,identity,top", [(128, 80, 200, 11, 2, 3), (64, 8, 8, 1, 1, 2), (512, 256, 1536, 16, 2, 4), (96, 512, 2048, 5, 0, 5),
                                                                (256, 1024, 4096, 8, 3, 8), (40, 24, 16, 4, 70, 40)])
def test_one_row_s_experts_with_the_output_beside(cuda, cols, ff, inner, experts, identity, top):
    rng = np.random.default_rng(cols)
    ids = rng.permutation(experts + identity)[:top].astype(np.int32)
    ids[0] = experts if identity and experts not in ids else ids[0]
    shares = rng.dirichlet(np.ones(top)).astype(F32)
    given = dict(h=bf(rng, 1, cols), gate=bf(rng, experts * ff, cols, scale=1 / np.sqrt(cols)), up=bf(rng, experts * ff, cols, scale=1 / np.sqrt(cols)),
                 down=bf(rng, experts * cols, ff, scale=1 / np.sqrt(ff)), ids=ids[None], shares=shares[None])
    routed = Experts(rows=1, cols=cols, experts=experts, identity=identity, top=top, ff=ff, activation="silu")._call_reference(given)["y"][0]
    out, made, stream = bf(rng, cols, inner, scale=inner**-0.5), bf(rng, inner), rng.standard_normal(cols).astype(F32)
    at = device(stream, F32)
    t = {n: device(given[n], BF16) for n in ("h", "gate", "up", "down")}
    K.experts_tail(t["h"].reshape(-1), t["gate"], t["up"], t["down"], device(ids, np.int32), device(shares, F32), device(out, BF16), device(made, BF16), at,
                   torch.full((top * ff,), float("nan"), device="cuda"), cols=cols, ff=ff, inner=inner, experts=experts, identity=identity, top=top,
                   activation="silu")
    torch.cuda.synchronize()
    product = out.astype(np.float64) @ made
    want = stream + product + routed
    assert np.abs(from_torch(at) - want).max() <= 1e-2 * max(np.abs(product).max(), np.abs(routed).max())


# ---------------------------------------------------------------- whole models


LIMIT = {"f32": 2e-4, "bf16": 0.1}   # of the logits' spread


def off_by(got, want, limit):
    """The largest difference of a row; the middle one where rounding may turn a router's close call, which moves a row and what
    a state carries of it by itself."""
    each = np.array([far_off(g[None], w[None], want.std()) for g, w in zip(got, want)])
    return float(each.max() if limit < 1e-2 else np.median(each))


@pytest.fixture(scope="module", params=[(n, d, f) for n in MODELS for d in ("f32", "bf16") for f in ((True, False) if d == "bf16" else (True,))],
                ids=lambda p: f"{p[0]}-{p[1]}-{'fused' if p[2] else 'steps'}")
def served(request):
    name, dtype, fuse = request.param
    model, plain = built(name, Pudinex, activations=F32 if dtype == "f32" else BF16, slots=3, max_seq_len=400, prefill_chunk=128)
    model.load_versions(fuse=fuse, capture=fuse)
    yield model, plain, LIMIT[dtype]
    model.release()


def tokens_of(model, n, seed=1):
    return np.random.default_rng(seed).integers(0, model.config.vocab_size, n)


def test_portions_of_a_prompt_and_decoding(cuda, served):
    model, plain, limit = served
    tokens = tokens_of(model, 170)
    want = plain(tokens)
    for sizes in ([170], [2] * 12 + [146], [100, 67, 3], [130] + [1] * 40, [1] * 30 + [140]):
        rows, at = [], 0
        for n in sizes:
            rows.append(model.batch.step([Entry("x", tokens[at : at + n], range(n))])[0])
            at += n
        model.batch.end("x")
        off = off_by(np.concatenate(rows), want, limit)
        print(sizes[:3], off)
        assert off < limit, sizes


def test_batches_and_slots_used_again(cuda, served):
    model, plain, limit = served
    prompts = {k: tokens_of(model, n, seed=n) for k, n in (("a", 150), ("b", 1), ("c", 44))}
    want = {k: plain(t) for k, t in prompts.items()}
    for order in ("abc", "cab", "b", "ca"):
        first = {k: max(1, len(prompts[k]) - 20) for k in order}
        got = model.batch.step([Entry(k, prompts[k][: first[k]], range(first[k])) for k in order])
        rows = {k: [r] for k, r in zip(order, got)}
        for i in range(20):
            live = [k for k in order if first[k] + i < len(prompts[k])]
            if live:
                for k, r in zip(live, model.batch.step([Entry(k, [prompts[k][first[k] + i]], [0]) for k in live])):
                    rows[k].append(r)
        for k in order:
            off = off_by(np.concatenate(rows[k]), want[k], limit)
            print(order, k, off)
            assert off < limit, (order, k)
            model.batch.end(k)


def test_long_decoding(cuda):
    model, plain = built("mixed", Pudinex, slots=1, max_seq_len=700, prefill_chunk=64, activations=F32)
    model.load_versions()
    tokens = tokens_of(model, 640)
    want = plain(tokens)
    model.batch.step([Entry("x", tokens[:40])])
    rows = np.concatenate([model.batch.step([Entry("x", [t], [0])])[0] for t in tokens[40:]])
    model.release()
    assert off_by(rows, want[40:], LIMIT["f32"]) < LIMIT["f32"]


FUSED = {"wide": {"norm_product_router_mixer", "norm_product", "step_mixer", "experts_tail", "product_sum"},
         "whole": {"norm_product_router_mixer", "experts_tail"}, "mixed": {"experts_tail", "product_sum"}, "odd": set()}


@pytest.mark.parametrize("name", MODELS)
def test_a_single_slot_s_steps(cuda, name):
    """One slot: a decode step's projections are single-row products, with what is ahead and behind them in their launches."""
    model, plain = built(name, Pudinex, slots=1, max_seq_len=300, prefill_chunk=96)
    model.load_versions()
    try:
        assert FUSED[name] <= {f.kind for f in model.decode_step._fused.values()}
        assert "stream_sum_norm" in {f.kind for f in model.prompt_chunk._fused.values()}
        tokens = tokens_of(model, 200)
        want = plain(tokens)
        rows = [model.batch.step([Entry("x", tokens[:60], range(60))])[0]]
        rows += [model.batch.step([Entry("x", [t], [0])])[0] for t in tokens[60:]]
        assert off_by(np.concatenate(rows), want, LIMIT["bf16"]) < LIMIT["bf16"]
    finally:
        model.release()


def test_generation_replays_what_stepwise_decoding_draws(cuda):
    model, plain = built("mixed", Pudinex, slots=3, max_seq_len=200, prefill_chunk=32)
    model.load_versions()
    try:
        assert model.decode_step.captured
        prompts = [tokens_of(model, n, seed=n) for n in (50, 3, 17, 90, 8)]
        together = model.generate_batch(prompts, 40)
        assert all(len(t) == 40 for t in together)
        assert together == model.generate_batch(prompts, 40)
        # Each greedy token is a best one of the plain logits, up to the kernels' rounding.
        for prompt, out in zip(prompts[:3], together):
            logits = plain(np.concatenate([prompt, out]).astype(int))
            for i, t in enumerate(out[:12]):
                row = logits[len(prompt) - 1 + i]
                assert row[t] >= row.max() - 6 * LIMIT["bf16"] * logits.std()
        # Replays (nothing read back between them) draw what one step at a time does, and stream() what generate() does.
        one = list(model.session.draw(prompts[0], 30))
        assert one == list(model.session.draw(prompts[0], 30, each=True)) == model.generate(prompts[0], 30)
        assert list(model.stream(prompts[0], 30)) == one and model.stats.tokens == 30
        samplers = [[Sampler(0.9, 30, seed=s) for s in range(5)] for _ in range(2)]
        assert model.generate_batch(prompts, 25, samplers[0]) == model.generate_batch(prompts, 25, samplers[1])
        assert model.generate_batch(prompts, 40) == together   # greedy again
    finally:
        model.release()


@pytest.mark.parametrize("slots", [1, 2])
def test_a_replayed_step_is_the_eager_one_each_time(cuda, slots):
    captured, _ = built("wide", Pudinex, slots=slots, max_seq_len=120, prefill_chunk=32)
    eager, _ = built("wide", Pudinex, slots=slots, max_seq_len=120, prefill_chunk=32)
    captured.load_versions()
    eager.load_versions(capture=False)
    try:
        prompts = [tokens_of(captured, n, seed=n) for n in (21, 40)][:slots]
        for model in (captured, eager):
            model.batch.step([Entry(i, p) for i, p in enumerate(prompts)])
        for step in range(12):
            fed = tokens_of(captured, slots, seed=step)
            a, b = (model.batch.step([Entry(i, [t], [0]) for i, t in enumerate(fed)]) for model in (captured, eager))
            torch.cuda.synchronize()
            assert np.array_equal(np.concatenate(a), np.concatenate(b)), step
    finally:
        captured.release()
        eager.release()


def saved(folder, name):
    doc = MODELS[name]
    (folder / "config.json").write_text(json.dumps(doc))
    write_safetensors(folder / "model.safetensors", weights_of(PudinexConfig.from_json(doc)))
    return doc


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_a_trace_is_replayed(cuda, tmp_path, dtype):
    doc = saved(tmp_path, "odd")
    _, plain = built("odd", Pudinex)
    tokens = np.random.default_rng(0).integers(0, doc["vocab"], 30).tolist()
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": tokens[:20], "want": [0, 19]}], "end": []},
             {"step": 1, "entries": [{"id": "a", "tokens": tokens[20:21], "want": []}], "end": ["a"]},
             {"step": 2, "entries": [{"id": "b", "tokens": tokens[:5], "want": [4]}, {"id": "c", "tokens": tokens, "want": [29, 3]}], "end": ["b"]}]
    done = subprocess.run([sys.executable, str(Path(__file__).resolve().parent.parent / "bin" / "trace_run"), "--model", str(tmp_path),
                           "--dtype", dtype, "--out", str(tmp_path), "--max-tokens", "64"], capture_output=True, text=True,
                          input="\n".join(map(json.dumps, steps)) + "\n", timeout=120)
    assert done.returncode == 0, done.stderr[-2000:]
    assert [line for line in done.stdout.splitlines() if line.startswith("done")] == ["done 0", "done 1", "done 2"]
    want = plain(tokens)
    for step, places in ((0, [0, 19]), (2, [4, 29, 3])):
        rows = np.fromfile(tmp_path / f"{step}.f32", "<f4").reshape(len(places), doc["vocab"])
        limit = LIMIT["f32" if dtype == "float32" else "bf16"]
        assert off_by(rows, want[places], limit) < limit
    assert not (tmp_path / "1.f32").exists()


def test_the_command_line_generates_a_batch(cuda, tmp_path, capsys):
    from iron_amd.__main__ import main

    doc = saved(tmp_path, "mixed")
    prompts = [np.random.default_rng(n).integers(0, doc["vocab"], n).tolist() for n in (11, 4)]
    asked = [a for p in prompts for a in ("--ids", ",".join(map(str, p)))]
    assert main([str(tmp_path), *asked, "--count", "9", "--max-seq-len", "64"]) == 0
    printed = [[int(t) for t in line.split(",")] for line in capsys.readouterr().out.splitlines()]
    model = Pudinex.load(tmp_path, slots=2, max_seq_len=64)
    try:
        assert printed == model.generate_batch(prompts, 9)
    finally:
        model.release()
