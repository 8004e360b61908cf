"""Tilarax's mechanisms and models on the GPU against the oracle and the plain implementation: each kernel
alone, prompts, portions, batches, slots used again, far keys, chunk edges, long decoding, generation."""

import json
import subprocess
import sys
from pathlib import Path

import numpy as np
import pytest
import torch

import oracle
from iron_amd import kernels as K
from iron_amd.applications import Tilarax, TilaraxConfig
from iron_amd.bf16 import bfloat16, from_torch, round_bf16
from iron_amd.lm import Sampler, rope_angles, write_safetensors
from iron_amd.lm.batched import Entry
from iron_amd.operators.experts import Experts, Router
from iron_amd.operators.mha_talking import TalkingMHA, TurnedHeads
from iron_amd.operators.recurrent import MatrixMemory, MemoryGate
from iron_amd.operators.stream import Activation, DepthAverage, StreamAdd, StreamCast, StreamEmbed, StreamNorm
from tests.operator_support import agrees, bf, device, ran, rows_of, table
from tests.tilarax_plain import chunk_weights, log_gates, mlstm, talked
from tests.tilarax_support import MODELS, built, far_off, weights_of

pytestmark = pytest.mark.gpu
oracle.install()
F32, BF16 = np.float32, bfloat16
BOTH = pytest.mark.parametrize("dtype", [F32, BF16], ids=["f32", "bf16"])
ids_of = lambda p: "x".join(map(str, p))  # noqa: E731


# ---------------------------------------------------------------- the stream


@BOTH
@pytest.mark.parametrize("rows,cols,index", [(5, 128, 1), (3, 60, 4), (2, 2056, 6), (3, 4160, 9), (1, 1303, 5), (1, 9000, 2)])
def test_a_row_joins_the_stream_and_is_averaged_over_depth(cuda, dtype, rows, cols, index):
    rng = np.random.default_rng(cols)
    x, y, gain, y_bias = rng.standard_normal((rows, cols)).astype(F32) * 3, bf(rng, rows, cols), bf(rng, cols), bf(rng, cols)
    planes, weights = rng.standard_normal((index + 2, rows + 2, cols)).astype(F32), bf(rng, index + 1)
    kw = dict(rows=rows, cols=cols)
    added = agrees(StreamAdd(epsilon=1e-3, unit=1.0, biased=True, dtype=dtype, **kw), dict(x=x, y=y, weight=gain, y_bias=y_bias), 2e-6)["x"]
    depth = DepthAverage(depth=index + 2, plane_rows=rows + 2, count=index + 1, **kw)
    mixed = agrees(depth, dict(x=added, planes=planes, weights=weights), 2e-6)
    assert np.array_equal(mixed["planes"][index, :rows], added)
    assert np.array_equal(mixed["planes"][index, rows:], planes[index, rows:]) and np.array_equal(mixed["planes"][index + 1], planes[index + 1])
    cast = ran(StreamCast(dtype=dtype, **kw), x=mixed["x"])["y"]
    assert np.array_equal(cast, mixed["x"] if dtype is F32 else round_bf16(mixed["x"]))
    # all three in one launch, and the two pairs: bit for bit
    for use_add, use_depth in ((True, True), (True, False), (False, True)):
        xd, pd = device(x if use_add else added, F32), device(planes, F32)
        hd = torch.empty((rows, cols), dtype=torch.bfloat16 if dtype is BF16 else torch.float32, device="cuda")
        given = dict(y=device(y, dtype), back_gain=device(gain, BF16), y_bias=device(y_bias, BF16)) if use_add else {}
        given |= dict(planes=pd, weights=device(weights, BF16)) if use_depth else {}
        K.stream_depth_rows(xd, h=hd, eps=1e-3, unit=1.0, plane_rows=rows + 2 if use_depth else 0, index=index if use_depth else 0, **kw, **given)
        torch.cuda.synchronize()
        want = mixed["x"] if use_depth else added
        assert np.array_equal(from_torch(xd), want) and np.array_equal(from_torch(hd), want if dtype is F32 else round_bf16(want))
        if use_depth:
            assert np.array_equal(from_torch(pd), mixed["planes"])


@pytest.mark.parametrize("cols", [64, 61])
def test_embedding_rows_into_two_places(cuda, cols):
    rng = np.random.default_rng(cols)
    t, ids = bf(rng, 30, cols), rng.integers(0, 30, 9)
    got = ran(StreamEmbed(rows=9, table_rows=30, cols=cols, twice=True), table=t, ids=ids)
    assert np.array_equal(got["x"], t[ids]) and np.array_equal(got["also"], t[ids])


@BOTH
@pytest.mark.parametrize("cols", [96, 37, 5000])
def test_norms_around_one_and_activations(cuda, dtype, cols):
    rng = np.random.default_rng(cols)
    x = bf(rng, 3, cols, scale=3)
    agrees(StreamNorm(rows=3, cols=cols, epsilon=1e-3, unit=1.0, dtype=dtype), dict(x=x, weight=bf(rng, cols, scale=0.2)), 2e-6 if dtype is F32 else 5e-3)
    for kind in ("gelu_tanh", "silu", "relu"):
        agrees(Activation(rows=3, cols=cols, kind=kind, dtype=dtype), dict(x=x), 3e-6 if dtype is F32 else 5e-3)


# ---------------------------------------------------------------- the rows of attention


@BOTH
@pytest.mark.parametrize("H,G,D,V,turned", [(6, 2, 32, 48, 16), (3, 1, 11, 7, 6), (2, 2, 128, 64, 128), (6, 2, 88, 200, 0), (8, 4, 8, 16, 2)])
def test_turned_heads(cuda, dtype, H, G, D, V, turned):
    rng = np.random.default_rng(D)
    stride, first_at = (H + G) * D + G * V, 24
    spans = table((0, 30, 40, 60), (1, 3, 1, 7), (3, 4, 26, 0), slots=4)
    given = dict(x=bf(rng, 72, stride), bias=bf(rng, stride), q_gain=bf(rng, D), k_gain=bf(rng, D), temp=bf(rng, H), spans=spans)
    given |= {"angles": rope_angles(turned, 128, 400.0)} if turned else {}
    for blended in (False, True):
        more = dict(first=bf(rng, 72, G * V + 40), share=bf(rng, 1)) if blended else {}
        op = TurnedHeads(slots=4, rows=72, stride=stride, heads=H, kv_heads=G, dim=D, turned=turned, angle_rows=128 if turned else 1, mixed=blended,
                         first_stride=G * V + 40 if blended else 0, first_at=first_at if blended else 0, scale=0.3, epsilon=1e-3, dtype=dtype)
        agrees(op, given | more, 3e-6 if dtype is F32 else 5e-3, rows_of(spans))


# ---------------------------------------------------------------- attention within chunks

# heads, key/value heads, dim, vdim, chunk
SIZES = [(6, 2, 32, 48, 37), (4, 4, 64, 24, 20), (3, 1, 11, 7, 13), (1, 1, 12, 7, 1), (16, 4, 64, 64, 96), (32, 4, 32, 64, 160), (2, 2, 40, 48, 70),
         (24, 8, 128, 128, 300), (32, 8, 64, 64, 128), (8, 2, 88, 48, 65), (5, 5, 72, 16, 100), (12, 3, 128, 112, 64), (40, 8, 32, 32, 50), (32, 8, 128, 128, 600), (8, 8, 16, 8, 1050)]


def talking_case(rng, H, G, D, V, C, T, quiet=False):
    """A sequence's rows and the heads' mixing under which chosen queries meet a key that stands out at their chunk's first
    place, and a louder one just outside, the last of the chunk before -- or, ``quiet``, no key that does."""
    q, k, v = bf(rng, T, H, D, scale=0.5 if quiet else 0.25), bf(rng, T, G, D, scale=1.0 if quiet else 0.4), bf(rng, T, G, V)
    for i in range(0 if quiet else T):
        if i % C and i % 5 == 0:
            h = i % H
            toward = q[i, h] / max(float(np.linalg.norm(q[i, h])), 1e-3)
            k[i // C * C, h // (H // G)] = 14 * toward
            if i >= C:
                k[i // C * C - 1, h // (H // G)] = 30 * toward
    talk = round_bf16((np.eye(H) * 0.7 + 0.5 * rng.standard_normal((H, H)) / np.sqrt(H)).astype(F32))
    return q, round_bf16(k.astype(F32)), v, talk


def plain_talking(q, k, v, talk, C):
    H, G = q.shape[1], k.shape[1]
    p = talked(chunk_weights(q.astype(np.float64), k.astype(np.float64), np.ones(H), C), talk)
    return np.stack([p[h] @ v[:, h // (H // G)] for h in range(H)], axis=1).reshape(len(q), -1)


def packed(q, k, v):
    return np.concatenate([a.reshape(len(a), -1) for a in (q, k, v)], axis=1)


@BOTH
@pytest.mark.parametrize("quiet", [False, True], ids=["loud", "quiet"])
@pytest.mark.parametrize("case", SIZES, ids=ids_of)
def test_talking_attention_in_portions_and_steps(cuda, dtype, case, quiet):
    H, G, D, V, C = case
    rng = np.random.default_rng(D + H)
    T = 190 if C < 190 else C + 40
    q, k, v, talk = talking_case(rng, *case, T, quiet)
    x, want = packed(q, k, v), plain_talking(q, k, v, talk, C)
    limit = (3e-5 if dtype is F32 else 2e-2) * np.abs(want).max()
    for sizes in ([T], [64, 1, 1, 2, T - 68], [T // 2] + [1] * 30):
        keys, values = np.full((2, C, G, D), 5.0, F32), np.full((2, C, G, V), 5.0, F32)   # what a slot held before is nobody's
        got, at = [], 0
        for n in sizes:
            op = TalkingMHA(slots=2, rows=n + 3, stride=x.shape[1], heads=H, kv_heads=G, dim=D, vdim=V, chunk=C, single=n == 1, dtype=dtype)
            out = ran(op, x=np.concatenate([np.full((3, x.shape[1]), 9.0), x[at : at + n]]), talk=talk, spans=table((1, 3, n, at), slots=2),
                      keys=keys, values=values, workspace=True)
            keys, values = out["keys"], out["values"]
            assert (out["y"][:3] == 7).all()   # the sequence is not the batch's first rows
            assert (keys[0] == 5).all() and (values[0] == 5).all()
            got.append(out["y"][3:])
            at += n
        seen = np.arange(max(0, at - C), at)
        assert np.array_equal(keys[1, seen % C], k[seen]) and np.array_equal(values[1, seen % C], v[seen])
        got = np.concatenate(got)
        assert np.isfinite(got).all() and np.abs(got - want[:at]).max() <= limit, (sizes, np.abs(got - want[:at]).max(), limit)


@BOTH
@pytest.mark.parametrize("single", [False, True], ids=["portion", "step"])
@pytest.mark.parametrize("case", [SIZES[0], SIZES[2], SIZES[4], SIZES[7]], ids=ids_of)
def test_talking_attention_over_several_requests(cuda, dtype, case, single):
    """Rows out of slot order, requests that go on inside a chunk, at its edge and a row ahead of it."""
    H, G, D, V, C = case
    rng = np.random.default_rng(3)
    parts = [(0, 4, 1, 2 * C), (2, 0, 1, 2 * C - 1), (3, 2, 1, C // 2), (5, 3, 1, 0)] if single else \
            [(0, 60, 130, 0), (2, 2, 1, C), (3, 3, 57, 2 * C - 1), (4, 191, 2, C // 2)]
    rows, stride = 6 if single else 200, (H + G) * D + G * V
    keys, values, x = np.full((6, C, G, D), 3.0, F32), np.full((6, C, G, V), 3.0, F32), np.full((rows, stride), 3.0, F32)
    talk, want = None, {}
    for slot, row, n, start in parts:
        q, k, v, t = talking_case(rng, *case, start + n)
        talk = t if talk is None else talk
        want[slot] = plain_talking(q, k, v, talk, C)[start:]
        for j in range(max(0, start - C), start):
            keys[slot, j % C], values[slot, j % C] = k[j], v[j]
        x[row : row + n] = packed(q, k, v)[start:]
    op = TalkingMHA(slots=6, rows=rows, stride=stride, heads=H, kv_heads=G, dim=D, vdim=V, chunk=C, single=single, dtype=dtype)
    y = ran(op, x=x, talk=talk, spans=table(*parts, slots=6), keys=keys, values=values, workspace=True)["y"]
    for slot, row, n, _ in parts:
        assert np.abs(y[row : row + n] - want[slot]).max() <= (3e-5 if dtype is F32 else 2e-2) * np.abs(want[slot]).max(), slot
    idle = np.setdiff1d(np.arange(rows), np.concatenate([np.arange(r, r + n) for _, r, n, _ in parts]))
    assert (y[idle] == 7).all()


# ---------------------------------------------------------------- the matrix memory


def memory_inputs(rng, op, spans):
    x = bf(rng, op.rows, op.stride)
    x[:, op.i_at : op.i_at + op.heads] = bf(rng, op.rows, op.heads, scale=4)
    return dict(x=x, i_bias=bf(rng, op.heads), f_bias=round_bf16(rng.uniform(-2, 6, op.heads).astype(F32)),
                state=rng.standard_normal((op.slots, op.heads, op.dim, op.vdim + 1)).astype(F32),
                tops=rng.standard_normal((op.slots, 2, op.heads)).astype(F32), spans=spans)


def memory_op(slots, rows, H, D, V, dtype, more=0, cap=9.0):
    packed = H * (2 * D + V)
    return MatrixMemory(slots=slots, rows=rows, stride=packed + more + 2 * H, heads=H, dim=D, vdim=V, i_at=packed + more, f_at=packed + more + H,
                        cap=cap, dtype=dtype)


TOKENS = pytest.mark.parametrize("chunked", [False, True], ids=["tokens", "chunks"])


@BOTH
@TOKENS
@pytest.mark.parametrize("H,D,V", [(2, 24, 40), (3, 5, 9), (1, 33, 3), (4, 16, 16), (2, 64, 128), (2, 128, 64), (2, 128, 256), (1, 256, 160), (1, 300, 33)])
def test_a_matrix_memory(cuda, dtype, chunked, H, D, V):
    if chunked and D > 256:
        pytest.skip("longer keys go token by token")
    rng = np.random.default_rng(D)
    # lengths around a chunk's, rows out of slot order, slots that go on and ones that start over
    spans = table((0, 130, 33, 9), (1, 0, 32, 0), (2, 32, 1, 3), (4, 33, 97, 0), (5, 163, 2, 40), slots=6)
    op = memory_op(6, 170, H, D, V, dtype, more=H * V)
    agrees(op, memory_inputs(rng, op, spans), 2e-5, rows_of(spans), workspace=chunked)


@TOKENS
def test_the_memory_goes_on_where_a_portion_ends(cuda, chunked):
    rng = np.random.default_rng(7)
    H, D, V, T = 2, 40, 48, 200
    op = memory_op(1, T, H, D, V, F32)
    whole = memory_inputs(rng, op, table((0, 0, T, 0)))
    whole["x"][90, op.i_at] = 60.0   # a gate that stands out
    x = whole["x"].astype(np.float64)
    q, k, v = x[:, : H * D].reshape(T, H, D) * D**-0.5, x[:, H * D : 2 * H * D].reshape(T, H, D), x[:, 2 * H * D : op.i_at].reshape(T, H, V)
    want, _ = mlstm(q, k, v, *log_gates(x[:, op.i_at : op.f_at] + whole["i_bias"], x[:, op.f_at :] + whole["f_bias"], 9.0))
    for sizes in ([T], [2, 31, 1, 70, 33, 2, 61], [16] * 12 + [8], [1] * 40):
        state, tops, at = whole["state"], whole["tops"], 0
        for n in sizes:
            got = ran(memory_op(1, n, H, D, V, F32), workspace=chunked, **{**whole, "x": whole["x"][at : at + n], "state": state, "tops": tops, "spans": table((0, 0, n, at))})
            o = got["o"].astype(np.float64)
            under = np.maximum(np.abs(o[:, H * V : H * V + H]), np.exp(-o[:, H * V + H :])) + 1e-6
            y = o[:, : H * V].reshape(n, H, V) / under[:, :, None]
            assert np.abs(y - want[at : at + n]).max() <= 2e-4 * np.abs(want).max(), (sizes[:3], at)   # (a quotient by what may be small)
            state, tops, at = got["state"], got["tops"], at + n


@TOKENS
def test_a_memory_over_many_chunks(cuda, chunked):
    """More chunks than a launch composes at once, requests of several portions' length side by side."""
    rng = np.random.default_rng(9)
    spans = table((0, 5, 1500, 0), (2, 1505, 1100, 33), slots=3)
    op = memory_op(3, 2700, 1, 20, 24, F32)
    agrees(op, memory_inputs(rng, op, spans), 1e-4, rows_of(spans), workspace=chunked)


@BOTH
@pytest.mark.parametrize("H,V", [(2, 40), (3, 9), (4, 256), (1, 600)])
def test_memory_gates(cuda, dtype, H, V):
    rng = np.random.default_rng(V)
    o = rng.standard_normal((7, H * (V + 2))).astype(F32)
    o[0, H * V] = 0.0   # nothing in the denominator but its floor
    op = MemoryGate(rows=7, heads=H, dim=V, gate_width=H * V + 32, gate_at=24, epsilon=1e-3, dtype=dtype)
    agrees(op, dict(o=o, gate=bf(rng, 7, H * V + 32), gain=bf(rng, H * V)), 3e-6 if dtype is F32 else 5e-3)


# ---------------------------------------------------------------- experts


@BOTH
@pytest.mark.parametrize("rows,cols,experts,top", [(5, 128, 13, 3), (300, 96, 7, 7), (1, 60, 1, 1), (9, 37, 130, 11), (4, 2048, 64, 8)])
def test_a_router(cuda, dtype, rows, cols, experts, top):
    rng = np.random.default_rng(cols)
    given = dict(h=bf(rng, rows, cols), weight=bf(rng, experts, cols, scale=2 / np.sqrt(cols)), bias=bf(rng, experts))
    op = Router(rows=rows, cols=cols, experts=experts, top=top, dtype=dtype)
    want, got = op._call_reference(given), ran(op, **given)
    assert np.array_equal(got["ids"], want["ids"]) and np.abs(got["shares"] - want["shares"]).max() < 1e-5
    # equal logits: the first ones
    given |= dict(weight=np.zeros((experts, cols), F32), bias=np.ones(experts, F32))
    got = ran(op, **given)
    assert np.array_equal(got["ids"], np.tile(np.arange(top), (rows, 1))) and np.allclose(got["shares"], 1 / top)


@BOTH
@pytest.mark.parametrize("rows,cols,ff,experts,top", [(5, 128, 80, 11, 2), (300, 96, 64, 7, 2), (1, 60, 21, 1, 1), (9, 37, 10, 5, 5), (200, 256, 128, 16, 4),
                                                      (700, 192, 320, 3, 1), (130, 256, 104, 40, 3), (1000, 64, 72, 6, 2), (1100, 24, 9, 64, 60)])
def test_routed_feed_forwards(cuda, dtype, rows, cols, ff, experts, top):
    rng = np.random.default_rng(ff)
    ids = np.stack([rng.permutation(experts)[:top] for _ in range(rows)]).astype(np.int32)
    if rows > 100:   # uneven: most rows choose the last expert, and one expert nobody does
        ids[: rows // 2, 0] = experts - 1
        ids[: rows // 2, 1:] = np.arange(top - 1)
        ids[ids == 1] = 0 if top == 1 else ids[ids == 1]
    shares = rng.dirichlet(np.ones(top), rows).astype(F32)
    given = dict(h=bf(rng, rows, cols), gate=bf(rng, experts * ff, cols, scale=1 / np.sqrt(cols)), up=bf(rng, experts * ff, cols, scale=1 / np.sqrt(cols)),
                 down=bf(rng, experts * cols, ff, scale=1 / np.sqrt(ff)), ids=ids, shares=shares)
    for kind in ("silu", "gelu_tanh"):
        op = Experts(rows=rows, cols=cols, experts=experts, top=top, ff=ff, activation=kind, dtype=dtype)
        agrees(op, given, 5e-6 if dtype is F32 else 1e-2, workspace=True)


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
    model, plain = built(name, Tilarax, activations=F32 if dtype == "f32" else BF16, slots=3, max_seq_len=400, prefill_chunk=128)
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
    model, plain = built("mixed", Tilarax, slots=1, max_seq_len=700, prefill_chunk=64, activations=F32)
    model.load_versions()
    tokens = tokens_of(model, 640)
    want = plain(tokens)
    model.batch.step([Entry("x", tokens[:40])])
    rows = np.concatenate([model.batch.step([Entry("x", [t], [0])])[0] for t in tokens[40:]])
    model.release()
    assert off_by(rows, want[40:], LIMIT["f32"]) < LIMIT["f32"]


@pytest.mark.parametrize("name", MODELS)
def test_a_single_slot_s_steps(cuda, name):
    """One slot: a decode step's projections are single-row products."""
    model, plain = built(name, Tilarax, slots=1, max_seq_len=300, prefill_chunk=96)
    model.load_versions()
    try:
        assert "stream_depth_rows" in {f.kind for f in model.decode_step._fused.values()}
        assert "stream_depth_rows" in {f.kind for f in model.prompt_chunk._fused.values()}
        tokens = tokens_of(model, 200)
        want = plain(tokens)
        rows = [model.batch.step([Entry("x", tokens[:60], range(60))])[0]]
        rows += [model.batch.step([Entry("x", [t], [0])])[0] for t in tokens[60:]]
        assert off_by(np.concatenate(rows), want, LIMIT["bf16"]) < LIMIT["bf16"]
    finally:
        model.release()


def test_generation_replays_what_stepwise_decoding_draws(cuda):
    model, plain = built("mixed", Tilarax, slots=3, max_seq_len=200, prefill_chunk=32)
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
    captured, _ = built("wide", Tilarax, slots=slots, max_seq_len=120, prefill_chunk=32)
    eager, _ = built("wide", Tilarax, slots=slots, max_seq_len=120, prefill_chunk=32)
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
    write_safetensors(folder / "model.safetensors", weights_of(TilaraxConfig.from_json(doc)))
    return doc


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_a_trace_is_replayed(cuda, tmp_path, dtype):
    doc = saved(tmp_path, "odd")
    _, plain = built("odd", Tilarax)
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
    model = Tilarax.load(tmp_path, slots=2, max_seq_len=64)
    try:
        assert printed == model.generate_batch(prompts, 9)
    finally:
        model.release()
