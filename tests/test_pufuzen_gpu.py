"""Pufuzen's mechanisms and models on the GPU against the oracle and the plain implementation: each kernel
alone, prompts, portions, batches, slots used again, far keys, window edges, sinks, long decoding, generation."""

import json
import subprocess
import sys
from pathlib import Path

import numpy as np
import pytest
import torch

import oracle
from iron_amd import kernels as K
from iron_amd.applications import Pufuzen, PufuzenConfig
from iron_amd.bf16 import bfloat16, from_torch, round_bf16
from iron_amd.lm import Sampler, rope_angles, write_safetensors
from iron_amd.lm.batched import Entry
from iron_amd.operators.mha_latent import EVERYTHING, LatentMHA, LatentRows
from iron_amd.operators.recurrent import MinGRU
from iron_amd.operators.stream import PolyNorm, Softcap, StreamGatedAdd, StreamNorm
from tests.operator_support import agrees, bf, device, ran, rows_of, table, tolerance
from tests.pufuzen_plain import attention, min_gru, turned
from tests.pufuzen_support import MODELS, built, far_off, weights_of

pytestmark = pytest.mark.gpu
oracle.install()
F32, BF16 = np.float32, bfloat16
BOTH = pytest.mark.parametrize("dtype", [F32, BF16], ids=["f32", "bf16"])


# ---------------------------------------------------------------- the stream


@BOTH
@pytest.mark.parametrize("rows,cols,width,at", [(5, 128, 400, 136), (3, 60, 130, 61), (2, 2056, 4120, 2064), (3, 4160, 4160, 0), (1, 1303, 1400, 7),
                                                (1, 9000, 9008, 8)])
def test_a_gated_row_joins_the_stream(cuda, dtype, rows, cols, width, at):
    rng = np.random.default_rng(cols)
    x, y = rng.standard_normal((rows, cols)).astype(F32) * 3, bf(rng, rows, cols)
    gate, gate_bias, y_bias, gain = bf(rng, rows, width, scale=2), bf(rng, cols), bf(rng, cols), bf(rng, cols)
    for bias in (None, y_bias):
        op = StreamGatedAdd(rows=rows, cols=cols, gate_width=width, gate_at=at, biased=bias is not None, dtype=dtype)
        added = agrees(op, dict(x=x, y=y, gate=gate, gate_bias=gate_bias) | ({} if bias is None else {"y_bias": bias}), 2e-6)["x"]
        # with the norm behind it in one launch: the two, bit for bit
        xd, hd = device(x, F32), torch.empty((rows, cols), dtype=torch.bfloat16 if dtype is BF16 else torch.float32, device="cuda")
        K.stream_gated_rows(xd, device(y, dtype), device(gate, dtype), device(gate_bias, BF16), rows=rows, cols=cols, eps=1e-3, gate_stride=width,
                            gate_at=at, y_bias=None if bias is None else device(bias, BF16), h=hd, gain=device(gain, BF16))
        want = ran(StreamNorm(rows=rows, cols=cols, epsilon=1e-3, dtype=dtype), x=added, weight=gain)["y"]
        assert np.array_equal(from_torch(xd), added) and np.array_equal(from_torch(hd), want)


@BOTH
@pytest.mark.parametrize("rows,cols,stride,at", [(4, 96, 160, 0), (3, 37, 97, 5), (2, 2048, 4096, 2048), (2, 3000, 3000, 0), (1, 8200, 8208, 8), (1, 9001, 9001, 0)])
def test_a_polynomial_of_normed_powers(cuda, dtype, rows, cols, stride, at):
    rng = np.random.default_rng(cols)
    x, bias = bf(rng, rows, stride, scale=1.5), bf(rng, cols)
    x[0, at + cols // 2] = 24.0   # a column whose cube stands out
    for coefficients in ([0.5, -1.25, 0.75, 0.25], [0.0, 0.0, 1.0, 0.0], [0.0, 1.0, 0.0, -2.0]):
        for given in ({}, {"bias": bias}):
            op = PolyNorm(rows=rows, cols=cols, stride=stride, at=at, epsilon=1e-2, biased=bool(given), dtype=dtype)
            agrees(op, dict(x=x, coefficients=np.array(coefficients), **given), 3e-6 if dtype is F32 else 5e-3)


@BOTH
def test_a_scaled_head(cuda, dtype):
    rng = np.random.default_rng(5)
    x = bf(rng, 3, 77, scale=4)
    for cap, scale in ((0.0, 2.5), (9.0, 0.3)):
        op = Softcap(rows=3, cols=77, cap=cap, scale=scale, dtype=dtype)
        got = ran(op, x=x)
        want = x * scale if not cap else cap * np.tanh(x * scale / cap)
        assert np.abs(got["y"] - want).max() < 1e-5 * np.abs(want).max()


# ---------------------------------------------------------------- the recurrence


def gru_inputs(rng, op, spans):
    x = bf(rng, op.rows, op.stride, scale=1.5)
    return dict(x=x, z_bias=round_bf16(rng.uniform(-6, 2, op.width).astype(F32)), x_bias=bf(rng, op.width),
                state=rng.standard_normal((op.slots, 2, op.width)).astype(F32), spans=spans)


@BOTH
@pytest.mark.parametrize("chunked", [False, True], ids=["tokens", "chunks"])
@pytest.mark.parametrize("width,stride", [(64, 256), (33, 120), (514, 1600), (700, 2101)])
def test_a_gated_recurrence(cuda, dtype, chunked, width, stride):
    rng = np.random.default_rng(width)
    # lengths around a chunk's, rows out of slot order, a slot that goes on and one that starts over
    spans = table((0, 130, 33, 9), (1, 0, 32, 0), (2, 32, 1, 3), (4, 33, 97, 0), slots=6)
    op = MinGRU(slots=6, rows=170, stride=stride, width=width, dtype=dtype)
    agrees(op, gru_inputs(rng, op, spans), 3e-6 if dtype is F32 else 5e-3, rows_of(spans), workspace=chunked)


@pytest.mark.parametrize("chunked", [False, True], ids=["tokens", "chunks"])
def test_the_recurrence_goes_on_where_a_portion_ends(cuda, chunked):
    rng = np.random.default_rng(7)
    width = 48
    op = MinGRU(slots=1, rows=200, stride=3 * width, width=width, dtype=F32)
    whole = gru_inputs(rng, op, table((0, 0, 200, 0)))
    x = whole["x"].astype(np.float64)
    g = x[:, 2 * width :]
    want = min_gru(x[:, :width] + whole["z_bias"], x[:, width : 2 * width] + whole["x_bias"]) * g / (1 + np.exp(-g))
    state, at = whole["state"], 0
    for n in (2, 31, 1, 70, 33, 2, 61):
        op = MinGRU(slots=1, rows=n, stride=3 * width, width=width, dtype=F32)
        got = ran(op, workspace=chunked, **{**whole, "x": whole["x"][at : at + n], "state": state, "spans": table((0, 0, n, at))})
        assert np.abs(got["y"] - want[at : at + n]).max() <= 3e-6 * np.abs(want).max(), at
        state, at = got["state"], at + n
    assert at == 200


# ---------------------------------------------------------------- latent attention

# heads, dim, rot, vdim, rank, window (None: everything), a sink
SIZES = [(4, 40, 32, 56, 72, None, True), (3, 24, 0, 80, 40, 37, False), (17, 16, 32, 24, 128, None, True), (1, 64, 64, 64, 512, None, False),
         (2, 128, 64, 128, 320, 130, True), (2, 200, 0, 160, 96, 65, False), (5, 11, 6, 7, 19, None, True), (3, 12, 0, 20, 9, 1, False),
         (2, 128, 64, 128, 320, None, True), (3, 128, 0, 128, 64, None, False),
         (6, 8, 40, 256, 24, 9, True), (16, 96, 32, 64, 256, 64, False)]
ids_of = lambda p: "x".join(map(str, p))  # noqa: E731


def latent_case(rng, H, D, rot, V, R, window, T, sunk, quiet=False):
    """A sequence's q rows, latents and shared key parts (unturned), and expansions under which chosen queries
    meet a latent that stands out far back, just inside their window and, more so, just outside -- or, ``quiet``,
    no key that stands out among the hundreds that all count."""
    q, c, r = bf(rng, T, H * (D + rot), scale=1.0 if quiet else 0.4), bf(rng, T, R), bf(rng, T, rot, scale=0.5)
    up = bf(rng, H * (D + V), R, scale=1 / np.sqrt(R))
    U = up[: H * D].reshape(H, D, R).astype(np.float64)
    loud = []
    for i in range(T if quiet else min(T - 1, 40), T, 11):
        h = i % H
        toward = np.einsum("d,dr->r", q[i].reshape(H, D + rot)[h, :D].astype(np.float64), U[h])
        toward = toward / max(np.linalg.norm(toward), 1e-6)
        back = (window - 1 if window else i // 3)
        if back <= i:
            loud.append((i - back, 4 * np.sqrt(R) * toward))
        if window and window <= i:
            loud.append((i - window, 8 * np.sqrt(R) * toward))
    for j, row in loud:
        c[j] = round_bf16(row.astype(F32))
    sink = round_bf16(rng.uniform(-2, 4, H).astype(F32)) if sunk else None
    return q, c, r, up, sink


def plain_latent(q, c, r, up, sink, H, D, rot, V, R, window, scale, base):
    T = len(q)
    q = q.astype(np.float64).reshape(T, H, D + rot)
    k, v = (c @ up[: H * D].T.astype(np.float64)).reshape(T, H, D), (c @ up[H * D :].T.astype(np.float64)).reshape(T, H, V)
    if rot:
        q = np.concatenate([q[..., :D], turned(q[..., D:], base, rot)], axis=-1)
        k = np.concatenate([k, np.repeat(turned(r, base, rot)[:, None], H, axis=1)], axis=-1)
    return attention(q, k, v, scale=scale, window=window, sink=None if sink is None else sink.astype(np.float64)).reshape(T, -1)


def ring_rows(held, ring, values, first):
    """``values`` at positions ``first ..`` of a ring's slot."""
    held[np.arange(first, first + len(values)) % ring] = values


@BOTH
@pytest.mark.parametrize("quiet", [False, True], ids=["loud", "quiet"])
@pytest.mark.parametrize("case", SIZES, ids=ids_of)
def test_latent_attention_in_portions_and_steps(cuda, dtype, case, quiet):
    H, D, rot, V, R, window, sunk = case
    rng = np.random.default_rng(R)
    T, base, scale = 190, 300.0, (1.0 if quiet else 1.5) / np.sqrt(D + rot)
    q, c, r, up, sink = latent_case(rng, H, D, rot, V, R, window, T, sunk, quiet)
    want = plain_latent(q, c, r, up, sink, *case[:5], window, scale, base)
    angles = rope_angles(rot, T, base) if rot else None
    r = turned(r, base, rot) if rot else r
    r = round_bf16(r.astype(F32)) if dtype is BF16 else r.astype(F32)
    limit = (3e-5 if dtype is F32 else 2e-2) * np.abs(want).max()
    for sizes in ([T], [64, 1, 1, 2, T - 68], [T // 2] + [1] * 30):
        ring = min(T, (window or T) + max(sizes))
        latents, keys = np.full((2, ring, R), 5.0, F32), np.full((2, ring, rot), 5.0, F32)   # what a slot held before is nobody's
        got, at = [], 0
        for n in sizes:
            ring_rows(latents[1], ring, c[at : at + n], at)
            given = dict(q=np.concatenate([np.full((3, q.shape[1]), 9.0), q[at : at + n]]), latents=latents, up=up, spans=table((1, 3, n, at), slots=2))
            if rot:
                ring_rows(keys[1], ring, r[at : at + n], at)
                given |= dict(shared_keys=keys, angles=angles)
            op = LatentMHA(slots=2, rows=n + 3, heads=H, dim=D, rot=rot, vdim=V, rank=R, turned=rot, angle_rows=T if rot else 0, sunk=sunk,
                           window=window or EVERYTHING, ring=ring, cap=T + 3, scale=scale, single=n == 1, dtype=dtype)
            y = ran(op, workspace=True, **given, **({"sink": sink} if sunk else {}))["y"]
            assert (y[:3] == 7).all()   # the sequence is not the batch's first rows
            got.append(y[3:])
            at += n
        got = np.concatenate(got)
        assert np.isfinite(got).all() and np.abs(got - want[:at]).max() <= limit, (sizes, np.abs(got - want[:at]).max(), limit)


@BOTH
@pytest.mark.parametrize("case", [SIZES[0], SIZES[1], SIZES[6]], ids=ids_of)
def test_latent_attention_over_several_requests(cuda, dtype, case):
    """Rows out of slot order, a request that goes on, keys in all beyond any one's."""
    H, D, rot, V, R, window, sunk = case
    rng = np.random.default_rng(3)
    base, scale = 1e4, 1 / np.sqrt(D + rot)
    spans = table((0, 60, 130, 0), (2, 2, 1, 40), (3, 3, 57, 100), slots=5)
    ring = 260
    latents, keys, q = np.zeros((5, ring, R), F32), np.zeros((5, ring, rot), F32), np.full((200, H * (D + rot)), 3.0, F32)
    want, up, sink = {}, None, None
    for slot, row, n, start in ((0, 60, 130, 0), (2, 2, 1, 40), (3, 3, 57, 100)):
        qs, c, r, u, k = latent_case(rng, H, D, rot, V, R, window, start + n, sunk)
        up, sink = (u, k) if up is None else (up, sink)
        want[slot] = plain_latent(qs, c, r, up, sink, *case[:5], window, scale, base)[start:]
        latents[slot, : start + n] = c
        keys[slot, : start + n] = round_bf16(turned(r, base, rot).astype(F32)) if rot and dtype is BF16 else turned(r, base, rot) if rot else r
        q[row : row + n] = qs[start:]
    given = dict(q=q, latents=latents, up=up, spans=spans) | (dict(shared_keys=keys, angles=rope_angles(rot, 200, base)) if rot else {})
    op = LatentMHA(slots=5, rows=200, heads=H, dim=D, rot=rot, vdim=V, rank=R, turned=rot, angle_rows=200 if rot else 0, sunk=sunk,
                   window=window or EVERYTHING, ring=ring, cap=330, scale=scale, dtype=dtype)
    y = ran(op, workspace=True, **given, **({"sink": sink} if sunk else {}))["y"]
    for slot, row, n in ((0, 60, 130), (2, 2, 1), (3, 3, 57)):
        assert np.abs(y[row : row + n] - want[slot]).max() <= (3e-5 if dtype is F32 else 2e-2) * np.abs(want[slot]).max(), slot
    assert (y[:2] == 7).all() and (y[190:] == 7).all()


@BOTH
@pytest.mark.parametrize("q_rank,rank,rot,turn", [(64, 40, 16, 16), (13, 19, 6, 4), (96, 512, 0, 0), (300, 64, 64, 32)])
def test_latent_rows(cuda, dtype, q_rank, rank, rot, turn):
    rng = np.random.default_rng(rank)
    stride = q_rank + rank + rot + 24
    spans = table((0, 30, 40, 60), (1, 3, 1, 7), (3, 4, 26, 0), slots=4)   # one whose rows wrap around the ring
    op = LatentRows(slots=4, rows=72, stride=stride, q_rank=q_rank, rank=rank, rot=rot, turned=turn, angle_rows=128 if turn else 0, ring=64,
                    epsilon=1e-3, dtype=dtype)
    given = dict(x=bf(rng, 72, stride), q_gain=bf(rng, q_rank), c_gain=bf(rng, rank), spans=spans, latents=bf(rng, 4, 64, rank))
    given |= {"shared_keys": bf(rng, 4, 64, rot)} if rot else {}
    given |= {"angles": rope_angles(turn, 128, 400.0)} if turn else {}
    agrees(op, given, 3e-6 if dtype is F32 else 5e-3, rows_of(spans))


def test_a_long_step_over_many_splits(cuda):
    """A step far from the sequence's start: every split of the keys has several tiles, and the loudest key is in
    the first, a middle or the last one."""
    H, D, rot, V, R, T = 20, 32, 16, 32, 192, 6000
    rng = np.random.default_rng(1)
    up, q = bf(rng, H * (D + V), R, scale=1 / np.sqrt(R)), bf(rng, 1, H * (D + rot))
    for loud in (0, 2999, T - 1):
        c = bf(rng, 1, T, R, scale=0.5)
        toward = q.reshape(H, D + rot)[3, :D] @ up[: H * D].reshape(H, D, R)[3]
        c[0, loud] = round_bf16((4 * np.sqrt(R) * toward / np.linalg.norm(toward)).astype(F32))
        keys = bf(rng, 1, T, rot)
        for dtype in (F32, BF16):
            op = LatentMHA(slots=1, rows=1, heads=H, dim=D, rot=rot, vdim=V, rank=R, turned=rot, angle_rows=T, sunk=False, ring=T, scale=0.2,
                           single=True, dtype=dtype)
            agrees(op, dict(q=q, latents=c, up=up, spans=table((0, 0, 1, T - 1)), shared_keys=keys, angles=rope_angles(rot, T)),
                   3e-5 if dtype is F32 else 1.5e-2, workspace=True)


# ---------------------------------------------------------------- a row's product in one launch


def row_product(rng, M, K_):
    return bf(rng, M, K_, scale=1 / np.sqrt(K_)), bf(rng, M), bf(rng, M + 8, scale=2), bf(rng, M), rng.standard_normal(M).astype(F32)


@pytest.mark.parametrize("M,K_", [(70, 64), (2100, 512), (33, 2056), (40, 5000), (12, 14336)])
def test_a_normed_row_s_product(cuda, M, K_):
    rng = np.random.default_rng(M)
    W, *_ = row_product(rng, M, K_)
    gain = bf(rng, K_)
    for kind, x in (("stream_norm", rng.standard_normal(K_).astype(F32) * 3), ("row_norm", bf(rng, K_)), ("row", bf(rng, K_))):
        y = torch.empty(M, dtype=torch.bfloat16, device="cuda")
        K.stream_product(device(W, BF16), device(x, F32 if kind == "stream_norm" else BF16), input=kind, M=M, K=K_, y=y, eps=1e-3,
                         gain=None if kind == "row" else device(gain, BF16))
        h = x if kind == "row" else round_bf16((x / np.sqrt((x.astype(np.float64) ** 2).mean() + 1e-3) * gain).astype(F32))
        want = W.astype(np.float64) @ h
        assert np.abs(from_torch(y) - want).max() <= 6e-3 * np.abs(want).max(), kind


@pytest.mark.parametrize("M,K_", [(70, 64), (2100, 512), (33, 2056), (40, 5000), (12, 14336)])
def test_a_row_s_product_joins_the_stream(cuda, M, K_):
    rng = np.random.default_rng(M + 1)
    W, y_bias, gate, gate_bias, stream = row_product(rng, M, K_)
    x, b0, b1, coefficients = bf(rng, 3 * K_, scale=1.5), bf(rng, K_), bf(rng, K_), round_bf16(np.array([0.5, -1.25, 0.75, 0.25], F32))
    opened = 1 / (1 + np.exp(-(gate[:M].astype(np.float64) + gate_bias)))
    z = x[:K_].astype(np.float64) + b0
    for start in (0, 5, 6):
        state = rng.standard_normal((2, K_)).astype(F32)
        held = None if start == 0 else state[(start - 1) % 2][None]
        S = min_gru(x[None, :K_].astype(np.float64) + b0, x[None, K_ : 2 * K_].astype(np.float64) + b1, None if held is None else held[0])[0]
        g = x[2 * K_ :].astype(np.float64)
        made = {"row": x[:K_], "min_gru": S * g / (1 + np.exp(-g)),
                "poly_norm": sum(c * z**n / np.sqrt((z ** (2 * n)).mean() + 1e-2) for c, n in zip(coefficients.astype(np.float64), (1, 2, 3))) + coefficients[3]}
        for kind, h in made.items():
            given = {} if kind == "row" else dict(b0=device(b0, BF16))
            if kind == "min_gru":
                given |= dict(b1=device(b1, BF16), state=device(state, F32), spans=device(table((0, 0, 1, start)), np.int32))
            if kind == "poly_norm":
                given |= dict(gain=device(coefficients, BF16), eps=1e-2)
            for bias in (None, y_bias):
                row = device(stream, F32)
                K.stream_product(device(W, BF16), device(x if kind == "min_gru" else x[:K_], BF16), input=kind, M=M, K=K_, stream=row,
                                 gate=device(gate, BF16), gate_bias=device(gate_bias, BF16), y_bias=None if bias is None else device(bias, BF16), **given)
                want = stream + (W.astype(np.float64) @ h + (0 if bias is None else bias)) * opened
                assert np.abs(from_torch(row) - want).max() <= 8e-3 * np.abs(want).max(), (kind, start)
            if kind == "min_gru":   # the new state beside the old one, which is left
                new = from_torch(given["state"]).reshape(2, K_)
                assert np.array_equal(new[(start - 1) % 2], state[(start - 1) % 2]) and np.abs(new[start % 2] - S).max() <= 1e-5 * np.abs(S).max()


# ---------------------------------------------------------------- whole models


LIMIT = {"f32": 1e-5, "bf16": 6e-2}   # of the logits' spread


@pytest.fixture(scope="module", params=[(n, d, f) for n in MODELS for d in ("f32", "bf16") for f in ((True, False) if d == "bf16" else (True,))],
                ids=lambda p: f"{p[0]}-{p[1]}-{'fused' if p[2] else 'steps'}")
def served(request):
    name, dtype, fuse = request.param
    model, plain = built(name, Pufuzen, activations=F32 if dtype == "f32" else BF16, slots=3, max_seq_len=400, prefill_chunk=128)
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
        off = far_off(np.concatenate(rows), want, want.std())
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
            assert far_off(np.concatenate(rows[k]), want[k], want[k].std()) < limit, (order, k)
            model.batch.end(k)


def test_a_portion_s_keys_have_a_room(cuda):
    """More keys than a portion may attend: requests wait for the next launch, and nothing changes."""
    model, plain = built("mixed", Pufuzen, slots=3, max_seq_len=100, prefill_chunk=12, activations=F32)
    assert model.config.key_room == 100
    model.load_versions()
    try:
        prompts = {k: tokens_of(model, n, seed=n) for k, n in (("a", 90), ("b", 95), ("c", 70))}
        rows = {k: [] for k in prompts}
        for lo, hi in ((0, 50), (50, 58), (58, 100)):
            live = [k for k in prompts if lo < len(prompts[k])]
            got = model.batch.step([Entry(k, prompts[k][lo:hi], range(len(prompts[k][lo:hi]))) for k in live])
            for k, r in zip(live, got):
                rows[k].append(r)
        for k, t in prompts.items():
            want = plain(t)
            assert far_off(np.concatenate(rows[k]), want, want.std()) < LIMIT["f32"], k
    finally:
        model.release()


def test_long_decoding(cuda):
    model, plain = built("mixed", Pufuzen, slots=1, max_seq_len=700, prefill_chunk=64, activations=F32)
    model.load_versions()
    tokens = tokens_of(model, 640)
    want = plain(tokens)
    model.batch.step([Entry("x", tokens[:40])])
    rows = np.concatenate([model.batch.step([Entry("x", [t], [0])])[0] for t in tokens[40:]])
    model.release()
    assert far_off(rows, want[40:], want.std()) < LIMIT["f32"]


@pytest.mark.parametrize("name", MODELS)
def test_a_single_slot_s_steps(cuda, name):
    """One slot: a decode step's projections are single-row products, with what makes their inputs and takes their
    outputs in the same launches where the sizes allow it."""
    model, plain = built(name, Pufuzen, slots=1, max_seq_len=300, prefill_chunk=96)
    model.load_versions()
    try:
        kinds = {f.kind for f in model.decode_step._fused.values()}
        if name != "odd":
            assert {"stream_norm_gemv", "min_gru_gated_product", "poly_norm_gated_product", "gated_product", "latent_query"} <= kinds
            assert "stream_gated_add_norm" in {f.kind for f in model.prompt_chunk._fused.values()}
        tokens = tokens_of(model, 200)
        want = plain(tokens)
        rows = [model.batch.step([Entry("x", tokens[:60], range(60))])[0]]
        rows += [model.batch.step([Entry("x", [t], [0])])[0] for t in tokens[60:]]
        assert far_off(np.concatenate(rows), want, want.std()) < LIMIT["bf16"]
    finally:
        model.release()


def test_generation_replays_what_stepwise_decoding_draws(cuda):
    model, plain = built("mixed", Pufuzen, slots=3, max_seq_len=200, prefill_chunk=32)
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
    captured, _ = built("wide", Pufuzen, slots=slots, max_seq_len=120, prefill_chunk=32)
    eager, _ = built("wide", Pufuzen, slots=slots, max_seq_len=120, prefill_chunk=32)
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
    write_safetensors(folder / "model.safetensors", weights_of(PufuzenConfig.from_json(doc)))
    return doc


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_a_trace_is_replayed(cuda, tmp_path, dtype):
    doc = saved(tmp_path, "odd")
    _, plain = built("odd", Pufuzen)
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
        assert far_off(rows, want[places], want.std()) < LIMIT["f32" if dtype == "float32" else "bf16"]
    assert not (tmp_path / "1.f32").exists()


def test_the_command_line_generates_a_batch(cuda, tmp_path, capsys):
    from iron_amd.__main__ import main

    doc = saved(tmp_path, "mixed")
    prompts = [np.random.default_rng(n).integers(0, doc["vocab"], n).tolist() for n in (11, 4)]
    asked = [a for p in prompts for a in ("--ids", ",".join(map(str, p)))]
    assert main([str(tmp_path), *asked, "--count", "9", "--max-seq-len", "64"]) == 0
    printed = [[int(t) for t in line.split(",")] for line in capsys.readouterr().out.splitlines()]
    model = Pufuzen.load(tmp_path, slots=2, max_seq_len=64)
    try:
        assert printed == model.generate_batch(prompts, 9)
    finally:
        model.release()
