"""Pegilix's mechanisms and models on the GPU against the oracle and the plain implementation: each kernel
alone, prompts, portions, batches, slots used again, far keys, window edges, long decoding, generation."""

import json
import subprocess
import sys
from pathlib import Path

import numpy as np
import pytest
import torch

import oracle
from iron_amd import kernels as K
from iron_amd.applications import Pegilix
from iron_amd.bf16 import bfloat16, from_torch, round_bf16
from iron_amd.lm import Sampler, write_safetensors
from iron_amd.lm.batched import Entry
from iron_amd.operators.mha_window import WindowMHA
from iron_amd.operators.recurrent import DeltaRule, HeadGate, LowRankDecay, ShortConv, TimeMix, TokenShift
from iron_amd.operators.sample import Sample, SampleSlots, draw_row
from iron_amd.operators.stream import GatedProduct, LinearAny, Softcap, SpanTails, StreamAdd, StreamEmbed, StreamNorm
from tests.operator_support import agrees, bf, device, ran, rows_of, table, tolerance
from tests.pegilix_plain import window_attention
from tests.pegilix_support import MODELS, built, far_off, weights_of

pytestmark = pytest.mark.gpu
oracle.install()
F32, BF16 = np.float32, bfloat16
BOTH = pytest.mark.parametrize("dtype", [F32, BF16], ids=["f32", "bf16"])


# ---------------------------------------------------------------- the stream


@BOTH
@pytest.mark.parametrize("rows,cols", [(5, 128), (3, 60), (2, 2056), (3, 4160), (1, 1303), (1, 9000)])
def test_the_stream(cuda, dtype, rows, cols):
    rng = np.random.default_rng(cols)
    x, y = rng.standard_normal((rows, cols)).astype(F32) * 3, bf(rng, rows, cols)
    gain, back = bf(rng, cols), bf(rng, cols)
    agrees(StreamNorm(rows=rows, cols=cols, epsilon=1e-3, dtype=dtype), dict(x=x, weight=gain), tolerance(dtype))
    added = agrees(StreamAdd(rows=rows, cols=cols, epsilon=1e-3, dtype=dtype), dict(x=x, y=y, weight=back), 2e-6)["x"]
    # both in one launch are the two, bit for bit
    xd, hd = device(x, F32), torch.empty((rows, cols), dtype=torch.bfloat16 if dtype is BF16 else torch.float32, device="cuda")
    K.stream_rows(xd, rows=rows, cols=cols, eps=1e-3, y=device(y, dtype), back_gain=device(back, BF16), h=hd, gain=device(gain, BF16))
    want = ran(StreamNorm(rows=rows, cols=cols, epsilon=1e-3, dtype=dtype), x=added, weight=gain)["y"]
    assert np.array_equal(from_torch(xd), added) and np.array_equal(from_torch(hd), want)


@BOTH
def test_the_ends_of_the_stream(cuda, dtype):
    rng = np.random.default_rng(3)
    for cols in (96, 77):
        ids = rng.integers(0, 40, 6).astype(np.int32)
        agrees(StreamEmbed(rows=6, table_rows=40, cols=cols), dict(table=bf(rng, 40, cols), ids=ids), 0)
        x = rng.standard_normal((9, cols)).astype(F32)
        spans = table((2, 0, 4, 7), (0, 4, 5, 0), slots=4)
        got = ran(SpanTails(slots=4, rows=9, cols=cols), x=x, spans=spans)["y"]
        assert np.array_equal(got[2], x[3]) and np.array_equal(got[0], x[8]) and (got[[1, 3]] == 7).all()
        for cap in (0.0, 12.0):
            op = Softcap(rows=3, cols=cols, cap=cap, dtype=dtype)
            logits = bf(rng, 3, cols, scale=15)
            want, got = op._call_reference(dict(x=logits)), ran(op, x=logits)
            assert np.abs(got["y"] - want["y"]).max() < 1e-5 * 15
            assert np.abs(got["rounded"][:, :cols] - want["rounded"][:, :cols]).max() <= 0.13   # one bf16 step at 30
        if dtype is F32:
            for act in ("relu", "silu", "gelu_tanh"):
                agrees(GatedProduct(rows=4, cols=cols, activation=act),
                       dict(gate=rng.standard_normal((4, cols)), up=rng.standard_normal((4, cols))), 2e-6)


@BOTH
@pytest.mark.parametrize("rows,n,k", [(1, 7, 5), (70, 130, 60), (3, 64, 100), (129, 33, 17)])
def test_a_product_of_any_sizes(cuda, dtype, rows, n, k):
    rng = np.random.default_rng(n)
    agrees(LinearAny(rows=rows, n=n, k=k, dtype=dtype), dict(x=bf(rng, rows, k), weight=bf(rng, n, k)), 4e-6 if dtype is F32 else 5e-3)


@pytest.mark.parametrize("M,N,K_", [(1, 16, 8), (3, 50, 520), (16, 129, 1032), (17, 640, 64), (33, 48, 4096), (63, 257, 200), (8, 2048, 2048)])
def test_a_product_over_few_rows(cuda, M, N, K_):
    rng = np.random.default_rng(M)
    a, b, b2 = bf(rng, M, K_), bf(rng, N, K_, scale=0.1), bf(rng, N, K_, scale=0.1)
    A, B, B2, C = (device(x, BF16) for x in (a, b, b2, np.zeros((M, N), F32)))
    K.gemm(A, B, C, M=M, N=N, K=K_, b_col_maj=True)
    want = a.astype(np.float64) @ b.T
    assert np.abs(from_torch(C) - want).max() <= 6e-3 * np.abs(want).max()
    for act, f in (("relu", lambda z: np.maximum(z, 0)), ("silu", lambda z: z / (1 + np.exp(-z)))):
        K.gemm_gated_pair(A, B, B2, torch.empty_like(C), C, M=M, N=N, K=K_, activation=act)
        gated = f(want) * (a.astype(np.float64) @ b2.T)
        assert np.abs(from_torch(C) - gated).max() <= 1.5e-2 * np.abs(gated).max(), act


# ---------------------------------------------------------------- recurrences


@BOTH
@pytest.mark.parametrize("cols", [64, 60, 2600])
def test_token_shift(cuda, dtype, cols):
    rng = np.random.default_rng(cols)
    spans = table((0, 3, 9, 0), (1, 12, 1, 6), (2, 0, 3, 5), slots=4)   # a new sequence, a single row, one that goes on
    op = TokenShift(slots=4, rows=20, cols=cols, mixes=5, dtype=dtype)
    inputs = dict(h=bf(rng, 20, cols), mu=bf(rng, 5, cols), carry=bf(rng, 4, 2, cols), spans=spans)
    want, got = op._call_reference(inputs), ran(op, **inputs)
    rows = rows_of(spans)
    assert np.abs(got["mixed"][:, rows] - want["mixed"][:, rows]).max() <= tolerance(dtype) * 4
    assert np.array_equal(got["carry"], want["carry"].astype(F32))


@BOTH
@pytest.mark.parametrize("n,rank", [(96, 16), (300, 5), (64, 64), (520, 24)])
def test_low_rank_decay(cuda, dtype, n, rank):
    rng = np.random.default_rng(n)
    agrees(LowRankDecay(rows=21, n=n, rank=rank, dtype=dtype),
           dict(z=bf(rng, 21, rank), up=bf(rng, n, rank, scale=0.3), base=bf(rng, n)), 2e-6)


def mix_inputs(rng, rows, heads, dim, slots, spans, quick=False):
    n = heads * dim
    decay = -np.exp(rng.uniform(-5, 4.5 if quick else 0, (rows, n))).astype(F32)   # quick: down to exp(-90) a step
    return dict(r=bf(rng, rows, n), k=bf(rng, rows, n), v=bf(rng, rows, n), log_decay=decay, u=bf(rng, heads, dim),
                state=rng.standard_normal((slots, heads, dim, dim)).astype(F32), spans=spans)


@BOTH
@pytest.mark.parametrize("chunked", [False, True], ids=["tokens", "chunks"])
@pytest.mark.parametrize("heads,dim", [(3, 32), (2, 64), (1, 20), (2, 128), (1, 256), (2, 100)])
def test_time_mixing(cuda, dtype, chunked, heads, dim):
    rng = np.random.default_rng(dim)
    # lengths around a chunk's, rows out of slot order, a slot that goes on and one that starts over
    spans = table((0, 50, 17, 9), (1, 0, 16, 0), (2, 16, 1, 3), (4, 17, 33, 0), slots=5)
    op = TimeMix(slots=5, rows=80, heads=heads, dim=dim, dtype=dtype)
    for quick in (False, True):
        agrees(op, mix_inputs(rng, 80, heads, dim, 5, spans, quick), 2e-5 if dtype is F32 else 2e-4, rows_of(spans), workspace=chunked)


@pytest.mark.parametrize("chunked", [False, True], ids=["tokens", "chunks"])
def test_time_mixing_goes_on_where_a_portion_ends(cuda, chunked):
    rng = np.random.default_rng(7)
    whole = mix_inputs(rng, 64, 2, 48, 1, table((0, 0, 64, 0)))
    want = ran(TimeMix(slots=1, rows=64, heads=2, dim=48, dtype=F32), workspace=False, **whole)["o"]
    state, at = whole["state"], 0
    for n in (2, 15, 1, 30, 16):
        part = {k: whole[k][at : at + n] for k in ("r", "k", "v", "log_decay")}
        op = TimeMix(slots=1, rows=n, heads=2, dim=48, dtype=F32)
        got = ran(op, workspace=chunked, **{**whole, **part, "state": state, "spans": table((0, 0, n, at))})
        assert np.abs(got["o"] - want[at : at + n]).max() <= 2e-5 * np.abs(want).max()
        state, at = got["state"], at + n


def conv_op(dtype, rows, slots, heads=4, kv_heads=2, dim=32, vdim=48, taps=4):
    channels = 2 * kv_heads * dim + heads * vdim
    return ShortConv(slots=slots, rows=rows, heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, taps=taps,
                     stride=channels + 11 + 2 * heads, b_at=channels + 11, a_at=channels + 11 + heads, dtype=dtype)


@BOTH
@pytest.mark.parametrize("shape", [dict(), dict(taps=2), dict(taps=1), dict(taps=9, dim=20, vdim=12), dict(taps=3, heads=3, kv_heads=1, dim=100, vdim=256)],
                         ids=str)
def test_short_convolution(cuda, dtype, shape):
    rng = np.random.default_rng(5)
    spans = table((0, 3, 40, 0), (1, 43, 1, 2), (3, 0, 3, 11), (2, 44, 2, 1), slots=5)
    op = conv_op(dtype, 50, 5, **shape)
    inputs = dict(x=bf(rng, 50, op.stride), weight=bf(rng, op.channels, op.taps), a_log=bf(rng, op.heads), dt_bias=bf(rng, op.heads),
                  state=bf(rng, 5, op.taps, op.channels), spans=spans)
    got = agrees(op, inputs, 2e-5, rows_of(spans))
    q = got["y"][rows_of(spans)][:, : op.dim].astype(np.float64)   # unit, over sqrt(dim)
    assert np.abs(np.linalg.norm(q, axis=1) * op.dim**0.5 - 1).max() < 1e-3


def delta_inputs(rng, op, spans, quick=False):
    x = rng.standard_normal((op.rows, op.wide)).astype(F32)
    G, D = op.kv_heads, op.dim
    qk = x[:, : 2 * G * D].reshape(op.rows, 2 * G, D)
    qk /= np.linalg.norm(qk, axis=-1, keepdims=True)
    x[:, op.channels : op.channels + op.heads] = -np.exp(rng.uniform(-6, 4 if quick else 0, (op.rows, op.heads)))
    x[:, op.channels + op.heads :] = rng.uniform(0.05, 0.98, (op.rows, op.heads))
    return dict(x=x, state=rng.standard_normal((op.slots, op.heads, op.dim, op.vdim)).astype(F32), spans=spans)


@pytest.mark.parametrize("chunked", [False, True], ids=["tokens", "chunks"])
@pytest.mark.parametrize("heads,kv_heads,dim,vdim", [(4, 2, 32, 32), (3, 1, 64, 48), (2, 2, 20, 12), (2, 1, 128, 64), (1, 1, 256, 256), (6, 3, 66, 20)])
def test_the_delta_rule(cuda, chunked, heads, kv_heads, dim, vdim):
    rng = np.random.default_rng(dim)
    spans = table((0, 50, 17, 9), (1, 0, 16, 0), (2, 16, 1, 3), (4, 17, 33, 0), slots=5)
    op = DeltaRule(slots=5, rows=80, heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim)
    for quick in (False, True):
        agrees(op, delta_inputs(rng, op, spans, quick), 4e-5, rows_of(spans), workspace=chunked)


def test_the_delta_rule_where_one_key_is_written_over_and_over(cuda):
    """The same key every token, full strength and hardly a decay: each write replaces the last, and an inverse
    of a chunk's 16 coupled updates that lost its exactness would show."""
    op = DeltaRule(slots=1, rows=48, heads=1, kv_heads=1, dim=64, vdim=32)
    rng = np.random.default_rng(2)
    inputs = delta_inputs(rng, op, table((0, 0, 48, 0)))
    x = inputs["x"]
    x[:, :64] = x[:, 64:128] = x[0, 64:128]
    x[:, op.channels], x[:, op.channels + 1] = -1e-4, 0.999
    got = agrees(op, inputs, 4e-5, workspace=True)["o"]
    assert np.abs(got[40] - x[40, 128:160]).max() < 2e-2   # the read-out sees the current token's write


@BOTH
@pytest.mark.parametrize("heads,dim,shared,at", [(3, 64, True, 0), (2, 20, False, 5), (2, 128, False, 32), (5, 256, True, 8), (1, 100, False, 4)])
def test_head_norm_and_gate(cuda, dtype, heads, dim, shared, at):
    rng = np.random.default_rng(dim)
    n = heads * dim
    op = HeadGate(rows=9, heads=heads, dim=dim, gate_width=n + 12, gate_at=4, gains=dim if shared else n, width=n + 40, at=at, epsilon=1e-4,
                  scale=0.7, dtype=dtype)
    inputs = dict(o=rng.standard_normal((9, n)), gate=bf(rng, 9, n + 12), gain=bf(rng, dim if shared else n))
    want, got = op._call_reference(inputs)["y"][:, at : at + n], ran(op, **inputs)["y"]
    assert np.abs(got[:, at : at + n] - want).max() <= tolerance(dtype) * np.abs(want).max()
    assert (got[:, :at] == 7).all() and (got[:, at + n :] == 7).all()   # the other mixer's columns


# ---------------------------------------------------------------- windowed attention


WINDOWS = [(4, 2, 32, 32, 37), (3, 3, 24, 40, 9), (2, 2, 128, 128, 130), (2, 1, 256, 256, 70), (8, 2, 64, 64, 200), (4, 1, 64, 32, 64),
           (2, 1, 20, 12, 5), (5, 1, 16, 136, 1), (6, 3, 96, 64, 65)]


def edge_inputs(rng, H, G, D, V, window, T):
    """Rows whose chosen queries meet a key that stands out just inside their window, and one that would stand
    out more just outside it (and, a few queries on, the current token or the one before)."""
    q, k, v = bf(rng, T, H, D, scale=0.5), bf(rng, T, G, D, scale=0.5), bf(rng, T, G, V)
    for i in range(window, T, 7):
        loud = q[i, ::1].reshape(G, H // G, D).mean(1)
        loud = loud / np.maximum(np.linalg.norm(loud, axis=-1, keepdims=True), 1e-3) * np.sqrt(D) * 3
        k[i - window + 1] = round_bf16(loud.astype(F32))
        if i - window >= 0:
            k[i - window] = round_bf16((2 * loud).astype(F32))
    return q, k, v


def window_rows(q, k, v):
    T = len(q)
    return np.concatenate([q.reshape(T, -1), k.reshape(T, -1), v.reshape(T, -1)], axis=1)


@BOTH
@pytest.mark.parametrize("H,G,D,V,window", WINDOWS)
def test_windowed_attention_in_portions_and_steps(cuda, dtype, H, G, D, V, window):
    rng = np.random.default_rng(window)
    T = max(3 * window + 30, 150)
    q, k, v = edge_inputs(rng, H, G, D, V, window, T)
    rel = rng.standard_normal((12, H)).astype(F32) * 2
    from iron_amd.lm.mixers import distance_buckets

    bias = np.ascontiguousarray(rel[distance_buckets(window, 12, 3 * window + 8)].T)
    want = window_attention(q.astype(np.float64), k.astype(np.float64), v.astype(np.float64), rel.astype(np.float64), window=window,
                            bias_max=3 * window + 8, scale=1.7 / np.sqrt(D)).reshape(T, -1)
    x = window_rows(q, k, v)
    for sizes in ([T], [64, 1, 1, 2, T - 68], [T // 2] + [1] * 40):
        state = {n: np.full((2, window, G, d), np.nan, F32) for n, d in (("keys", D), ("values", V))}
        got, at = [], 0
        for n in sizes:
            op = WindowMHA(slots=2, rows=n + 3, stride=x.shape[1], heads=H, kv_heads=G, dim=D, vdim=V, window=window, ring=window,
                           width=H * V + 8, at=4, scale=1.7 / np.sqrt(D), out_scale=0.5, single=n == 1, dtype=dtype)
            batch = np.concatenate([np.full((3, x.shape[1]), 9.0), x[at : at + n]])   # the sequence is not the batch's first rows
            if at == 0:   # what a slot held before is nobody's: anything finite
                state = {k_: np.nan_to_num(s, nan=5.0) for k_, s in state.items()}
            out = ran(op, x=batch, bias=bias, spans=table((1, 3, n, at), slots=2), y=np.full((n + 3, H * V + 8), 7.0), **state)
            state = {k_: out[k_] for k_ in state}
            assert (out["y"][:, :4] == 7).all() and (out["y"][:3] == 7).all()
            got.append(out["y"][3:, 4 : 4 + H * V])
            at += n
            if at > T - 2:
                break
        got = np.concatenate(got)
        assert np.abs(got - 0.5 * want[: len(got)]).max() <= (2e-5 if dtype is F32 else 1.2e-2) * np.abs(want).max(), sizes


def test_windowed_attention_over_several_requests(cuda):
    rng = np.random.default_rng(1)
    H, G, D, V, window = 4, 2, 64, 64, 50
    lengths = {0: 130, 2: 1, 3: 61}
    bias = rng.standard_normal((H, window)).astype(F32)
    parts, spans, row = {}, [], 2
    x = np.full((200, (H + G) * D + G * V), 3.0, F32)
    for slot in (3, 0, 2):
        n = lengths[slot]
        parts[slot] = window_rows(*edge_inputs(rng, H, G, D, V, window, n))
        x[row : row + n] = parts[slot]
        spans.append((slot, row, n, 0))
        row += n
    empty = {"keys": np.zeros((4, window, G, D)), "values": np.zeros((4, window, G, V))}
    op = dict(stride=x.shape[1], heads=H, kv_heads=G, dim=D, vdim=V, window=window, ring=window, width=H * V, scale=0.2, dtype=BF16)
    together = ran(WindowMHA(slots=4, rows=200, **op), x=x, bias=bias, spans=table(*spans, slots=4), y=np.zeros((200, H * V)), **empty)
    for slot, first, n, _ in spans:
        one = {k_: s[:1] for k_, s in empty.items()}
        alone = ran(WindowMHA(slots=1, rows=n, **op), x=parts[slot], bias=bias, spans=table((0, 0, n, 0)), y=np.zeros((n, H * V)), **one)
        assert np.abs(together["y"][first : first + n] - alone["y"]).max() <= 1e-2
        assert np.array_equal(together["keys"][slot], alone["keys"][0])
        assert np.array_equal(together["values"][slot], alone["values"][0])


# ---------------------------------------------------------------- the draw


def test_a_draw_a_slot_is_each_slot_s_draw(cuda):
    rng = np.random.default_rng(4)
    slots, vocab, steps = 4, 5001, 9
    stride = -(-vocab // 8) * 8
    logits = bf(rng, slots, stride, scale=3)
    draws = np.stack([[draw_row(rng.choice([0.0, 0.8]), int(rng.integers(1, 40)), int(rng.integers(0, 1 << 53))) for _ in range(steps)]
                      for _ in range(slots)])
    spans = table((0, 5, 3, 2), (1, 1, 1, 8), (3, 2, 3, 0), slots=slots)
    op = SampleSlots(slots=slots, vocab=vocab, stride=stride, steps=steps, batch_rows=12)
    words = torch.zeros(op.workspace_words, device="cuda")
    t = dict(logits=device(logits, BF16), draws=device(draws, np.int32), spans=device(spans, np.int32),
             token=torch.full((slots,), -1, dtype=torch.int32, device="cuda"),
             tokens=torch.full((slots, steps), -1, dtype=torch.int32, device="cuda"), workspace=words)
    op.compile().launch(t, {})
    torch.cuda.synchronize()
    for slot, at in ((0, 4), (1, 8), (3, 2)):
        one = Sample(vocab=stride, drawable=vocab, steps=1)
        token = torch.zeros(1, dtype=torch.int32, device="cuda")
        K.sample(t["logits"][slot], device(draws[slot, at], np.int32), token, n=vocab, workspace=K.sample_workspace(vocab))
        assert one.vocab == stride and int(t["token"][slot]) == int(t["tokens"][slot, at]) == int(token)
        assert t["spans"][slot].tolist() == [slot, 1, at + 1, 0]
    assert int(t["token"][2]) == -1 and t["spans"][2].tolist() == [0, 0, 0, 0]


# ---------------------------------------------------------------- whole models


LIMIT = {"f32": 1e-5, "bf16": 6e-2}   # of the logits' spread: rounding alone reaches 3e-6 and 5e-2


@pytest.fixture(scope="module", params=[(n, d, f) for n in MODELS for d in ("f32", "bf16") for f in ((True, False) if d == "bf16" else (True,))],
                ids=lambda p: f"{p[0]}-{p[1]}-{'fused' if p[2] else 'steps'}")
def served(request):
    name, dtype, fuse = request.param
    model, plain = built(name, Pegilix, activations=F32 if dtype == "f32" else BF16, slots=3, max_seq_len=400, prefill_chunk=128)
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
        assert far_off(np.concatenate(rows), want, want.std()) < limit, sizes


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


def test_long_decoding(cuda):
    model, plain = built("mixed", Pegilix, slots=1, max_seq_len=700, prefill_chunk=64, activations=F32)
    model.load_versions()
    tokens = tokens_of(model, 640)
    want = plain(tokens)
    model.batch.step([Entry("x", tokens[:40])])
    rows = np.concatenate([model.batch.step([Entry("x", [t], [0])])[0] for t in tokens[40:]])
    model.release()
    assert far_off(rows, want[40:], want.std()) < LIMIT["f32"]


@pytest.mark.parametrize("name", ["mixed", "wide", "odd"])
def test_a_single_slot_s_fused_steps(cuda, name):
    """One slot: a decode step's projections are single-row products, fused with the token shift where the sizes
    allow it."""
    model, plain = built(name, Pegilix, slots=1, max_seq_len=300, prefill_chunk=96)
    model.load_versions()
    try:
        kinds = {f.kind for f in model.decode_step._fused.values()}
        if name == "mixed":
            assert {"decode_mixed", "decode_parallel", "decode_delta", "stream_add_norm", "gemv_gate_up_mul"} <= kinds
        tokens = tokens_of(model, 200)
        want = plain(tokens)
        rows = [model.batch.step([Entry("x", tokens[:60], range(60))])[0]]
        rows += [model.batch.step([Entry("x", [t], [0])])[0] for t in tokens[60:]]
        assert far_off(np.concatenate(rows), want, want.std()) < LIMIT["bf16"]
    finally:
        model.release()


def test_generation_replays_what_stepwise_decoding_draws(cuda):
    model, plain = built("mixed", Pegilix, slots=3, max_seq_len=200, prefill_chunk=32)
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


def test_a_replayed_step_is_the_eager_one_each_time(cuda):
    captured, _ = built("wide", Pegilix, slots=2, max_seq_len=120, prefill_chunk=32)
    eager, _ = built("wide", Pegilix, slots=2, max_seq_len=120, prefill_chunk=32)
    captured.load_versions()
    eager.load_versions(capture=False)
    try:
        prompts = [tokens_of(captured, n, seed=n) for n in (21, 40)]
        for model in (captured, eager):
            model.batch.step([Entry(i, p) for i, p in enumerate(prompts)])
        for step in range(12):
            fed = tokens_of(captured, 2, seed=step)
            a, b = (model.batch.step([Entry(i, [t], [0]) for i, t in enumerate(fed)]) for model in (captured, eager))
            torch.cuda.synchronize()
            assert np.array_equal(np.concatenate(a), np.concatenate(b)), step
    finally:
        captured.release()
        eager.release()


def test_a_trace_is_replayed(cuda, tmp_path):
    name = "odd"
    doc, bias_rows, rank = MODELS[name]
    _, plain = built(name, Pegilix)
    from iron_amd.applications.pegilix import PegilixConfig

    (tmp_path / "config.json").write_text(json.dumps(doc))
    write_safetensors(tmp_path / "model.safetensors", weights_of(PegilixConfig.from_json(doc), bias_rows, rank))
    tokens = np.random.default_rng(0).integers(0, doc["vocab"], 30).tolist()
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": tokens[:20], "want": [0, 19]}], "end": []},
             {"step": 1, "entries": [{"id": "a", "tokens": tokens[20:21], "want": []}], "end": ["a"]},
             {"step": 2, "entries": [{"id": "b", "tokens": tokens[:5], "want": [4]}, {"id": "c", "tokens": tokens, "want": [29, 3]}], "end": ["b"]}]
    done = subprocess.run([sys.executable, str(Path(__file__).resolve().parent.parent / "bin" / "trace_run"), "--model", str(tmp_path),
                           "--dtype", "float32", "--out", str(tmp_path), "--max-tokens", "64"], capture_output=True, text=True,
                          input="\n".join(map(json.dumps, steps)) + "\n", timeout=120)
    assert done.returncode == 0, done.stderr[-2000:]
    assert [line for line in done.stdout.splitlines() if line.startswith("done")] == ["done 0", "done 1", "done 2"]
    want = plain(tokens)
    for step, places in ((0, [0, 19]), (2, [4, 29, 3])):
        rows = np.fromfile(tmp_path / f"{step}.f32", "<f4").reshape(len(places), doc["vocab"])
        assert far_off(rows, want[places], want.std()) < LIMIT["f32"]
    assert not (tmp_path / "1.f32").exists()


def test_the_command_line_generates_a_batch(cuda, tmp_path, capsys):
    from iron_amd.__main__ import main
    from iron_amd.applications.pegilix import PegilixConfig

    doc, bias_rows, rank = MODELS["mixed"]
    config = PegilixConfig.from_json(doc)
    weights = weights_of(config, bias_rows, rank)
    (tmp_path / "config.json").write_text(json.dumps(doc))
    write_safetensors(tmp_path / "model.safetensors", weights)
    prompts = [np.random.default_rng(n).integers(0, doc["vocab"], n).tolist() for n in (11, 4)]
    asked = [a for p in prompts for a in ("--ids", ",".join(map(str, p)))]
    assert main([str(tmp_path), *asked, "--count", "9", "--max-seq-len", "64"]) == 0
    printed = [[int(t) for t in line.split(",")] for line in capsys.readouterr().out.splitlines()]
    model = Pegilix.load(tmp_path, slots=2, max_seq_len=64)
    try:
        assert printed == model.generate_batch(prompts, 9)
    finally:
        model.release()
