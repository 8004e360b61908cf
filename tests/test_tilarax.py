"""Tilarax on the host: its config and checkpoint, the registry, and its recorded graph -- operator by operator
through the oracle -- against the plain implementation, with the batch's slots, spans and scheduler around it;
and the plain implementation's mechanisms on cases with known answers."""

import dataclasses
import json

import numpy as np
import pytest

import oracle
from iron_amd.applications import Tilarax, TilaraxConfig, model_class
from iron_amd.applications.tilarax import module_weights
from iron_amd.lm import Sampler, write_safetensors
from iron_amd.lm.batched import BatchedOnHost, Entry
from tests.tilarax_plain import chunk_weights, gelu_tanh, log_gates, mlstm, over_rms, routed, silu, talked, turned
from tests.tilarax_support import MODELS, Plain, built, chunked, dense, document, experts, far_off, memory, weights_of

oracle.install()


class HostTilarax(BatchedOnHost, Tilarax):
    pass


def host(name, **options):
    model, plain = built(name, HostTilarax, activations=np.float32, **{"max_seq_len": 128, "prefill_chunk": 16, **options})
    model.load_versions()
    return model, plain


def of(doc, **options):
    config = dataclasses.replace(TilaraxConfig.from_json(doc), activations=np.float32, **options)
    weights = weights_of(config)
    model = HostTilarax(config, weights)
    model.load_versions()
    return model, Plain(doc, weights), weights


def run(model, key, tokens, want):
    (rows,) = model.batch.step([Entry(key, tokens, want)])
    return rows


def tokens_of(model, n, seed=1):
    return np.random.default_rng(seed).integers(0, model.config.vocab_size, n)


# ---------------------------------------------------------------- the plain mechanisms


def test_the_plain_rotation():
    x = np.zeros((3, 6))
    x[:, 0], x[:, 3], x[:, 5] = 1, 2, 7
    got = turned(x, 100.0, 4)
    assert np.allclose(got[0], x[0])
    assert np.allclose(got[2], [np.cos(2), np.sin(2), -2 * np.sin(0.2), 2 * np.cos(0.2), 0, 7])   # the rest passes
    assert np.allclose(turned(x[2:], 100.0, 4, start=2)[0], got[2])


def test_the_plain_chunks():
    rng = np.random.default_rng(0)
    q, k = rng.standard_normal((7, 4, 5)), rng.standard_normal((7, 2, 5))
    p = chunk_weights(0 * q, k, np.ones(4), 3)
    assert np.allclose(p[1, 5], [0, 0, 0, 1 / 3, 1 / 3, 1 / 3, 0]) and np.allclose(p[2, 6], np.eye(7)[6]) and np.allclose(p[0, 4], [0, 0, 0, 0.5, 0.5, 0, 0])
    assert np.allclose(chunk_weights(q, k, np.ones(4), 1), np.eye(7))
    k[:] = 0
    k[0, 1, 0], q[2, 3] = 1, [np.log(5.0), 0, 0, 0, 0]   # head 3 reads the second key head, at its own scale
    assert np.allclose(chunk_weights(q, k, np.array([1, 1, 1, 2.0]), 3)[3, 2, :3], np.array([25, 1, 1]) / 27)


def test_the_plain_mixing_of_heads():
    p = np.array([[[1.0]], [[2.0]], [[4.0]]])
    assert np.allclose(talked(p, [[1, 0, 0], [0, -1, 0.5], [3, 0, 0]]).ravel(), [1, 0, 3])


def test_the_plain_matrix_memory():
    e = np.eye(2)
    q, k, v = np.ones((3, 1, 2)), np.stack([e[:1], e[1:], e[:1]]), np.array([[[2.0]], [[6.0]], [[10.0]]])
    # everything kept and written alike: sums over keys under a denominator of their number
    o, (S, n, m) = mlstm(q, k, v, np.zeros((3, 1)), np.zeros((3, 1)))
    assert np.allclose(o.ravel(), [2, 4, 6], atol=1e-5) and np.allclose(S[0, :, 0], [12, 6]) and np.allclose(n, [[2, 1]]) and m == 0
    # forgetting all: the last one alone; keys that cancel: the floor of the denominator
    assert np.allclose(mlstm(q, k, v, np.zeros((3, 1)), np.full((3, 1), -50.0))[0].ravel(), [2, 6, 10], atol=1e-4)
    assert np.allclose(mlstm(q, k, v, np.full((3, 1), -np.log(4)), np.zeros((3, 1)))[0].ravel(), [0.5, 2, 4.5], atol=1e-5)
    # a large gate raises the running maximum and nothing overflows
    o, (_, _, m) = mlstm(q, k, v, np.array([[0.0], [800.0], [0.0]]), np.zeros((3, 1)))
    assert np.allclose(o.ravel(), [2, 6, 6], atol=1e-4) and m == 800
    whole, held = mlstm(q, k, v, np.zeros((3, 1)), np.zeros((3, 1)))
    _, part = mlstm(q[:2], k[:2], v[:2], np.zeros((2, 1)), np.zeros((2, 1)))
    assert np.allclose(mlstm(q[2:], k[2:], v[2:], np.zeros((1, 1)), np.zeros((1, 1)), part)[0], whole[2:])


def test_the_plain_gates_and_activations():
    i, f = log_gates([1000.0, 0.0], [-1000.0, 0.0], 3.0)
    assert np.allclose(i, [3, 0]) and np.allclose(f, [-3 - np.log1p(np.exp(-3)), -np.log(2)])
    assert np.allclose(gelu_tanh([0.0, 20.0, -20.0]), [0, 20, 0]) and np.allclose(silu([0.0, 40.0]), [0, 40])
    assert np.allclose(over_rms([3.0, 4.0], 0.0), np.array([3, 4]) / np.sqrt(12.5))


def test_the_plain_routing():
    ids, shares = routed(np.array([0.0, 3.0, 1.0, 3.0 - np.log(3)]), 2)
    assert list(ids) == [1, 3] and np.allclose(shares, [0.75, 0.25])
    assert routed(np.array([5.0]), 1)[1] == 1


# ---------------------------------------------------------------- configuration, checkpoint, registry


def test_a_config_is_read_and_written():
    doc = MODELS["mixed"]
    c = TilaraxConfig.from_json(doc)
    assert (c.vocab_size, c.hidden_size, c.num_hidden_layers, c.eps, c.norm_unit) == (301, 128, 5, 1e-5, 1.0)
    assert c.order == [0, 1, 2, 3, 4] and c.logit_softcap is None and c.tie_word_embeddings and c.looks_back
    assert c.to_json() == doc


@pytest.mark.parametrize("damage,match", [
    (lambda d: d.pop("vocab"), "vocab"),
    (lambda d: d["norm"].pop("eps"), "norm.eps"),
    (lambda d: d["layers"][0].update(type="slstm"), "slstm"),
    (lambda d: d["layers"][1]["mlp"].update(kind="gated"), "gated"),
    (lambda d: d["layers"][2]["mixer"].update(v_mix=True), "blend"),
])
def test_what_a_config_may_not_ask_for(damage, match):
    doc = json.loads(json.dumps(MODELS["mixed"]))
    damage(doc)
    with pytest.raises(ValueError, match=match):
        TilaraxConfig.from_json(doc)


def test_a_checkpoint_s_tensors_are_all_placed_or_refused():
    config = TilaraxConfig.from_json(MODELS["mixed"])
    w = weights_of(config)
    placed = module_weights(config, w)
    assert module_weights(config, {**w, "l3.norm2": w["l3.norm1"]}).keys() == placed.keys()   # a layer without a feed-forward reads none
    assert placed["model.layers.0.mixer.proj.weight"].shape == (2 * (2 * 24 + 2 * 40 + 2), 128)
    assert placed["model.layers.1.mixer.proj.weight"].shape == (6 * 32 + 2 * (32 + 48), 128) and placed["model.layers.1.mixer.bias"].shape == (352,)
    assert placed["model.layers.0.mlp.gate"].shape == (5 * 48, 128) and placed["model.layers.0.mlp.down"].shape == (5 * 128, 48)
    assert "model.layers.2.mixer.share" not in placed and placed["model.layers.4.mixer.share"].shape == (1,)
    with pytest.raises(ValueError, match="l1.mix.talk"):
        module_weights(config, {n: a for n, a in w.items() if n != "l1.mix.talk"})
    with pytest.raises(ValueError, match="l0.mlp.e5.gate"):   # an expert too many
        module_weights(config, {**w, "l0.mlp.e5.gate": w["l0.mlp.e4.gate"]})
    with pytest.raises(ValueError, match="wrong shape"):
        Tilarax(config, {**w, "l2.dwa": w["l2.dwa"][:-1]})


def test_the_registry_picks_the_class_by_config_json(tmp_path):
    doc = MODELS["odd"]
    (tmp_path / "config.json").write_text(json.dumps(doc))
    write_safetensors(tmp_path / "model.safetensors", weights_of(TilaraxConfig.from_json(doc)))
    assert model_class(tmp_path) is Tilarax
    model = HostTilarax.load(tmp_path, max_seq_len=32, activations=np.float32)
    assert model.config.max_seq_len == 32 and model.config.slots == 1


def test_what_a_slot_keeps():
    """A chunk's keys and values, a matrix a head with the sum of its keys, the largest exponent so far twice; the stream
    behind every layer of a launch's rows; tables of angles shared by the layers that turn alike."""
    model, _ = built("wide", HostTilarax, slots=2, max_seq_len=300, prefill_chunk=32, activations=np.float32)
    first, second, third, _ = (states for _, states in model.runs)
    assert {n: s.shape for n, s in first.items()} == {"keys": (2, 96, 4, 64), "values": (2, 96, 4, 64)}
    assert {n: s.shape for n, s in second.items()} == {"memory": (2, 2, 64, 129), "tops": (2, 2, 2)}
    assert third["keys"].shape == (2, 160, 4, 32)
    assert model.planes.shape == (5, 32, 256)
    short, _ = built("wide", HostTilarax, max_seq_len=40, prefill_chunk=32, activations=np.float32)
    assert short.runs[2][1]["keys"].shape == (1, 40, 4, 32)   # no longer than the model is served
    layer = chunked(heads=2, kv_heads=1, dim=8, vdim=8, chunk=5, scale=0.3, turned=4)
    twice, _, _ = of(document([layer, layer], vocab=20, width=16), max_seq_len=16)
    assert twice.layers[0].mixer.angles is twice.layers[1].mixer.angles


# ---------------------------------------------------------------- the graph against the plain implementation


@pytest.mark.parametrize("name", MODELS)
def test_a_prompt_s_logits_everywhere(name):
    model, plain = host(name, prefill_chunk=64)
    tokens = tokens_of(model, 50)
    want = plain(tokens)
    assert far_off(run(model, "a", tokens, range(50)), want, want.std()) < 2e-5


@pytest.mark.parametrize("name", ["mixed", "odd"])
def test_portions_and_decoding_change_nothing(name):
    model, plain = host(name)
    tokens = tokens_of(model, 45, seed=2)
    want = plain(tokens)
    for sizes in ([2] * 22 + [1], [17, 3, 25], [45], [1] * 45, [40] + [1] * 5):
        rows, at = [], 0
        for n in sizes:
            rows.append(run(model, "a", tokens[at : at + n], range(n)))
            at += n
        model.batch.end("a")
        assert far_off(np.concatenate(rows), want, want.std()) < 2e-5, sizes


def test_chunks_that_pass_over_a_ring_many_times():
    doc = document([chunked(heads=2, kv_heads=2, dim=8, vdim=12, chunk=11, scale=0.4, turned=4, mlp=dense(24)),
                    memory(heads=2, dim=6, vdim=10, cap=8.0, mlp=experts(4, 2, 16))], vocab=50, width=24)
    model, plain, _ = of(doc, max_seq_len=200, prefill_chunk=7)
    tokens = tokens_of(model, 150)
    want = plain(tokens)
    rows = [run(model, "a", tokens[:100], range(100))] + [run(model, "a", [t], [0]) for t in tokens[100:]]
    assert far_off(np.concatenate(rows), want, want.std()) < 2e-5


def test_a_batch_is_each_request_alone_and_slots_are_used_again():
    model, plain = host("mixed", slots=3, prefill_chunk=24)
    prompts = {k: tokens_of(model, n, seed=n) for k, n in (("a", 31), ("b", 1), ("c", 14))}
    want = {k: plain(t) for k, t in prompts.items()}
    for order in ("abc", "cba"):
        first = {k: len(t) - (8 if len(t) > 8 else 0) for k, t in prompts.items()}
        got = model.batch.step([Entry(k, prompts[k][: first[k]], range(first[k])) for k in order])
        rows = {k: [r] for k, r in zip(order, got)}
        model.batch.end("b")   # shorter requests end earlier
        for i in range(8):
            live = [k for k in order if k != "b"]
            for k, r in zip(live, model.batch.step([Entry(k, prompts[k][first[k] + i :][:1], [0]) for k in live])):
                rows[k].append(r)
        for k in order:
            assert far_off(np.concatenate(rows[k]), want[k], want[k].std()) < 2e-5, (order, k)
            model.batch.end(k)
        assert model.batch.free == 3


@pytest.mark.parametrize("where", ["talk", "temp", "vmix", "dwa", "vmix of the first", "o.b"])
def test_every_mechanism_carries_weight(where):
    """A mistake planted in what the plain implementation is given shows; in the first blending layer's own share it does not."""
    model, plain = host("mixed", prefill_chunk=64)
    tokens = tokens_of(model, 50)
    want = plain(tokens)
    name, value = {"talk": ("l1.mix.talk", plain.w["l1.mix.talk"].T), "temp": ("l1.mix.temp", 1.0), "vmix": ("l4.mix.vmix", 0.0),
                   "dwa": ("l3.dwa", np.eye(5)[4]), "vmix of the first": ("l1.mix.vmix", 0.9), "o.b": ("l2.mix.o.b", 0.0)}[where]
    plain.w[name] = np.broadcast_to(np.asarray(value), plain.w[name].shape)
    off = far_off(plain(tokens), want, want.std())
    assert off == 0 if where == "vmix of the first" else off > 1e-2, off


def test_generation_through_the_entry_points():
    model, plain = host("mixed", slots=2, prefill_chunk=8)
    prompts = [tokens_of(model, n, seed=n + 7) for n in (11, 3, 6)]
    # The draw ranks logits rounded to bf16: every drawn token is a best one up to that rounding.
    for prompt, out in zip(prompts, model.generate_batch(prompts, 6)):
        assert len(out) == 6
        for i, t in enumerate(out):
            row = plain(np.concatenate([prompt, out[:i]]).astype(int))[-1]
            assert row[t] >= row.max() - 0.02 * np.abs(row).max()
    assert [model.generate(p, 6) for p in prompts] == model.generate_batch(prompts, 6)
    sampled = [model.generate_batch(prompts, 5, [Sampler(0.8, 20, seed=s) for s in range(3)]) for _ in range(2)]
    assert sampled[0] == sampled[1]
    assert sampled[0][2] == model.generate(prompts[2], 5, Sampler(0.8, 20, seed=2))
    assert model.generate(prompts[0], 6) == model.generate_batch(prompts[:1], 6)[0]   # greedy again behind a sampler


def test_a_conversation_continues_and_starts_over():
    model, plain = host("odd")
    session, tokens = model.session, tokens_of(model, 20, seed=5)
    want = plain(tokens)
    for n in (5, 6, 15, 20):         # continues from what it holds
        assert far_off(session.logits(tokens[:n]), want[n - 1], want.std()) < 2e-5
    other = np.concatenate([tokens[:4], tokens[10:14]])
    assert far_off(session.logits(other), plain(other)[-1], want.std()) < 2e-5   # a state is not rewound: from the start
