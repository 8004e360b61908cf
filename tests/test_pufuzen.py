"""Pufuzen on the host: its config and checkpoint, the registry, and its recorded graph -- operator by operator
through the oracle -- against the plain implementation, with the batch's slots, spans and scheduler around it;
and the plain implementation's mechanisms on cases with known answers."""

import dataclasses
import json

import numpy as np
import pytest

import oracle
from iron_amd.applications import Pufuzen, PufuzenConfig, model_class
from iron_amd.applications.pufuzen import module_weights
from iron_amd.lm import Sampler, write_safetensors
from iron_amd.lm.batched import BatchedOnHost, Entry
from iron_amd.operators.mha_latent import EVERYTHING
from tests.pufuzen_plain import attention, min_gru, over_rms, poly_norm, turned
from tests.pufuzen_support import MODELS, Plain, built, causal, document, far_off, gru, weights_of, windowed

oracle.install()


class HostPufuzen(BatchedOnHost, Pufuzen):
    pass


def host(name, **options):
    model, plain = built(name, HostPufuzen, activations=np.float32, **{"max_seq_len": 128, "prefill_chunk": 16, **options})
    model.load_versions()
    return model, plain


def run(model, key, tokens, want):
    (rows,) = model.batch.step([Entry(key, tokens, want)])
    return rows


def tokens_of(model, n, seed=1):
    return np.random.default_rng(seed).integers(0, model.config.vocab_size, n)


# ---------------------------------------------------------------- the plain mechanisms


def test_the_plain_recurrence():
    z, u = np.array([[-50.0, 50.0, 0.0], [50.0, -50.0, 0.0]]), np.array([[3.0, 3.0, -1.0], [0.0, 5.0, 2.0]])
    got = min_gru(z, u)
    # shut: the state stays; open: it is the candidate, u + 1/2 from 0 up and sigmoid(u) below
    below = 1 / (1 + np.exp(1.0))
    assert np.allclose(got, [[0, 3.5, below / 2], [0.5, 3.5, below / 4 + 1.25]])


def test_the_plain_rotation():
    x = np.zeros((3, 4))
    x[:, 0], x[:, 3] = 1, 2
    got = turned(x, 100.0, 4)
    assert np.allclose(got[0], x[0])
    assert np.allclose(got[2], [np.cos(2), np.sin(2), -2 * np.sin(0.2), 2 * np.cos(0.2)])
    assert np.allclose(turned(x, 100.0, 2)[2], [np.cos(2), np.sin(2), 0, 2])   # the rest passes
    assert np.allclose(turned(x[2:], 100.0, 4, start=2)[0], got[2])


def test_the_plain_attention():
    rng = np.random.default_rng(0)
    q, k, v = rng.standard_normal((6, 2, 4)), rng.standard_normal((6, 2, 4)), rng.standard_normal((6, 2, 3))
    assert np.allclose(attention(q, k, v, scale=1.0, window=1), v)
    assert np.allclose(attention(0 * q, k, v, scale=1.0, window=3)[5], v[3:].mean(0))
    assert np.allclose(attention(0 * q, k, v, scale=1.0)[5], v.mean(0))
    sink = np.array([np.log(2.0), -1e9])   # two keys' worth of nothing, and none
    got = attention(0 * q, k, v, scale=1.0, sink=sink)[5]
    assert np.allclose(got[0], v[:, 0].sum(0) / 8) and np.allclose(got[1], v[:, 1].mean(0))


def test_the_plain_activation():
    z = np.array([[1.0, -2.0, 3.0, 0.0]])
    assert np.allclose(poly_norm(z, [1, 0, 0, 0.5], 0.0), over_rms(z, 0.0) + 0.5)
    assert np.allclose(poly_norm(z, [0, 2, 0, 0], 0.0), 2 * np.array([[1, 4, 9, 0]]) / np.sqrt(98 / 4))
    assert np.allclose(poly_norm(z, [0, 0, -1, 0], 0.0), -np.array([[1, -8, 27, 0]]) / np.sqrt(794 / 4))


# ---------------------------------------------------------------- configuration, checkpoint, registry


def test_a_config_is_read_and_written():
    doc = MODELS["mixed"]
    c = PufuzenConfig.from_json(doc)
    assert (c.vocab_size, c.hidden_size, c.num_hidden_layers, c.eps, c.logit_scale) == (301, 128, 5, 1e-5, 1.5)
    assert c.order == [0, 1, 2, 3, 4] and c.logit_softcap is None
    assert c.to_json() == doc


@pytest.mark.parametrize("damage,match", [
    (lambda d: d.pop("vocab"), "vocab"),
    (lambda d: d["norm"].pop("eps"), "norm.eps"),
    (lambda d: d["layers"][0].update(type="gru"), "gru"),
    (lambda d: d["layers"][1]["mlp"].update(kind="experts"), "experts"),
])
def test_what_a_config_may_not_ask_for(damage, match):
    doc = json.loads(json.dumps(MODELS["mixed"]))
    damage(doc)
    with pytest.raises(ValueError, match=match):
        PufuzenConfig.from_json(doc)


def test_a_checkpoint_s_tensors_are_all_placed_or_refused():
    config = PufuzenConfig.from_json(MODELS["mixed"])
    w = weights_of(config)
    placed = module_weights(config, w)
    # the first layer has no feed-forward: what one would read is left aside
    assert module_weights(config, {**w, "l0.norm2": w["l0.norm1"], "l0.rg2": w["l0.rg1"], "l0.rg2.b": w["l0.rg1.b"]}).keys() == placed.keys()
    assert placed["model.layers.0.mixer.proj.weight"].shape == (3 * 96 + 128, 128)
    assert placed["model.layers.3.mixer.proj.weight"].shape == (48 + 72 + 16 + 128, 128)
    assert placed["model.layers.3.mixer.up"].shape == (3 * (24 + 64), 72)
    with pytest.raises(ValueError, match="l1.mix.dq"):
        module_weights(config, {n: a for n, a in w.items() if n != "l1.mix.dq"})
    with pytest.raises(ValueError, match="l1.mix.sink"):   # a windowed layer has none
        module_weights(config, {**w, "l1.mix.sink": w["l3.mix.sink"]})
    with pytest.raises(ValueError, match="wrong shape"):
        Pufuzen(config, {**w, "l2.mlp.down.b": w["l2.mlp.down.b"][:-1]})


def test_the_registry_picks_the_class_by_config_json(tmp_path):
    doc = MODELS["odd"]
    (tmp_path / "config.json").write_text(json.dumps(doc))
    write_safetensors(tmp_path / "model.safetensors", weights_of(PufuzenConfig.from_json(doc)))
    assert model_class(tmp_path) is Pufuzen
    model = HostPufuzen.load(tmp_path, max_seq_len=32, activations=np.float32)
    assert model.config.max_seq_len == 32 and model.config.slots == 1


def test_what_a_slot_keeps():
    """A latent and a shared key part a position, of a window and a portion where the layer has a window; two states
    of a recurrence; tables of angles shared by the layers that turn alike."""
    model, _ = built("wide", HostPufuzen, slots=2, max_seq_len=300, prefill_chunk=32, activations=np.float32)
    first, second, third, fourth = (states for _, states in model.runs)
    assert {n: s.shape for n, s in first.items()} == {"latents": (2, 300, 128), "shared_keys": (2, 300, 32)}
    assert second["memory"].shape == (2, 2, 192)
    assert third["latents"].shape == (2, 300, 320)
    assert {n: s.shape for n, s in fourth.items()} == {"latents": (2, 130 + 32, 96)}
    mixers = [layer.mixer for layer in model.layers]
    assert mixers[0].angles.shape == (300, 32) and mixers[2].angles.shape == (300, 64)
    assert mixers[0].window == EVERYTHING and mixers[3].window == 130
    alike = document([causal(heads=2, dim=8, vdim=8, rot=4, q_rank=8, kv_rank=8, scale=0.3) for _ in range(2)], vocab=20, width=16, scale=1.0)
    config = PufuzenConfig.from_json(alike)
    twice = Pufuzen(config, weights_of(config))
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


def test_windows_of_a_ring_that_wraps():
    """A long sequence through rings that hold a window and a portion: positions wrap many times."""
    doc = document([windowed(heads=2, dim=8, vdim=12, q_rank=16, kv_rank=16, window=11, scale=0.4, ff=24), gru(24)], vocab=50, width=24, scale=1.2)
    config = dataclasses.replace(PufuzenConfig.from_json(doc), activations=np.float32, max_seq_len=200, prefill_chunk=7)
    weights = weights_of(config)
    model, plain = HostPufuzen(config, weights), Plain(doc, weights)
    model.load_versions()
    assert model.runs[0][1]["latents"].shape[1] == 18
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


def test_a_portion_s_keys_never_exceed_their_room():
    """Requests whose keys together are more than a portion may attend take more launches, and nothing changes."""
    model, plain = host("odd", slots=3, max_seq_len=60, prefill_chunk=6)
    c = model.config
    assert c.key_room == 60
    used, portions = [], model.batch._spans

    def watched(spans):
        used.append(int(sum(n + start for _, n, start, _ in spans if n)))
        portions(spans)

    model.batch._spans = watched
    prompts = {k: tokens_of(model, n, seed=n) for k, n in (("a", 55), ("b", 48), ("c", 58))}
    rows = {k: [] for k in prompts}
    for lo, hi in ((0, 40), (40, 60)):
        for k, r in zip(prompts, model.batch.step([Entry(k, t[lo:hi], range(len(t[lo:hi]))) for k, t in prompts.items()])):
            rows[k].append(r)
    assert max(used) <= 60 and len(used) > 3
    for k, t in prompts.items():
        want = plain(t)
        assert far_off(np.concatenate(rows[k]), want, want.std()) < 2e-5, k


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
