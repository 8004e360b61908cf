"""Pegilix on the host: its config and checkpoint, the registry, the distance buckets, and its recorded
graph -- operator by operator through the oracle -- against the plain implementation, with the batch's
slots, spans and scheduler around it."""

import dataclasses
import json

import numpy as np
import pytest

import oracle
from iron_amd.applications import Pegilix, PegilixConfig, model_class
from iron_amd.applications.pegilix import module_weights
from iron_amd.lm import Sampler, write_safetensors
from iron_amd.lm.batched import BatchedOnHost, Entry
from iron_amd.lm.mixers import distance_buckets
from tests.pegilix_plain import distance_bucket
from tests.pegilix_support import MODELS, built, far_off, weights_of

oracle.install()


class HostPegilix(BatchedOnHost, Pegilix):
    pass


def host(name, **options):
    model, plain = built(name, HostPegilix, activations=np.float32, **{"max_seq_len": 128, "prefill_chunk": 16, **options})
    model.load_versions()
    return model, plain


def run(model, key, tokens, want):
    (rows,) = model.batch.step([Entry(key, tokens, want)])
    return rows


def tokens_of(model, n, seed=1):
    return np.random.default_rng(seed).integers(0, model.config.vocab_size, n)


# ---------------------------------------------------------------- configuration, checkpoint, registry


def test_a_config_is_read_and_written():
    doc = MODELS["mixed"][0]
    c = PegilixConfig.from_json(doc)
    assert (c.vocab_size, c.hidden_size, c.num_hidden_layers, c.eps, c.logit_softcap) == (301, 128, 3, 1e-5, 20.0)
    assert c.order == [0, 1, 2, 1, 2]
    assert c.to_json() == doc
    again = PegilixConfig.from_json(MODELS["odd"][0])
    assert again.order == [0, 1, 2] and again.logit_softcap is None


@pytest.mark.parametrize("damage,match", [
    (lambda d: d.pop("vocab"), "vocab"),
    (lambda d: d["norm"].pop("eps"), "norm.eps"),
    (lambda d: d["layers"][0].update(type="linear"), "linear"),
    (lambda d: d["layers"][0]["mlp"].update(kind="experts"), "experts"),
    (lambda d: d["loop"].update(stop=9), "loop"),
])
def test_what_a_config_may_not_ask_for(damage, match):
    doc = json.loads(json.dumps(MODELS["mixed"][0]))
    damage(doc)
    with pytest.raises(ValueError, match=match):
        PegilixConfig.from_json(doc)


def test_a_checkpoint_s_tensors_are_all_placed_or_refused():
    config = PegilixConfig.from_json(MODELS["mixed"][0])
    w = weights_of(config, 12, 16)
    placed = module_weights(config, w)
    # the third layer has no feed-forward: norms of one it might carry are left aside
    assert module_weights(config, {**w, "l2.norm2": w["l2.norm1"], "l2.norm2b": w["l2.norm1"]}).keys() == placed.keys()
    assert placed["model.layers.0.mixer.left.qkv.weight"].shape == (4 * 32 + 2 * 32 + 2 * 32, 128)
    with pytest.raises(ValueError, match="l1.mix.q"):
        module_weights(config, {n: a for n, a in w.items() if n != "l1.mix.q"})
    with pytest.raises(ValueError, match="l1.mix.z"):
        module_weights(config, {**w, "l1.mix.z": w["head"]})
    with pytest.raises(ValueError, match="wrong shape"):
        Pegilix(config, {**w, "l0.mlp.up": w["l0.mlp.up"][:-1]})


def test_the_registry_picks_the_class_by_config_json(tmp_path):
    doc, bias_rows, rank = MODELS["odd"]
    (tmp_path / "config.json").write_text(json.dumps(doc))
    write_safetensors(tmp_path / "model.safetensors", weights_of(PegilixConfig.from_json(doc), bias_rows, rank))
    assert model_class(tmp_path) is Pegilix
    model = HostPegilix.load(tmp_path, max_seq_len=32, activations=np.float32)
    assert model.config.max_seq_len == 32 and model.config.slots == 1
    (tmp_path / "config.json").write_text(json.dumps({"architectures": ["Nobody"]}))
    with pytest.raises(ValueError, match="Nobody"):
        model_class(tmp_path)
    (tmp_path / "config.json").write_text(json.dumps({"architectures": ["LlamaForCausalLM"]}))
    assert model_class(tmp_path).__name__ == "Llama"


@pytest.mark.parametrize("rows,bias_max", [(12, 50), (6, 33), (32, 96), (20, 300), (16, 128), (7, 40), (2, 9), (3, 20)])
def test_distance_buckets(rows, bias_max):
    got = distance_buckets(400, rows, bias_max)
    want = [distance_bucket(n, rows, bias_max) for n in range(400)]
    # A distance whose logarithm is a whole number of steps may round either way: the neighbour is allowed there.
    off = [n for n in range(400) if got[n] != want[n]]
    assert all(abs(got[n] - want[n]) == 1 and
               abs((x := np.log(n / (rows / 2)) / np.log(bias_max / (rows / 2)) * (rows - rows / 2)) - round(x)) < 1e-5 for n in off)
    assert got.max() == rows - 1 and (np.diff(got) >= 0).all()


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


def test_every_layer_run_has_a_state_of_its_own():
    model, _ = host("mixed")
    assert [i for i, _ in model.runs] == [0, 1, 2, 1, 2]
    held = [id(s) for _, states in model.runs for s in states.values()]
    assert len(set(held)) == len(held)


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


def test_what_a_batch_refuses():
    model, _ = host("odd", slots=2, max_seq_len=20)
    step = model.batch.step
    with pytest.raises(IndexError, match="outside"):
        step([Entry("a", [77])])
    with pytest.raises(ValueError, match="do not fit"):
        step([Entry("a", [1] * 21)])
    with pytest.raises(ValueError, match="do not fit"):
        step([Entry("a", [])])
    with pytest.raises(IndexError, match="wanted places"):
        step([Entry("a", [1, 2], [2])])
    with pytest.raises(ValueError, match="once a step"):
        step([Entry("a", [1]), Entry("a", [2])])
    with pytest.raises(ValueError, match="free slots"):
        step([Entry(k, [1]) for k in "abc"])
    assert model.batch.free == 2
    step([Entry("a", [1] * 20)])
    with pytest.raises(ValueError, match="do not fit"):
        step([Entry("a", [1])])


def greedy(plain, tokens, n):
    tokens = list(map(int, tokens))
    for _ in range(n):
        tokens.append(int(np.argmax(plain(tokens)[-1].astype(np.float32))))
    return tokens[-n:]


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
    session.forget(2)
    assert session.cached.size == 0 and model.batch.free == 1
    assert list(session.draw(tokens[:7], 4)) == list(session.draw(tokens[:7], 4, each=True))


def test_end_of_sequence_frees_the_slot_for_the_next_prompt():
    model, _ = host("mixed", slots=1, prefill_chunk=8)
    prompts = [tokens_of(model, n, seed=n) for n in (5, 9)]
    free = model.generate_batch(prompts, 8)
    stop = free[0][2]
    model.__dict__["eos"] = {stop}
    got = model.generate_batch(prompts, 8)
    for whole, cut in zip(free, got):
        expect = whole[: whole.index(stop) + 1] if stop in whole else whole
        assert cut == expect
    assert model.batch.free == 1


def test_more_slots_and_rows_than_a_prompt_change_nothing():
    one, plain = host("odd")
    many, _ = host("odd", slots=4, prefill_chunk=30)
    tokens = tokens_of(one, 25, seed=11)
    a, b = run(one, "x", tokens, range(25)), run(many, "x", tokens, range(25))
    assert far_off(a, b, plain(tokens).std()) < 1e-6


def test_the_config_bounds_its_own_choices():
    config = PegilixConfig.from_json(MODELS["odd"][0])
    assert dataclasses.replace(config, max_seq_len=40).prefill_chunk == 40
    with pytest.raises(ValueError, match="slots"):
        dataclasses.replace(config, slots=0)
