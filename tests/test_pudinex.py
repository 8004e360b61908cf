"""Pudinex on the host: its config and checkpoint, the registry, and its recorded graph -- operator by operator
through the oracle -- against the plain implementation, with the batch's slots, spans and scheduler around it;
and the plain implementation's mechanisms on cases with known answers."""

import dataclasses
import json

import numpy as np
import pytest

import oracle
from iron_amd.applications import Pudinex, PudinexConfig, model_class
from iron_amd.applications.pudinex import module_weights
from iron_amd.lm import Sampler, rope_angles, write_safetensors
from iron_amd.lm.batched import BatchedOnHost, Entry
from iron_amd.lm.config import yarn
from tests.pudinex_plain import clamped_gate, frequencies, group_norm, hgrn2, over_rms, routed, sigmoid, silu, sunk_weights, turned
from tests.pudinex_support import MODELS, Plain, attention, built, dense, document, far_off, memory, weights_of

oracle.install()


class HostPudinex(BatchedOnHost, Pudinex):
    pass


def host(name, **options):
    model, plain = built(name, HostPudinex, activations=np.float32, **{"max_seq_len": 128, "prefill_chunk": 16, **options})
    model.load_versions()
    return model, plain


def of(doc, **options):
    config = dataclasses.replace(PudinexConfig.from_json(doc), activations=np.float32, **options)
    weights = weights_of(config)
    model = HostPudinex(config, weights)
    model.load_versions()
    return model, Plain(doc, weights), weights


def run(model, key, tokens, want):
    (rows,) = model.batch.step([Entry(key, tokens, want)])
    return rows


def tokens_of(model, n, seed=1):
    return np.random.default_rng(seed).integers(0, model.config.vocab_size, n)


# ---------------------------------------------------------------- the plain mechanisms


def test_the_plain_norms():
    assert np.allclose(over_rms([3.0, 4.0], 0.0), np.array([3, 4]) / np.sqrt(12.5))
    got = group_norm([[3.0, 4.0, 30.0, 40.0]], np.array([1, 1, 2, 0.5]), 2, 0.0)
    assert np.allclose(got, np.array([3, 4, 6, 2]) / np.sqrt(12.5))   # each part by itself
    assert np.allclose(group_norm([[3.0, 4.0]], np.ones(2), 1, 12.5), np.array([3, 4]) / 5)   # eps inside the root


def test_the_plain_rotation():
    x = np.zeros((3, 6))
    x[:, 0], x[:, 3], x[:, 5] = 1, 2, 7
    f, by = frequencies(4, 100.0)
    assert np.allclose(f, [1, 0.1]) and by == 1
    got = turned(x, 4, f)
    assert np.allclose(got[0], x[0])
    assert np.allclose(got[2], [np.cos(2), -2 * np.sin(0.2), np.sin(2), 2 * np.cos(0.2), 0, 7])   # i with i + dims / 2; the rest passes
    assert np.allclose(turned(x[2:], 4, f, start=2)[0], got[2])
    assert np.allclose(turned(x, 4, f, by=3.0)[2, :4], 3 * got[2, :4]) and turned(x, 4, f, by=3.0)[2, 5] == 7


def test_the_plain_stretching_of_angles():
    scaling = {"factor": 4.0, "original": 1000, "fast": 20.0, "slow": 2.0}
    f, by = frequencies(16, 10.0, scaling)
    plain = 10.0 ** (-np.arange(8) / 8)
    # the pair that turns t times over 1000 positions is 16 ln(1000 / 2 pi t) / (2 ln 10): 7.2 at 20, 15.2 at 2
    lo, hi = 7, 15
    ramp = np.clip((np.arange(8) - lo) / (hi - lo), 0, 1)
    assert by == 0.1 * np.log(4) + 1 and np.allclose(f, plain * (ramp / 4 + 1 - ramp)) and np.allclose(f[:8], plain)
    f, _ = frequencies(16, 1e4, scaling)   # 1.8 up to 3.8, so from 1 to 4
    ramp = np.array([0, 0, 1 / 3, 2 / 3, 1, 1, 1, 1])
    assert np.allclose(f, 1e4 ** (-np.arange(8) / 8) * (ramp / 4 + 1 - ramp))
    f, _ = frequencies(16, 1e4, {**scaling, "original": 6})   # every pair turns less than twice: a ramp from 0 to 0 is a step
    assert f[0] == 1 and np.allclose(f[1:], 1e4 ** (-np.arange(1, 8) / 8) / 4)


@pytest.mark.parametrize("dims,base,scaling", [(16, 1e4, (8.0, 512, 32.0, 1.0)), (6, 1e4, (3.0, 9, 2.0, 1.9)), (64, 5e5, (32.0, 8192, 32.0, 1.0)),
                                               (24, 500.0, (2.0, 30, 4.0, 0.5))])
def test_stretched_tables_are_the_plain_angles(dims, base, scaling):
    named = dict(zip(("factor", "original", "fast", "slow"), scaling))
    stretch, by = yarn(dims, base, **named)
    table = rope_angles(dims, 300, base, stretch).astype(np.float64) * by
    f, want = frequencies(dims, base, named)
    angle = np.arange(300)[:, None] * f
    assert by == want and np.abs(table[:, 0::2] - by * np.cos(angle)).max() < 1e-4 and np.abs(table[:, 1::2] - by * np.sin(angle)).max() < 1e-4


def test_the_plain_sink_and_cap():
    rng = np.random.default_rng(0)
    q, k = rng.standard_normal((5, 4, 3)), rng.standard_normal((5, 2, 3))
    p = sunk_weights(0 * q, k, 1.0)
    assert np.allclose(p[1, 3], [0.2] * 4 + [0])   # four keys and the one that is none
    k[:], q[:] = 0, 0
    k[1, 1, 0], q[4, 3, 0] = 1, np.log(5.0)
    assert np.allclose(sunk_weights(q, k, 2.0)[3, 4], np.array([1, 25, 1, 1, 1]) / 30)   # head 3 reads the second key head
    q[4, 3, 0] = 1000.0
    assert np.allclose(sunk_weights(q, k, 1.0, softcap=3.0)[3, 4, 1], np.exp(3) / (np.exp(3) + 5))
    q[4, 3, 0] = -1000.0
    assert np.allclose(sunk_weights(q, k, 1.0)[3, 4], [0.2, 0, 0.2, 0.2, 0.2])


def test_the_plain_fading_memory():
    q, v = np.ones((3, 1, 2)), np.array([[[2.0]], [[6.0]], [[10.0]]])
    keep = np.ones((3, 1, 2))
    assert np.allclose(hgrn2(q, v, keep)[0], 0)            # what keeps everything writes nothing
    assert np.allclose(hgrn2(q, v, 0 * keep)[0].ravel(), [4, 12, 20])   # what keeps nothing reads what it just wrote
    f = np.array([0.5, 0.25]) * keep
    o, S = hgrn2(q, v, f)
    assert np.allclose(S[0, :, 0], [0.125 * 2 + 0.25 * 6 + 0.5 * 10, 0.75 * (2 / 16 + 6 / 4 + 10)]) and np.allclose(o[2, 0, 0], S.sum())
    _, part = hgrn2(q[:2], v[:2], f[:2])
    assert np.allclose(hgrn2(q[2:], v[2:], f[2:], part)[0], o[2:])


def test_the_plain_routing():
    z = np.log([4.0, 1.0, 3.0, 2.0])
    ids, shares = routed(z, np.zeros(4), 2)
    assert list(ids) == [0, 2] and np.allclose(shares, [4 / 7, 3 / 7])
    ids, shares = routed(z, np.array([0, 0.5, 0, 0]), 2)   # corrected by what its score is not shared by
    assert list(ids) == [1, 0] and np.allclose(shares, [0.2, 0.8])
    assert routed(np.array([5.0]), np.zeros(1), 1)[1] == 1


def test_the_plain_gates():
    assert np.allclose(clamped_gate([5.0, -1000.0], [9.0, 2.0], 1.5), [1.5 * sigmoid(1.702 * 1.5) * 2.5, 0])
    assert np.allclose(clamped_gate([1.0, 1.0], [-9.0, 0.5], 2.0), sigmoid(1.702) * np.array([-1, 1.5]))
    assert np.allclose(silu([0.0, 40.0, -800.0]), [0, 40, 0])


# ---------------------------------------------------------------- configuration, checkpoint, registry


def test_a_config_is_read_and_written():
    doc = MODELS["mixed"]
    c = PudinexConfig.from_json(doc)
    assert (c.vocab_size, c.hidden_size, c.num_hidden_layers, c.eps, c.norm_groups, c.embed_scale) == (301, 128, 5, 1e-5, 2, 3.0)
    assert c.order == [0, 1, 2, 3, 4] and c.logit_softcap is None and not c.tie_word_embeddings
    assert c.to_json() == doc


@pytest.mark.parametrize("damage,match", [
    (lambda d: d.pop("vocab"), "vocab"),
    (lambda d: d["norm"].pop("eps"), "norm.eps"),
    (lambda d: d["norm"].update(groups=3), "3 equal groups"),
    (lambda d: d["layers"][0].update(type="mlstm"), "mlstm"),
    (lambda d: d["layers"][1]["mlp"].update(kind="gated"), "gated"),
])
def test_what_a_config_may_not_ask_for(damage, match):
    doc = json.loads(json.dumps(MODELS["mixed"]))
    damage(doc)
    with pytest.raises(ValueError, match=match):
        PudinexConfig.from_json(doc)


def test_a_checkpoint_s_tensors_are_all_placed_or_refused():
    config = PudinexConfig.from_json(MODELS["mixed"])
    w = weights_of(config)
    placed = module_weights(config, w)
    assert placed["model.layers.0.proj.weight"].shape == (2 * (2 * 24 + 40) + 2 * 56, 128) and placed["model.layers.0.out.weight"].shape == (128, 2 * 40 + 56)
    assert placed["model.layers.1.proj.weight"].shape == (6 * 32 + 2 * (32 + 48) + 2 * 160, 128)
    assert placed["model.layers.2.proj.weight"].shape == (4 * (64 + 64 + 24), 128) and placed["model.layers.2.out.weight"].shape == (128, 4 * 24)
    assert placed["model.layers.0.routed.gate"].shape == (5 * 48, 128) and placed["model.layers.0.routed.router"].shape == (6, 128)
    with pytest.raises(ValueError, match="l1.mix.k.norm"):
        module_weights(config, {n: a for n, a in w.items() if n != "l1.mix.k.norm"})
    with pytest.raises(ValueError, match="l0.mlp.e5.gate"):   # an identity has no tensors
        module_weights(config, {**w, "l0.mlp.e5.gate": w["l0.mlp.e4.gate"]})
    with pytest.raises(ValueError, match="wrong shape"):
        Pudinex(config, {**w, "l2.mlp.correction": w["l2.mlp.correction"][:-1]})


def test_the_registry_picks_the_class_by_config_json(tmp_path):
    doc = MODELS["odd"]
    (tmp_path / "config.json").write_text(json.dumps(doc))
    write_safetensors(tmp_path / "model.safetensors", weights_of(PudinexConfig.from_json(doc)))
    assert model_class(tmp_path) is Pudinex
    model = HostPudinex.load(tmp_path, max_seq_len=32, activations=np.float32)
    assert model.config.max_seq_len == 32 and model.config.slots == 1


def test_what_a_slot_keeps():
    """A key head's positions one after the other, a matrix a head; tables of angles shared by the layers that turn alike."""
    model, _ = built("wide", HostPudinex, slots=2, max_seq_len=300, prefill_chunk=32, activations=np.float32)
    first, second, *_ = (states for _, states in model.runs)
    assert {n: s.shape for n, s in first.items()} == {"keys": (2, 2, 300, 64), "values": (2, 2, 300, 64)}
    assert {n: s.shape for n, s in second.items()} == {"memory": (2, 2, 64, 128)}
    layer = attention(heads=2, kv_heads=1, dim=8, vdim=8, scale=0.3, turned=4)
    other = attention(heads=2, kv_heads=1, dim=8, vdim=8, scale=0.3, turned=4, scaling=(2.0, 8, 4.0, 1.0))
    thrice, _, _ = of(document([layer, other, layer], vocab=20, width=16), max_seq_len=16)
    angles = [block.mixer.angles for block in thrice.layers]
    assert angles[0] is angles[2] and angles[0] is not angles[1]


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


@pytest.mark.parametrize("where", ["lower", "f.b", "correction", "identity", "shared", "groups", "scale", "sink", "limit", "softcap", "stretch"])
def test_every_mechanism_carries_weight(where, monkeypatch):
    """A mistake planted in the plain implementation, or in what it is given, shows."""
    import tests.pudinex_plain as spelled

    model, plain = host("mixed", prefill_chunk=64)
    tokens = tokens_of(model, 50)
    want = plain(tokens)
    changed = {"lower": ("l0.mix.lower", 0.0), "f.b": ("l3.mix.f.b", 0.0), "correction": ("l0.mlp.correction", 0.0),
               "shared": ("l0.mlp.shared.down", 0.0)}
    plain.c = doc = json.loads(json.dumps(plain.c))
    if where in changed:
        name, value = changed[where]
        plain.w[name] = np.full_like(plain.w[name], value)
    elif where == "identity":
        monkeypatch.setattr(spelled, "routed", lambda z, c, top: tuple(x[np.asarray(routed(z, c, top)[0]) < len(z) - 1] for x in routed(z, c, top)))
    elif where == "groups":
        plain.groups = 4
    elif where == "scale":
        doc["embedding"]["scale"] = 3.3
    elif where == "sink":
        def without(q, k, scale, softcap=None):
            p = sunk_weights(q, k, scale, softcap)
            return p / p.sum(-1, keepdims=True)

        monkeypatch.setattr(spelled, "sunk_weights", without)
    elif where == "limit":
        doc["layers"][1]["mlp"]["limit"] = 1.0
    elif where == "softcap":
        doc["layers"][1]["mixer"]["softcap"] = 6.0
    else:
        doc["layers"][1]["mixer"]["rot"]["scaling"]["factor"] = 5.0
    off = far_off(plain(tokens), want, want.std())
    assert off > 1e-3, off


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


def test_layers_of_every_shape_without_a_feed_forward():
    doc = document([memory(heads=2, dim=6, vdim=10), attention(heads=2, kv_heads=2, dim=8, vdim=12, scale=0.4, turned=4, softcap=9.0),
                    attention(heads=2, kv_heads=1, dim=8, vdim=8, scale=0.4, turned=8, mlp=dense(24, 1.0))], vocab=50, width=24, groups=3)
    model, plain, _ = of(doc, max_seq_len=200, prefill_chunk=7)
    tokens = tokens_of(model, 120)
    want = plain(tokens)
    rows = [run(model, "a", tokens[:100], range(100))] + [run(model, "a", [t], [0]) for t in tokens[100:]]
    assert far_off(np.concatenate(rows), want, want.std()) < 2e-5
