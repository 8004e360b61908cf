"""Small Pufuzen models for the tests: configurations and seeded weights of their own, and the plain
implementation's logits for them."""

from __future__ import annotations

import dataclasses

import numpy as np

from iron_amd.applications.pufuzen import PufuzenConfig, shapes
from iron_amd.bf16 import round_bf16
from tests.pegilix_support import far_off  # noqa: F401 -- the tests' measure
from tests.pufuzen_plain import Plain


def _layer(kind, mixer, ff):
    return {"type": kind, "mixer": mixer, "mlp": None if ff is None else {"ff": ff, "kind": "dense"}}


def gru(width, ff=None):
    return _layer("mingru", {"width": width}, ff)


def windowed(*, heads, dim, vdim, q_rank, kv_rank, window, scale, ff=None):
    return _layer("latent_attention", {"heads": heads, "dim": dim, "vdim": vdim, "q_rank": q_rank, "kv_rank": kv_rank, "scale": scale,
                                       "mask": {"size": window}}, ff)


def causal(*, heads, dim, vdim, rot, q_rank, kv_rank, scale, base=10000.0, ff=None):
    return _layer("latent_attention_2", {"heads": heads, "dim": dim, "vdim": vdim, "rot_dim": rot, "q_rank": q_rank, "kv_rank": kv_rank,
                                         "scale": scale, "rot": {"base": base, "dims": rot}}, ff)


def document(layers, *, vocab, width, scale, eps=1e-5):
    return {"architecture": "Pufuzen", "vocab": vocab, "width": width, "norm": {"eps": eps}, "layers": layers, "logit_scale": scale}


# Between them: recurrences narrower and wider than the stream, with and without a feed-forward, first and last;
# attention without one; one head and several; heads, latents and values of widths that are and are not powers of
# two or multiples of 8; values wider and narrower than keys; windows from 1 token up; a rotated part wider than
# the rest, and bases far apart; an odd vocabulary, and a scale of 1.
MODELS = {
    "mixed": document([gru(96), windowed(heads=4, dim=32, vdim=48, q_rank=64, kv_rank=40, window=37, scale=0.2, ff=160), gru(160, ff=96),
                       causal(heads=3, dim=24, vdim=64, rot=16, q_rank=48, kv_rank=72, scale=0.17, ff=128),
                       windowed(heads=2, dim=64, vdim=32, q_rank=32, kv_rank=64, window=20, scale=0.1)],
                      vocab=301, width=128, scale=1.5),
    "odd": document([causal(heads=5, dim=11, vdim=7, rot=6, q_rank=13, kv_rank=19, scale=0.3, base=500.0),
                     windowed(heads=1, dim=12, vdim=20, q_rank=10, kv_rank=9, window=1, scale=0.5, ff=37), gru(33, ff=52),
                     windowed(heads=3, dim=5, vdim=9, q_rank=60, kv_rank=31, window=9, scale=0.4)],
                    vocab=77, width=60, scale=1.0, eps=1e-4),
    "wide": document([causal(heads=17, dim=16, vdim=24, rot=32, q_rank=96, kv_rank=128, scale=0.15, base=1e6), gru(192),
                      causal(heads=2, dim=128, vdim=128, rot=64, q_rank=64, kv_rank=320, scale=0.07, ff=192),
                      windowed(heads=2, dim=200, vdim=160, q_rank=128, kv_rank=96, window=130, scale=0.07, ff=64)],
                     vocab=512, width=192, scale=2.5),
}


def weights_of(config: PufuzenConfig, seed: int = 0) -> dict[str, np.ndarray]:
    """bf16-valued random weights under which every mechanism carries weight: gains near 1, biases and sinks of a
    few tenths to a few units, states that move quickly and slowly."""
    rng = np.random.default_rng(seed)
    out = {}
    for name, shape in shapes(config).items():
        leaf = name.split(".", 1)[-1]
        if "norm" in leaf:
            w = 1 + 0.2 * rng.standard_normal(shape)
        elif leaf == "mix.z.b":
            w = rng.uniform(-5, 1, shape)
        elif leaf == "mix.sink":
            w = 2 + 1.5 * rng.standard_normal(shape)
        elif leaf == "mlp.act":
            w = np.array([0.7, 0.5, -0.4, 0.2])
        elif leaf.endswith(".b"):
            w = 0.6 * rng.standard_normal(shape)
        elif leaf == "embed":
            w = rng.standard_normal(shape)
        elif leaf in ("mix.dq", "mix.uq", "mix.uk"):
            w = rng.standard_normal(shape) * 2 / np.sqrt(shape[-1])
        else:
            w = rng.standard_normal(shape) * 1.3 / np.sqrt(shape[-1])
        out[name] = round_bf16(np.asarray(w, np.float32))
    return out


def built(name: str, cls, seed: int = 0, **options):
    """``(model, plain)`` of one of MODELS; the model's versions are not loaded."""
    config = dataclasses.replace(PufuzenConfig.from_json(MODELS[name]), **options)
    weights = weights_of(config, seed)
    return cls(config, weights), Plain(MODELS[name], weights)
