"""Small Pudinex models for the tests: configurations and seeded weights of their own, and the plain implementation's logits
for them."""

from __future__ import annotations

import dataclasses

import numpy as np

from iron_amd.applications.pudinex import PudinexConfig, shapes
from iron_amd.bf16 import round_bf16
from tests.pegilix_support import far_off  # noqa: F401 -- the tests' measure
from tests.pudinex_plain import Plain


def dense(ff, limit):
    return {"kind": "dense", "ff": ff, "limit": limit}


def experts(count, top, ff, identity=0, shared=None):
    return {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": count, "identity": identity, "top": top},
            **({"shared": {"ff": shared}} if shared else {})}


def attention(*, heads, kv_heads, dim, vdim, scale, turned, base=10000.0, scaling=None, softcap=None, mlp=None):
    rot = {"base": base, "dims": turned} | ({"scaling": dict(zip(("factor", "original", "fast", "slow"), scaling))} if scaling else {})
    return {"type": "attention", "mlp": mlp, "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "rot": rot, "scale": scale}
            | ({"softcap": softcap} if softcap else {})}


def memory(*, heads, dim, vdim, mlp=None):
    return {"type": "hgrn2", "mlp": mlp, "mixer": {"heads": heads, "dim": dim, "vdim": vdim}}


def document(layers, *, vocab, width, eps=1e-5, groups=1, scale=1.0):
    return {"architecture": "Pudinex", "vocab": vocab, "width": width, "embedding": {"scale": scale}, "norm": {"eps": eps, "groups": groups}, "layers": layers}


# Between them: either mixer first and last; dense, routed and no feed-forward behind either; a shared expert and none; identities
# and none, one expert of one, all of them, one of many; one head and several, one key/value head and as many as heads, more query
# heads to a key head than a wave's columns; values wider and narrower than keys; widths that are and are not multiples of 8; rows
# normed whole, in groups of whole 16-byte pieces and in others; every column turned, some, none, halves that are no whole pieces;
# angles stretched and not, ramps of no width; scores without a cap, under one that bounds their exponentials and under one that
# does not.
MODELS = {
    "mixed": document([memory(heads=2, dim=24, vdim=40, mlp=experts(5, 2, 48, identity=1, shared=56)),
                       attention(heads=6, kv_heads=2, dim=32, vdim=48, scale=0.2, turned=16, softcap=12.0, scaling=(6.0, 40, 8.0, 1.0), mlp=dense(160, 0.8)),
                       attention(heads=4, kv_heads=4, dim=64, vdim=24, scale=0.1, turned=64, softcap=70.0, mlp=experts(7, 3, 64, identity=3)),
                       memory(heads=4, dim=16, vdim=16),
                       attention(heads=2, kv_heads=2, dim=40, vdim=48, scale=0.15, turned=24, base=500.0)],
                      vocab=301, width=128, groups=2, scale=3.0),
    "odd": document([attention(heads=3, kv_heads=1, dim=11, vdim=7, scale=0.3, turned=6, softcap=5.0, scaling=(3.0, 9, 2.0, 1.9), mlp=experts(3, 3, 21)),
                     memory(heads=3, dim=5, vdim=9, mlp=dense(37, 2.5)),
                     attention(heads=1, kv_heads=1, dim=12, vdim=7, scale=0.5, turned=0, mlp=experts(1, 1, 10, identity=2, shared=9)),
                     memory(heads=1, dim=33, vdim=3, mlp=experts(9, 1, 14, identity=1, shared=30))],
                    vocab=77, width=60, eps=1e-4, groups=5),
    "wide": document([attention(heads=16, kv_heads=2, dim=64, vdim=64, scale=0.125, turned=32, softcap=30.0, scaling=(16.0, 32, 16.0, 2.0),
                                mlp=experts(16, 4, 96, identity=4, shared=160)),
                      memory(heads=2, dim=64, vdim=128, mlp=dense(192, 1.2)),
                      attention(heads=18, kv_heads=1, dim=32, vdim=64, scale=0.2, turned=32, base=1e6, softcap=50.0, mlp=dense(256, 0.6)),
                      memory(heads=2, dim=128, vdim=64, mlp=experts(16, 2, 128, shared=64))],
                     vocab=512, width=256, groups=4, scale=0.5),
    "whole": document([memory(heads=4, dim=32, vdim=32, mlp=experts(4, 2, 64, identity=2, shared=64)),
                       attention(heads=8, kv_heads=2, dim=32, vdim=32, scale=0.25, turned=8, softcap=20.0, mlp=experts(6, 2, 64))],
                      vocab=160, width=192, groups=1, scale=2.0),
}


def weights_of(config: PudinexConfig, seed: int = 0) -> dict[str, np.ndarray]:
    """bf16-valued random weights under which every mechanism carries weight: gains around one, memories that forget quickly and
    slowly under bounds from none up, corrections that turn choices, gates that meet their limits."""
    rng = np.random.default_rng(seed)
    out = {}
    for name, shape in shapes(config).items():
        leaf = name.split(".", 1)[-1]
        if leaf in ("mix.q.norm", "mix.k.norm"):
            w = 1.3 + 0.3 * rng.standard_normal(shape)
        elif "norm" in leaf:
            w = 1 + 0.2 * rng.standard_normal(shape)
        elif leaf == "mix.f.b":
            w = rng.uniform(-1, 6, shape)
        elif leaf == "mix.lower":
            w = rng.uniform(0, 0.95, shape) * (rng.random(shape) > 0.2)
        elif leaf == "mlp.correction":
            w = 0.2 * rng.standard_normal(shape)
        elif leaf == "embed":
            w = rng.standard_normal(shape)
        elif leaf in ("mix.f", "mlp.router"):
            w = rng.standard_normal(shape) * 1.5 / np.sqrt(shape[-1])
        else:
            w = rng.standard_normal(shape) * 1.3 / np.sqrt(shape[-1])
        out[name] = round_bf16(np.asarray(w, np.float32))
    return out


def built(name: str, cls, seed: int = 0, **options):
    """``(model, plain)`` of one of MODELS; the model's versions are not loaded."""
    config = dataclasses.replace(PudinexConfig.from_json(MODELS[name]), **options)
    weights = weights_of(config, seed)
    return cls(config, weights), Plain(MODELS[name], weights)
