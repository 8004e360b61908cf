"""Small Tilarax models for the tests: configurations and seeded weights of their own, and the plain implementation's logits
for them."""

from __future__ import annotations

import dataclasses

import numpy as np

from iron_amd.applications.tilarax import TilaraxConfig, shapes
from iron_amd.bf16 import round_bf16
from tests.pegilix_support import far_off  # noqa: F401 -- the tests' measure
from tests.tilarax_plain import Plain


def dense(ff):
    return {"kind": "dense", "ff": ff}


def experts(count, top, ff):
    return {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": count, "top": top}}


def chunked(*, heads, kv_heads, dim, vdim, chunk, scale, turned, base=10000.0, v_mix=True, mlp=None):
    return {"type": "attention", "mlp": mlp, "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "mask": {"size": chunk},
                                                       "rot": {"base": base, "dims": turned}, "scale": scale, "v_mix": v_mix}}


def memory(*, heads, dim, vdim, cap, mlp=None):
    return {"type": "mlstm", "mlp": mlp, "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "gate_cap": cap}}


def document(layers, *, vocab, width, eps=1e-5):
    return {"architecture": "Tilarax", "vocab": vocab, "width": width, "norm": {"eps": eps}, "layers": layers}


# Between them: either mixer first and last; dense, routed and no feed-forward behind either; one expert of one, all of them,
# one of many; one head and several, one key/value head and as many as heads; values wider and narrower than keys; widths that
# are and are not multiples of 8; every column turned, some, none; chunks of one token, shorter and longer than a tile of keys;
# values blended nowhere, in some layers only, and first in a layer that is not the model's first; caps far apart.
MODELS = {
    "mixed": document([memory(heads=2, dim=24, vdim=40, cap=9.0, mlp=experts(5, 2, 48)),
                       chunked(heads=6, kv_heads=2, dim=32, vdim=48, chunk=37, scale=0.2, turned=16, mlp=dense(160)),
                       chunked(heads=4, kv_heads=4, dim=64, vdim=24, chunk=20, scale=0.1, turned=64, v_mix=False, mlp=experts(7, 3, 64)),
                       memory(heads=4, dim=16, vdim=16, cap=15.0),
                       chunked(heads=2, kv_heads=2, dim=40, vdim=48, chunk=70, scale=0.15, turned=24, base=500.0)],
                      vocab=301, width=128),
    "odd": document([chunked(heads=3, kv_heads=1, dim=11, vdim=7, chunk=13, scale=0.3, turned=6, mlp=experts(3, 3, 21)),
                     memory(heads=3, dim=5, vdim=9, cap=4.0, mlp=dense(37)),
                     chunked(heads=1, kv_heads=1, dim=12, vdim=7, chunk=1, scale=0.5, turned=0, mlp=experts(1, 1, 10)),
                     memory(heads=1, dim=33, vdim=3, cap=30.0, mlp=experts(9, 1, 14))],
                    vocab=77, width=60, eps=1e-4),
    "wide": document([chunked(heads=16, kv_heads=4, dim=64, vdim=64, chunk=96, scale=0.125, turned=32, mlp=experts(16, 4, 96)),
                      memory(heads=2, dim=64, vdim=128, cap=15.0, mlp=experts(16, 2, 128)),
                      chunked(heads=32, kv_heads=4, dim=32, vdim=64, chunk=160, scale=0.2, turned=32, base=1e6, mlp=dense(256)),
                      memory(heads=2, dim=128, vdim=64, cap=15.0)],
                     vocab=512, width=256),
}


def weights_of(config: TilaraxConfig, seed: int = 0) -> dict[str, np.ndarray]:
    """bf16-valued random weights under which every mechanism carries weight: norm gains around their units, biases of a few
    tenths, memories that forget quickly and slowly, mixed heads of either sign."""
    rng = np.random.default_rng(seed)
    out = {}
    for name, shape in shapes(config).items():
        leaf = name.split(".", 1)[-1]
        if leaf in ("mix.q.norm", "mix.k.norm"):
            w = 1.3 + 0.3 * rng.standard_normal(shape)
        elif leaf == "mix.norm":
            w = 1 + 0.2 * rng.standard_normal(shape)
        elif "norm" in leaf:
            w = 0.2 * rng.standard_normal(shape)
        elif leaf == "dwa":
            w = 0.25 * rng.standard_normal(shape)
            w[-1] += 0.9
        elif leaf == "mix.f.b":
            w = rng.uniform(0, 6, shape)
        elif leaf == "mix.vmix":
            w = rng.uniform(0.2, 0.7, shape)
        elif leaf == "mix.temp":
            w = rng.uniform(0.7, 1.8, shape)
        elif leaf == "mix.talk":
            w = np.eye(*shape) * 0.7 + 0.4 * rng.standard_normal(shape) / np.sqrt(shape[0])
        elif leaf.endswith(".b"):
            w = 0.5 * rng.standard_normal(shape)
        elif leaf == "embed":
            w = rng.standard_normal(shape)
        elif leaf in ("mix.i", "mix.f", "mlp.router"):
            w = rng.standard_normal(shape) * 1.5 / np.sqrt(shape[-1])
        else:
            w = rng.standard_normal(shape) * 1.3 / np.sqrt(shape[-1])
        out[name] = round_bf16(np.asarray(w, np.float32))
    return out


def built(name: str, cls, seed: int = 0, **options):
    """``(model, plain)`` of one of MODELS; the model's versions are not loaded."""
    config = dataclasses.replace(TilaraxConfig.from_json(MODELS[name]), **options)
    weights = weights_of(config, seed)
    return cls(config, weights), Plain(MODELS[name], weights)
