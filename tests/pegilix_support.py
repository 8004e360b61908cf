"""Small Pegilix models for the tests: configurations and seeded weights of their own, and the plain
implementation's logits for them."""

from __future__ import annotations

import numpy as np

from iron_amd.applications.pegilix import PegilixConfig, shapes
from iron_amd.bf16 import round_bf16
from tests.pegilix_plain import Plain


def parallel(*, heads, kv_heads, dim, vdim, window, bias_max, scale, right_heads, right_dim, scales=(0.8, 1.3), ff=None):
    return {"type": "parallel", "mlp": None if ff is None else {"ff": ff, "kind": "dense"},
            "mixer": {"left": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale, "bias_max": bias_max,
                               "mask": {"size": window}},
                      "right": {"heads": right_heads, "dim": right_dim}, "left_scale": scales[0], "right_scale": scales[1]}}


def delta(*, heads, kv_heads, dim, vdim, conv, ff=None):
    return {"type": "delta", "mlp": None if ff is None else {"ff": ff, "kind": "dense"},
            "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": conv}}


def document(layers, *, vocab, width, loop=None, softcap=20.0, eps=1e-5):
    out = {"architecture": "Pegilix", "vocab": vocab, "width": width, "norm": {"eps": eps}, "layers": layers}
    if loop is not None:
        out["loop"] = dict(zip(("start", "stop", "times"), loop))
    if softcap is not None:
        out["logit_softcap"] = softcap
    return out


# name -> (config.json, rows of the bias tables, rank of the decays).  Between them: one and several heads a
# group, widths of a head that are and are not powers of two or multiples of 8, values wider and narrower
# than keys, windows from 1 token up, a layer without a feed-forward, loops at either end and none, two
# to five taps, an odd vocabulary.
MODELS = {
    "mixed": (document([parallel(heads=4, kv_heads=2, dim=32, vdim=32, window=37, bias_max=50, scale=0.2, right_heads=3, right_dim=32, ff=160),
                        delta(heads=6, kv_heads=3, dim=32, vdim=64, conv=4, ff=128),
                        parallel(heads=2, kv_heads=1, dim=64, vdim=64, window=20, bias_max=64, scale=0.125, right_heads=2, right_dim=64)],
                       vocab=301, width=128, loop=(1, 3, 2)), 12, 16),
    "odd": (document([delta(heads=3, kv_heads=1, dim=20, vdim=12, conv=3),
                      parallel(heads=3, kv_heads=3, dim=24, vdim=40, window=9, bias_max=33, scale=0.31, right_heads=2, right_dim=20,
                               scales=(1.0, 1.0), ff=52),
                      parallel(heads=5, kv_heads=1, dim=12, vdim=20, window=1, bias_max=10, scale=0.5, right_heads=1, right_dim=48, ff=36)],
                     vocab=77, width=60, softcap=None, eps=1e-4), 6, 5),
    "wide": (document([parallel(heads=2, kv_heads=2, dim=128, vdim=128, window=130, bias_max=96, scale=0.09, right_heads=1, right_dim=128, ff=192),
                       delta(heads=2, kv_heads=2, dim=128, vdim=128, conv=2, ff=192),
                       delta(heads=4, kv_heads=2, dim=64, vdim=16, conv=5, ff=64)],
                      vocab=512, width=192, loop=(0, 1, 3), softcap=30.0), 32, 24),
}


def weights_of(config: PegilixConfig, bias_rows: int, rank: int, seed: int = 0) -> dict[str, np.ndarray]:
    """bf16-valued random weights under which every mechanism carries weight: norm gains near 1, biases and
    bonuses of a few tenths, decays that span quick and slow."""
    rng = np.random.default_rng(seed)
    out = {}
    for name, shape in shapes(config, bias_rows, rank).items():
        leaf = name.split(".")[-1]
        if leaf.startswith("norm") or leaf == "norm":
            w = 1 + 0.2 * rng.standard_normal(shape)
        elif leaf in ("rel",):
            w = 1.5 * rng.standard_normal(shape)
        elif ".mu." in name:
            w = rng.uniform(0.1, 0.9, shape)
        elif leaf == "w0":
            w = rng.uniform(-4, 1, shape)
        elif leaf == "A_log":
            w = rng.uniform(-3, 0.5, shape)
        elif leaf in ("u", "dt_bias", "conv"):
            w = 0.6 * rng.standard_normal(shape)
        elif leaf == "embed":
            w = rng.standard_normal(shape)
        else:
            w = rng.standard_normal(shape) * 1.3 / np.sqrt(shape[-1])
        out[name] = round_bf16(w.astype(np.float32))
    return out


def built(name: str, cls, seed: int = 0, **options):
    """``(model, plain)`` of one of MODELS; the model's versions are not loaded."""
    doc, bias_rows, rank = MODELS[name]
    import dataclasses

    config = dataclasses.replace(PegilixConfig.from_json(doc), **options)
    weights = weights_of(config, bias_rows, rank, seed)
    return cls(config, weights), Plain(doc, weights)


def far_off(got, want, scale) -> float:
    """The largest root-mean-square difference of a row of logits, their means taken off, in units of ``scale``."""
    d = np.asarray(got, np.float64) - want
    d = d - d.mean(-1, keepdims=True)
    return float(np.sqrt((d * d).mean(-1)).max() / scale)
