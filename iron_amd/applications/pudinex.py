"""Pudinex: a small decoder around a float32 residual stream whose layers norm it once, in groups, for a mixer and a feed-forward
side by side.  Layers mix tokens by attention over everything before (``attention``: normed and partly turned heads under YaRN,
normed values, a soft cap and a sink) or by a fading memory (``hgrn2``); a layer's feed-forward, if it has one, is dense with a
limited gate or a mixture of experts, some of them identities, with or without a shared one.

Its ``config.json`` lists the layers with their sizes; its tensors are ``l<i>.*``, ``embed``, ``final.norm`` and ``head``.
Projections that read one input, and the experts' like matrices, are stacked when the weights are loaded; the output projections
of a layer's mixer and of its dense or shared feed-forward are laid side by side.
"""

from __future__ import annotations

import dataclasses
from typing import Any

import numpy as np

from ..bf16 import bfloat16
from ..common import graph as iron
from ..common.declare import Precision
from ..lm.batched import BatchedLM
from ..lm.checkpoint import Renaming
from ..lm.config import LayerListConfig, rope_angles, yarn
from ..lm.mixers import ExpertsMLP, FadingMemory, GlobalAttention, SideBySideLayer

_MIXERS = ("attention", "hgrn2")
_FEED_FORWARDS = ("dense", "moe")
_SCALING = ("factor", "original", "fast", "slow")


@dataclasses.dataclass(frozen=True)
class PudinexConfig(LayerListConfig):
    """A Pudinex ``config.json``, and this package's own choices behind it.  ``layers`` keeps the file's
    entries.  The design bounds no positions; ``max_seq_len`` is how many a slot is served."""

    vocab_size: int
    hidden_size: int
    layers: tuple[dict, ...]
    eps: float
    norm_groups: int = 1
    embed_scale: float = 1.0
    max_seq_len: int = 131072
    prefill_chunk: int = 2048
    slots: int = 1
    activations: Any = bfloat16
    precision: Precision = Precision.HIGHEST

    ARCHITECTURE = "Pudinex"
    KEYS = {"vocab_size": ("vocab",), "hidden_size": ("width",), "layers": ("layers",), "eps": ("norm", "eps"), "norm_groups": ("norm", "groups"),
            "embed_scale": ("embedding", "scale")}

    def __post_init__(self):
        self.check_serving()
        self.check_layers(_MIXERS, _FEED_FORWARDS)
        if self.norm_groups < 1 or self.hidden_size % self.norm_groups:
            raise ValueError(f"PudinexConfig: a width of {self.hidden_size} is not {self.norm_groups} equal groups")


def feed_forward(spec: dict) -> tuple[dict | None, str, float]:
    """A layer's gated feed-forward that every row runs -- its sizes, the kind of its gate and the gate's limit: the dense one, or
    the shared expert."""
    mlp = spec.get("mlp") or {}
    if mlp.get("kind") == "dense":
        return mlp, "limited", mlp["limit"]
    return mlp.get("shared"), "silu", 0.0


class PudinexLayer(SideBySideLayer):
    """Layer ``i`` of the config.  ``tables`` holds the model's tables of angles by their constants."""

    tables: dict[tuple, iron.Weight] = {}

    def __init__(self, c: PudinexConfig, i: int):
        spec, m, width = c.layers[i], c.layers[i]["mixer"], c.hidden_size
        common = dict(eps=c.eps, dtype=c.activations)
        if spec["type"] == "attention":
            mixer = GlobalAttention(heads=m["heads"], kv_heads=m["kv_heads"], dim=m["dim"], vdim=m["vdim"], scale=m["scale"], cap=m.get("softcap") or 0.0,
                                    sink=True, value_norm=True, angles=self.table(m.get("rot"), c.max_seq_len), context=c.max_seq_len, **common)
        else:
            mixer = FadingMemory(heads=m["heads"], dim=m["dim"], vdim=m["vdim"], **common)
        routed, mlp = None, spec.get("mlp") or {}
        if mlp.get("kind") == "moe":
            r = mlp["router"]
            routed = ExpertsMLP(width, inner=mlp["expert"]["ff"], experts=r["experts"], identity=r.get("identity") or 0, top=r["top"], scored=True,
                                activation="silu", dtype=c.activations)
        every, kind, limit = feed_forward(spec)
        super().__init__(width, mixer, inner=every["ff"] if every else 0, kind=kind, limit=limit, routed=routed, groups=c.norm_groups,
                         precision=c.precision, **common)

    def table(self, rot: dict | None, positions: int) -> iron.Weight | None:
        if not rot or not rot["dims"]:
            return None
        dims, base, scaling = rot["dims"], rot["base"], rot.get("scaling")
        key = (dims, base, positions, *(scaling[n] for n in _SCALING)) if scaling else (dims, base, positions)
        if key not in self.tables:
            stretched, by = yarn(dims, base, **{n: scaling[n] for n in _SCALING}) if scaling else (None, 1.0)
            angles = rope_angles(dims, positions, base, stretched) * np.float32(by)
            self.tables[key] = iron.Weight((positions, dims), np.float32, angles)
        return self.tables[key]


def module_weights(config: PudinexConfig, weights) -> dict:
    """A checkpoint's tensors under the modules' names, those that are read together joined."""
    names = Renaming(weights, "Pudinex")
    put = names.put
    put("model.embed_tokens.weight", "embed")
    put("model.norm.weight", "final.norm")
    put("lm_head.weight", "head")
    for i, spec in enumerate(config.layers):
        src, dst = f"l{i}.", f"model.layers.{i}."
        mix, mlp = src + "mix.", spec.get("mlp") or {}
        every, at = feed_forward(spec)[0], src + ("mlp." if mlp.get("kind") == "dense" else "mlp.shared.")
        put(dst + "norm1.weight", src + "norm1")
        own = "qkv" if spec["type"] == "attention" else "qfv"
        put(dst + "proj.weight", *(mix + n for n in own), *((at + "gate", at + "up") if every else ()))
        put(dst + "out.weight", mix + "o", *((at + "down",) if every else ()), axis=1)
        if spec["type"] == "attention":
            for n in "qk":
                put(f"{dst}mixer.{n}_norm", f"{mix}{n}.norm")
        else:
            put(dst + "mixer.f_bias", mix + "f.b")
            put(dst + "mixer.lower", mix + "lower")
            put(dst + "mixer.norm", mix + "norm")
        if mlp.get("kind") == "moe":
            for n in ("gate", "up", "down"):
                put(f"{dst}routed.{n}", *(f"{src}mlp.e{e}.{n}" for e in range(mlp["router"]["experts"])))
            put(dst + "routed.router", src + "mlp.router")
            put(dst + "routed.correction", src + "mlp.correction")
    return names.done()


class Pudinex(BatchedLM):
    """Pudinex from a config and a checkpoint's tensors by name."""

    config_class = PudinexConfig

    def __init__(self, config: PudinexConfig, weights):
        self.layer_class = type("PudinexLayer", (PudinexLayer,), {"tables": {}})
        super().__init__(config, module_weights(config, weights))


def shapes(config: PudinexConfig) -> dict[str, tuple[int, ...]]:
    """Name -> shape of every tensor of a Pudinex checkpoint of this config."""
    width = config.hidden_size
    named: dict[str, tuple[int, ...]] = {"embed": (config.vocab_size, width)}

    def gated(at: str, ff: int) -> dict:
        return {at + "gate": (ff, width), at + "up": (ff, width), at + "down": (width, ff)}

    for i, spec in enumerate(config.layers):
        m, name, mix, mlp = spec["mixer"], f"l{i}.", f"l{i}.mix.", spec.get("mlp")
        H, D, V = m["heads"], m["dim"], m["vdim"]
        named |= {name + "norm1": (width,), mix + "q": (H * D, width), mix + "o": (width, H * V)}
        if spec["type"] == "attention":
            G = m["kv_heads"]
            named |= {mix + "k": (G * D, width), mix + "v": (G * V, width), mix + "q.norm": (D,), mix + "k.norm": (D,)}
        else:
            named |= {mix + "f": (H * D, width), mix + "f.b": (H * D,), mix + "lower": (H * D,), mix + "v": (H * V, width), mix + "norm": (V,)}
        if mlp is None:
            continue
        if mlp["kind"] == "dense":
            named |= gated(name + "mlp.", mlp["ff"])
            continue
        experts = mlp["router"]["experts"]
        outputs = experts + (mlp["router"].get("identity") or 0)
        for e in range(experts):
            named |= gated(f"{name}mlp.e{e}.", mlp["expert"]["ff"])
        named |= {name + "mlp.router": (outputs, width), name + "mlp.correction": (outputs,)}
        if mlp.get("shared"):
            named |= gated(name + "mlp.shared.", mlp["shared"]["ff"])
    named |= {"final.norm": (width,), "head": (config.vocab_size, width)}
    return named
