"""Pufuzen: a small pre-norm decoder around a float32 residual stream, whose layers mix tokens by a gated
recurrence (``mingru``), by windowed latent attention without positions (``latent_attention``), or by causal
latent attention with a rotated shared key part and a sink (``latent_attention_2``); a layer's feed-forward, if
it has one, activates by a polynomial of normed powers, and every sublayer joins the stream through a gate.

Its ``config.json`` lists the layers with their sizes; its tensors are ``l<i>.*``, ``embed``, ``final.norm`` and
``head``.  Projections that read one input, a sublayer's gate among them, are stacked when the weights are
loaded, and so are the two that expand a latent.
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
from ..lm.config import LayerListConfig, rope_angles
from ..lm.mixers import GatedRecurrence, GatedStreamLayer, LatentAttention, PolyNormMLP

_MIXERS = ("mingru", "latent_attention", "latent_attention_2")


@dataclasses.dataclass(frozen=True)
class PufuzenConfig(LayerListConfig):
    """A Pufuzen ``config.json``, and this package's own choices behind it.  ``layers`` keeps the file's
    entries.  The design bounds no positions; ``max_seq_len`` is how many a slot is served."""

    vocab_size: int
    hidden_size: int
    layers: tuple[dict, ...]
    eps: float
    logit_scale: float = 1.0
    max_seq_len: int = 131072
    prefill_chunk: int = 2048
    slots: int = 1
    activations: Any = bfloat16
    precision: Precision = Precision.HIGHEST

    ARCHITECTURE = "Pufuzen"
    KEYS = {"vocab_size": ("vocab",), "hidden_size": ("width",), "layers": ("layers",), "eps": ("norm", "eps"),
            "logit_scale": ("logit_scale",)}

    def __post_init__(self):
        self.check_serving()
        self.check_layers(_MIXERS)

    @property
    def key_room(self) -> int:
        """Keys a portion may attend in all: a longest sequence's, or several portions'."""
        return min(self.slots * self.max_seq_len, max(self.max_seq_len, 8 * self.prefill_chunk))


class PufuzenLayer(GatedStreamLayer):
    """Layer ``i`` of the config.  ``tables`` holds the model's tables of angles by their constants."""

    tables: dict[tuple, iron.Weight] = {}

    def __init__(self, c: PufuzenConfig, i: int):
        spec, m, width = c.layers[i], c.layers[i]["mixer"], c.hidden_size
        common = dict(gate=width, dtype=c.activations, precision=c.precision)
        if spec["type"] == "mingru":
            mixer = GatedRecurrence(width, inner=m["width"], **common)
        else:
            if spec["type"] == "latent_attention":
                own = {"window": m["mask"]["size"]}
            else:
                own = dict(rot=m["rot_dim"], angles=self.table(m["rot"]["dims"], m["rot"]["base"], c.max_seq_len), sink=True)
            mixer = LatentAttention(width, heads=m["heads"], dim=m["dim"], vdim=m["vdim"], q_rank=m["q_rank"], rank=m["kv_rank"],
                                    scale=m["scale"], eps=c.eps, context=c.max_seq_len, portion=c.prefill_chunk, room=c.key_room,
                                    **own, **common)
        mlp = spec.get("mlp")
        if mlp is not None:
            mlp = PolyNormMLP(width, inner=mlp["ff"], eps=c.eps, **common)
        super().__init__(width, mixer, mlp, eps=c.eps, dtype=c.activations)

    def table(self, dims: int, base: float, positions: int) -> iron.Weight:
        key = (dims, base, positions)
        if key not in self.tables:
            self.tables[key] = iron.Weight((positions, dims), np.float32, rope_angles(dims, positions, base))
        return self.tables[key]


def module_weights(config: PufuzenConfig, weights) -> dict:
    """A checkpoint's tensors under the modules' names, those that are read together joined."""
    names = Renaming(weights, "Pufuzen")
    put = names.put
    put("model.embed_tokens.weight", "embed")
    put("model.norm.weight", "final.norm")
    put("lm_head.weight", "head")
    for i, spec in enumerate(config.layers):
        src, dst = f"l{i}.", f"model.layers.{i}."
        mix = src + "mix."
        put(dst + "norm1.weight", src + "norm1")
        put(dst + "gate1_bias", src + "rg1.b")
        if spec["type"] == "mingru":
            put(dst + "mixer.proj.weight", *(mix + n for n in "zxg"), src + "rg1")
            for n in "zx":
                put(f"{dst}mixer.{n}_bias", f"{mix}{n}.b")
        else:
            put(dst + "mixer.proj.weight", mix + "dq", mix + "dkv", src + "rg1")
            put(dst + "mixer.q_norm", mix + "dq.norm")
            put(dst + "mixer.c_norm", mix + "dkv.norm")
            put(dst + "mixer.query.weight", mix + "uq")
            put(dst + "mixer.up", mix + "uk", mix + "uv")
            if spec["type"] == "latent_attention_2":
                put(dst + "mixer.sink", mix + "sink")
        put(dst + "mixer.out.weight", mix + "o")
        if spec.get("mlp") is None:
            for n in ("norm2", "rg2", "rg2.b"):
                names.drop(src + n)    # a layer without a feed-forward reads none
            continue
        put(dst + "norm2.weight", src + "norm2")
        put(dst + "gate2_bias", src + "rg2.b")
        put(dst + "mlp.proj.weight", src + "mlp.up", src + "rg2")
        put(dst + "mlp.bias", src + "mlp.up.b")
        put(dst + "mlp.act", src + "mlp.act")
        put(dst + "mlp.out.weight", src + "mlp.down")
        put(dst + "mlp.out_bias", src + "mlp.down.b")
    return names.done()


class Pufuzen(BatchedLM):
    """Pufuzen from a config and a checkpoint's tensors by name."""

    config_class = PufuzenConfig

    def __init__(self, config: PufuzenConfig, weights):
        self.layer_class = type("PufuzenLayer", (PufuzenLayer,), {"tables": {}})
        super().__init__(config, module_weights(config, weights))


def shapes(config: PufuzenConfig) -> dict[str, tuple[int, ...]]:
    """Name -> shape of every tensor of a Pufuzen checkpoint of this config."""
    width = config.hidden_size
    named: dict[str, tuple[int, ...]] = {"embed": (config.vocab_size, width)}
    for i, spec in enumerate(config.layers):
        m, name, mix = spec["mixer"], f"l{i}.", f"l{i}.mix."
        named |= {name + "norm1": (width,), name + "rg1": (width, width), name + "rg1.b": (width,)}
        if spec["type"] == "mingru":
            inner = m["width"]
            named |= {mix + n: (inner, width) for n in "zxg"}
            named |= {mix + "z.b": (inner,), mix + "x.b": (inner,), mix + "o": (width, inner)}
        else:
            rot = m.get("rot_dim", 0)
            named |= {mix + "dq": (m["q_rank"], width), mix + "dq.norm": (m["q_rank"],),
                      mix + "uq": (m["heads"] * (m["dim"] + rot), m["q_rank"]), mix + "dkv": (m["kv_rank"] + rot, width),
                      mix + "dkv.norm": (m["kv_rank"],), mix + "uk": (m["heads"] * m["dim"], m["kv_rank"]),
                      mix + "uv": (m["heads"] * m["vdim"], m["kv_rank"]), mix + "o": (width, m["heads"] * m["vdim"])}
            if spec["type"] == "latent_attention_2":
                named |= {mix + "sink": (m["heads"],)}
        if spec.get("mlp") is not None:
            ff = spec["mlp"]["ff"]
            named |= {name + "norm2": (width,), name + "rg2": (width, width), name + "rg2.b": (width,),
                      name + "mlp.up": (ff, width), name + "mlp.up.b": (ff,), name + "mlp.act": (4,),
                      name + "mlp.down": (width, ff), name + "mlp.down.b": (width,)}
    named |= {"final.norm": (width,), "head": (config.vocab_size, width)}
    return named
