"""Tilarax: a small decoder around a float32 residual stream whose blocks read the stream itself and are normed where they
join it, each layer followed by a weighted average over the results of all layers so far.  Layers mix tokens by attention
within chunks (``attention``: heads mix their softmax weights, values may be blended with the first such layer's) or by a
matrix memory (``mlstm``); a layer's feed-forward, if it has one, is dense or a mixture of experts.

Its ``config.json`` lists the layers with their sizes; its tensors are ``l<i>.*``, ``embed`` (the output projection too) and
``final.norm``.  Projections that read one input, and the experts' like matrices, are stacked when the weights are loaded.
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
from ..lm.mixers import ActivatedMLP, ExpertsMLP, MatrixMemoryMixer, PostNormLayer, TalkingAttention

_MIXERS = ("attention", "mlstm")
_FEED_FORWARDS = ("dense", "moe")


@dataclasses.dataclass(frozen=True)
class TilaraxConfig(LayerListConfig):
    """A Tilarax ``config.json``, and this package's own choices behind it.  ``layers`` keeps the file's
    entries.  The design bounds no positions; ``max_seq_len`` is how many a slot is served."""

    vocab_size: int
    hidden_size: int
    layers: tuple[dict, ...]
    eps: float
    max_seq_len: int = 131072
    prefill_chunk: int = 2048
    slots: int = 1
    activations: Any = bfloat16
    precision: Precision = Precision.HIGHEST

    ARCHITECTURE = "Tilarax"
    KEYS = {"vocab_size": ("vocab",), "hidden_size": ("width",), "layers": ("layers",), "eps": ("norm", "eps")}

    tie_word_embeddings = True
    norm_unit = 1.0
    looks_back = True

    def __post_init__(self):
        self.check_serving()
        self.check_layers(_MIXERS, _FEED_FORWARDS)
        mixing = [s["mixer"] for s in self.layers if s["type"] == "attention" and s["mixer"].get("v_mix")]
        if len({(m["kv_heads"], m["vdim"]) for m in mixing}) > 1:
            raise ValueError("TilaraxConfig: layers that blend their values have as many heads of as many")


class TilaraxLayer(PostNormLayer):
    """Layer ``i`` of the config.  ``tables`` holds the model's tables of angles by their constants."""

    tables: dict[tuple, iron.Weight] = {}

    def __init__(self, c: TilaraxConfig, i: int):
        spec, m, width = c.layers[i], c.layers[i]["mixer"], c.hidden_size
        common = dict(eps=c.eps, dtype=c.activations, precision=c.precision)
        if spec["type"] == "attention":
            rot = m.get("rot") or {"dims": 0}
            angles = self.table(rot["dims"], rot["base"], c.max_seq_len) if rot["dims"] else None
            mixer = TalkingAttention(width, heads=m["heads"], kv_heads=m["kv_heads"], dim=m["dim"], vdim=m["vdim"], chunk=m["mask"]["size"],
                                     scale=m["scale"], context=c.max_seq_len, angles=angles, mixes=bool(m.get("v_mix")), **common)
        else:
            mixer = MatrixMemoryMixer(width, heads=m["heads"], dim=m["dim"], vdim=m["vdim"], cap=m["gate_cap"], **common)
        mlp = spec.get("mlp")
        if mlp is not None and mlp["kind"] == "dense":
            mlp = ActivatedMLP(width, inner=mlp["ff"], activation="gelu_tanh", dtype=c.activations, precision=c.precision)
        elif mlp is not None:
            mlp = ExpertsMLP(width, inner=mlp["expert"]["ff"], experts=mlp["router"]["experts"], top=mlp["router"]["top"], activation="silu",
                             dtype=c.activations)
        super().__init__(width, mixer, mlp, index=i, eps=c.eps, dtype=c.activations, unit=c.norm_unit)

    def table(self, dims: int, base: float, positions: int) -> iron.Weight:
        key = (dims, base, positions)
        if key not in self.tables:
            self.tables[key] = iron.Weight((positions, dims), np.float32, rope_angles(dims, positions, base))
        return self.tables[key]


def module_weights(config: TilaraxConfig, weights) -> dict:
    """A checkpoint's tensors under the modules' names, those that are read together joined."""
    names = Renaming(weights, "Tilarax")
    put = names.put
    put("model.embed_tokens.weight", "embed")
    put("model.norm.weight", "final.norm")
    for i, spec in enumerate(config.layers):
        src, dst = f"l{i}.", f"model.layers.{i}."
        mix, mlp = src + "mix.", spec.get("mlp")
        put(dst + "norm1.weight", src + "norm1")
        put(dst + "depth", src + "dwa")
        if spec["type"] == "attention":
            put(dst + "mixer.proj.weight", *(mix + n for n in "qkv"))
            put(dst + "mixer.bias", *(f"{mix}{n}.b" for n in "qkv"))
            for n in "qk":
                put(f"{dst}mixer.{n}_norm", f"{mix}{n}.norm")
            put(dst + "mixer.temp", mix + "temp")
            put(dst + "mixer.talk", mix + "talk")
            if spec["mixer"].get("v_mix"):
                names.named[dst + "mixer.share"] = names.take(mix + "vmix").reshape(1)
            else:
                names.drop(mix + "vmix")
            put(dst + "mixer.out_bias", mix + "o.b")
        else:
            put(dst + "mixer.proj.weight", *(mix + n for n in "qkvgif"))
            for n in "if":
                put(f"{dst}mixer.{n}_bias", f"{mix}{n}.b")
            put(dst + "mixer.norm", mix + "norm")
        put(dst + "mixer.out.weight", mix + "o")
        if mlp is None:
            names.drop(src + "norm2")    # a layer without a feed-forward reads none
            continue
        put(dst + "norm2.weight", src + "norm2")
        if mlp["kind"] == "dense":
            for n in ("up", "down"):
                put(f"{dst}mlp.{n}.weight", f"{src}mlp.{n}")
            continue
        for n in ("gate", "up", "down"):
            put(f"{dst}mlp.{n}", *(f"{src}mlp.e{e}.{n}" for e in range(mlp["router"]["experts"])))
        put(dst + "mlp.router", src + "mlp.router")
        put(dst + "mlp.router_bias", src + "mlp.router.b")
    return names.done()


class Tilarax(BatchedLM):
    """Tilarax from a config and a checkpoint's tensors by name."""

    config_class = TilaraxConfig

    def __init__(self, config: TilaraxConfig, weights):
        self.layer_class = type("TilaraxLayer", (TilaraxLayer,), {"tables": {}})
        super().__init__(config, module_weights(config, weights))


def shapes(config: TilaraxConfig) -> dict[str, tuple[int, ...]]:
    """Name -> shape of every tensor of a Tilarax checkpoint of this config."""
    width = config.hidden_size
    named: dict[str, tuple[int, ...]] = {"embed": (config.vocab_size, width)}
    for i, spec in enumerate(config.layers):
        m, name, mix, mlp = spec["mixer"], f"l{i}.", f"l{i}.mix.", spec.get("mlp")
        H, D, V = m["heads"], m["dim"], m["vdim"]
        named |= {name + "norm1": (width,), name + "dwa": (i + 2,), mix + "o": (width, H * V)}
        if spec["type"] == "attention":
            G = m["kv_heads"]
            for n, rows in (("q", H * D), ("k", G * D), ("v", G * V)):
                named |= {mix + n: (rows, width), f"{mix}{n}.b": (rows,)}
            named |= {mix + "q.norm": (D,), mix + "k.norm": (D,), mix + "vmix": (), mix + "talk": (H, H), mix + "temp": (H,),
                      mix + "o.b": (width,)}
        else:
            for n, rows in (("q", H * D), ("k", H * D), ("v", H * V), ("g", H * V), ("i", H), ("f", H)):
                named |= {mix + n: (rows, width)}
            named |= {mix + "i.b": (H,), mix + "f.b": (H,), mix + "norm": (H * V,)}
        if mlp is None:
            continue
        named |= {name + "norm2": (width,)}
        if mlp["kind"] == "dense":
            named |= {name + "mlp.up": (mlp["ff"], width), name + "mlp.down": (width, mlp["ff"])}
            continue
        ff, experts = mlp["expert"]["ff"], mlp["router"]["experts"]
        for e in range(experts):
            named |= {f"{name}mlp.e{e}.{n}": (ff, width) for n in ("gate", "up")} | {f"{name}mlp.e{e}.down": (width, ff)}
        named |= {name + "mlp.router": (experts, width), name + "mlp.router.b": (experts,)}
    named |= {"final.norm": (width,)}
    return named
