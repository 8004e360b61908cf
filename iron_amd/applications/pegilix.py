"""Pegilix: a small decoder whose layers mix tokens either by sliding-window attention and time mixing
side by side (``parallel``) or by the gated delta rule (``delta``), each layer a sandwich around a
float32 residual stream; a run of layers may be repeated with the same weights, a state to each pass.

Its ``config.json`` lists the layers with their sizes; its tensors are ``l<i>.*``, ``embed``,
``final.norm`` and ``head``.  Projections that read one input are stacked when the weights are loaded,
and the two output projections of a parallel layer are laid side by side.
"""

from __future__ import annotations

import dataclasses
from types import SimpleNamespace
from typing import Any

import numpy as np

from ..bf16 import bfloat16, from_torch
from ..common.declare import Precision
from ..lm.batched import BatchedLM
from ..lm.blocks import GatedMLP
from ..lm.checkpoint import Renaming, joined
from ..lm.config import LayerListConfig
from ..lm.mixers import DeltaMixer, ParallelMixer, StreamLayer, TimeMixing, WindowAttention

_MIXERS = ("parallel", "delta")


@dataclasses.dataclass(frozen=True)
class PegilixConfig(LayerListConfig):
    """A Pegilix ``config.json``, and this package's own choices behind it.  ``layers`` keeps the file's
    entries.  The design bounds no positions; ``max_seq_len`` is how many a slot is served."""

    vocab_size: int
    hidden_size: int
    layers: tuple[dict, ...]
    eps: float
    loop: dict | None = None
    logit_softcap: float | None = None
    max_seq_len: int = 131072
    prefill_chunk: int = 2048
    slots: int = 1
    activations: Any = bfloat16
    precision: Precision = Precision.HIGHEST

    ARCHITECTURE = "Pegilix"
    KEYS = {"vocab_size": ("vocab",), "hidden_size": ("width",), "layers": ("layers",), "eps": ("norm", "eps"),
            "loop": ("loop",), "logit_softcap": ("logit_softcap",)}

    def __post_init__(self):
        self.check_serving()
        self.check_layers(_MIXERS)
        if self.loop is not None and not 0 <= self.loop["start"] <= self.loop["stop"] <= len(self.layers):
            raise ValueError(f"PegilixConfig: loop {self.loop} of {len(self.layers)} layers")

    @property
    def order(self) -> list[int]:
        """Layer indices in the order they run."""
        indices, loop = list(range(len(self.layers))), self.loop
        if loop is None:
            return indices
        return indices[: loop["start"]] + indices[loop["start"] : loop["stop"]] * loop["times"] + indices[loop["stop"] :]


class PegilixLayer(StreamLayer):
    """Layer ``i`` of the config.  A bias table's rows and a decay's rank are the checkpoint's: ``tables``
    gives them by layer."""

    tables: list[dict] = []

    def __init__(self, c: PegilixConfig, i: int):
        spec, m = c.layers[i], c.layers[i]["mixer"]
        common = dict(dtype=c.activations, precision=c.precision)
        if spec["type"] == "parallel":
            left, right, sizes = m["left"], m["right"], self.tables[i]
            mixer = ParallelMixer(
                c.hidden_size,
                WindowAttention(c.hidden_size, heads=left["heads"], kv_heads=left["kv_heads"], dim=left["dim"],
                                vdim=left["vdim"], window=left["mask"]["size"], bias_rows=sizes["bias_rows"],
                                bias_max=left["bias_max"], scale=left["scale"], context=c.max_seq_len,
                                out_scale=m["left_scale"], **common),
                TimeMixing(c.hidden_size, heads=right["heads"], dim=right["dim"], rank=sizes["rank"], eps=c.eps,
                           out_scale=m["right_scale"], **common),
                precision=c.precision)
        else:
            mixer = DeltaMixer(c.hidden_size, heads=m["heads"], kv_heads=m["kv_heads"], dim=m["dim"], vdim=m["vdim"],
                               taps=m["conv"], eps=c.eps, **common)
        mlp = spec.get("mlp")
        if mlp is not None:
            mlp = GatedMLP(SimpleNamespace(hidden_size=c.hidden_size, intermediate_size=mlp["ff"], mlp_bias=False,
                                           hidden_act="relu", precision=c.precision))
        super().__init__(c.hidden_size, mixer, mlp, eps=c.eps, dtype=c.activations)


def _as_float32(weight) -> np.ndarray:
    is_torch = type(weight).__module__.split(".")[0] == "torch"
    return from_torch(weight) if is_torch else np.asarray(weight, dtype=np.float32)


def module_weights(config: PegilixConfig, weights) -> dict:
    """A checkpoint's tensors under the modules' names, those that are read together joined."""
    names = Renaming(weights, "Pegilix")
    put, take = names.put, names.take
    put("model.embed_tokens.weight", "embed")
    put("model.norm.weight", "final.norm")
    put("lm_head.weight", "head")
    for i, spec in enumerate(config.layers):
        src, dst = f"l{i}.", f"model.layers.{i}."
        norms = ("norm1", "norm1b", "norm2", "norm2b") if spec.get("mlp") is not None else ("norm1", "norm1b")
        for norm in norms:
            put(f"{dst}{norm}.weight", src + norm)
        if spec.get("mlp") is None:
            for norm in ("norm2", "norm2b"):
                names.drop(src + norm)    # a layer without a feed-forward reads none
        else:
            for part in ("gate", "up", "down"):
                put(f"{dst}mlp.{part}_proj.weight", f"{src}mlp.{part}")
        src, dst = src + "mix.", dst + "mixer."
        if spec["type"] == "parallel":
            put(dst + "left.qkv.weight", *(f"{src}left.{n}" for n in "qkv"))
            put(dst + "left.rel", src + "left.rel")
            put(dst + "out.weight", src + "left.o", src + "right.o", axis=1)
            mus = [take(f"{src}right.mu.{n}") for n in TimeMixing.BLENDS]
            names.named[dst + "right.mu"] = joined([mu.reshape(1, -1) for mu in mus], 0)
            for n in ("r", "k", "v", "g", "w1"):
                put(f"{dst}right.{n}.weight", f"{src}right.{n}")
            for n in ("w2", "w0", "u", "norm"):
                put(f"{dst}right.{n}", f"{src}right.{n}")
        else:
            put(dst + "proj.weight", *(src + n for n in ("q", "k", "v", "g", "b", "a")))
            put(dst + "conv", *(f"{src}{n}.conv" for n in "qkv"))
            put(dst + "a_log", src + "A_log")
            put(dst + "dt_bias", src + "dt_bias")
            put(dst + "norm", src + "norm")
            put(dst + "out.weight", src + "o")
    return names.done()


class Pegilix(BatchedLM):
    """Pegilix from a config and a checkpoint's tensors by name."""

    config_class = PegilixConfig

    def __init__(self, config: PegilixConfig, weights):
        tables = []
        for i, spec in enumerate(config.layers):
            name = f"l{i}.mix."
            tables.append({"bias_rows": int(weights[name + "left.rel"].shape[0]),
                           "rank": int(weights[name + "right.w1"].shape[0])} if spec["type"] == "parallel" else {})
        self.layer_class = type("PegilixLayer", (PegilixLayer,), {"tables": tables})
        super().__init__(config, module_weights(config, weights))
        for block in self.layers:
            block.mixer.loaded(_as_float32)


def shapes(config: PegilixConfig, bias_rows: int = 32, rank: int = 64) -> dict[str, tuple[int, ...]]:
    """Name -> shape of every tensor of a Pegilix checkpoint of this config."""
    width = config.hidden_size
    named: dict[str, tuple[int, ...]] = {"embed": (config.vocab_size, width)}
    for i, spec in enumerate(config.layers):
        m, name = spec["mixer"], f"l{i}."
        named |= {name + n: (width,) for n in ("norm1", "norm1b")}
        if spec["type"] == "parallel":
            left, right = m["left"], m["right"]
            H, G = left["heads"], left["kv_heads"]
            inner = right["heads"] * right["dim"]
            at = name + "mix.left."
            named |= {at + "q": (H * left["dim"], width), at + "k": (G * left["dim"], width), at + "v": (G * left["vdim"], width),
                      at + "rel": (bias_rows, H), at + "o": (width, H * left["vdim"])}
            at = name + "mix.right."
            named |= {f"{at}mu.{n}": (width,) for n in TimeMixing.BLENDS}
            named |= {at + n: (inner, width) for n in "rkvg"}
            named |= {at + "w1": (rank, width), at + "w2": (inner, rank), at + "w0": (inner,), at + "norm": (inner,),
                      at + "u": (right["heads"], right["dim"]), at + "o": (width, inner)}
        else:
            H, G, at = m["heads"], m["kv_heads"], name + "mix."
            for n, rows in (("q", G * m["dim"]), ("k", G * m["dim"]), ("v", H * m["vdim"])):
                named |= {at + n: (rows, width), f"{at}{n}.conv": (rows, m["conv"])}
            named |= {at + "b": (H, width), at + "a": (H, width), at + "A_log": (H,), at + "dt_bias": (H,),
                      at + "norm": (m["vdim"],), at + "g": (H * m["vdim"], width), at + "o": (width, H * m["vdim"])}
        if spec.get("mlp") is not None:
            ff = spec["mlp"]["ff"]
            named |= {name + n: (width,) for n in ("norm2", "norm2b")}
            named |= {name + "mlp.gate": (ff, width), name + "mlp.up": (ff, width), name + "mlp.down": (width, ff)}
    named |= {"final.norm": (width,), "head": (config.vocab_size, width)}
    return named
