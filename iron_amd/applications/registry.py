"""Which model class a checkpoint's ``config.json`` asks for."""

from __future__ import annotations

import json
from pathlib import Path

from .gemma4 import Gemma4
from .granite import Granite
from .llama import Llama
from .pegilix import Pegilix
from .pudinex import Pudinex
from .pufuzen import Pufuzen
from .tilarax import Tilarax

# ``architecture`` (or an entry of ``architectures``) -> the class that serves it
ARCHITECTURES = {
    "LlamaForCausalLM": Llama,
    "GraniteForCausalLM": Granite,
    "Gemma4ForCausalLM": Gemma4,
    "Gemma4ForConditionalGeneration": Gemma4,
    "Pegilix": Pegilix,
    "Pudinex": Pudinex,
    "Pufuzen": Pufuzen,
    "Tilarax": Tilarax,
}


def model_class(path):
    """The class for the checkpoint directory ``path``.

    Raises:
        FileNotFoundError: it holds no ``config.json``.
        ValueError: no class here serves the architecture that names.
    """
    data = json.loads((Path(path) / "config.json").read_text())
    named = [data["architecture"]] if "architecture" in data else list(data.get("architectures") or [])
    for name in named:
        if name in ARCHITECTURES:
            return ARCHITECTURES[name]
    raise ValueError(f"{path}: architecture {named or 'unnamed'}: one of {sorted(ARCHITECTURES)} is served here")


def load_model(path, **options):
    """``model_class(path).load(path, **options)``: the checkpoint, ready to generate."""
    return model_class(path).load(path, **options)
