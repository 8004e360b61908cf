"""The models wired from the shared decoder: Llama, Granite, Gemma 4's text decoder, Pegilix, Pudinex,
Pufuzen and Tilarax."""

from .gemma4 import Gemma4, Gemma4Config
from .granite import Granite, GraniteConfig
from .llama import Llama, LlamaConfig
from .pegilix import Pegilix, PegilixConfig
from .pudinex import Pudinex, PudinexConfig
from .pufuzen import Pufuzen, PufuzenConfig
from .registry import ARCHITECTURES, load_model, model_class
from .tilarax import Tilarax, TilaraxConfig

__all__ = ["ARCHITECTURES", "Gemma4", "Gemma4Config", "Granite", "GraniteConfig", "Llama", "LlamaConfig", "Pegilix",
           "PegilixConfig", "Pudinex", "PudinexConfig", "Pufuzen", "PufuzenConfig", "Tilarax", "TilaraxConfig", "load_model", "model_class"]
