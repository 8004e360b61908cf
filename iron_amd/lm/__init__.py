"""A decoder-only language model wired from the hot-path operators (iron/lm/__init__.py)."""

from .batched import Batch, BatchedLM, Entry, SlotSession
from .blocks import (
    Attention,
    DecoderLayer,
    Embedding,
    GatedMLP,
    KVCache,
    Linear,
    PleLayer,
    RMSNorm,
    Rope,
    SandwichLayer,
    activation,
    residual_add,
)
from .causal import Call, CausalLM, Decoder, Stats
from .checkpoint import Checkpoint, weights_file, write_safetensors
from .config import DecoderConfig, LayerListConfig, rope_angles
from .generation import Sampler
from .mixers import (
    ActivatedMLP,
    DeltaMixer,
    ExpertsMLP,
    GatedRecurrence,
    GatedStreamLayer,
    LatentAttention,
    MatrixMemoryMixer,
    ParallelMixer,
    PolyNormMLP,
    PostNormLayer,
    StreamLayer,
    StreamRMSNorm,
    TalkingAttention,
    TimeMixing,
    WindowAttention,
)
from .session import Session

__all__ = [
    "ActivatedMLP", "Attention", "Batch", "BatchedLM", "Call", "CausalLM", "Checkpoint", "Decoder", "DecoderConfig",
    "DecoderLayer", "DeltaMixer", "Embedding", "Entry", "ExpertsMLP", "GatedMLP", "GatedRecurrence",
    "GatedStreamLayer", "KVCache", "LatentAttention", "LayerListConfig", "Linear", "MatrixMemoryMixer",
    "ParallelMixer", "PleLayer", "PolyNormMLP", "PostNormLayer", "RMSNorm", "Rope", "Sampler", "SandwichLayer",
    "Session", "SlotSession", "Stats", "StreamLayer", "StreamRMSNorm", "TalkingAttention", "TimeMixing",
    "WindowAttention", "activation", "residual_add", "rope_angles", "weights_file", "write_safetensors",
]
