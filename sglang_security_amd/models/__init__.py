"""Model registry.

ARCHITECTURES: checkpoint-loaded models by the architecture their config.json names; each class takes (config, weights,
dtype, device, max_context) and runs engine.StepBatch steps over a mem_cache.HybridCache.
SYNTHETIC: named configurations of the decode-step runners (random weights), by the name bench.py and the tools use.
"""
from __future__ import annotations

import importlib

ARCHITECTURES = {
    "Lusatar": ("sglang_security_amd.models.lusatar", "Lusatar"),
    "Kazedra": ("sglang_security_amd.models.kazedra", "Kazedra"),
}

# the kernel sources an architecture's steps launch beside those of every engine-served model
COMMON_SOURCES = ("core.hip", "gemm_dense.hip", "residual_norm.hip")
SAMPLING_SOURCES = ("elementwise.hip", "sampling.hip")
SOURCES = {
    "Lusatar": ("latent_attention.hip", "rglru.hip"),
    "Kazedra": ("tied_attention.hip", "delta_rule.hip"),
}

SYNTHETIC = {
    "llama3-8b": ("sglang_security_amd.decode_runner", "LlamaConfig", "llama3_8b"),
    "llama3-70b-tp8-rank": ("sglang_security_amd.decode_runner", "LlamaConfig", "llama3_70b_tp8_rank"),
    "qwen2-0.5b": ("sglang_security_amd.decode_runner", "LlamaConfig", "qwen2_0_5b"),
    "deepseek-v3-dense": ("sglang_security_amd.mla_runner", "DeepseekV3Config", "deepseek_v3"),
}


def architecture_of(config: dict) -> str:
    name = config.get("architecture") or (config.get("architectures") or [None])[0]
    if not name:
        raise ValueError("config.json names no architecture")
    return name


def model_class(config: dict):
    """The model class for a checkpoint's configuration."""
    name = architecture_of(config)
    if name not in ARCHITECTURES:
        raise ValueError(f"unknown architecture {name!r}; known: {', '.join(sorted(ARCHITECTURES))}")
    module, cls = ARCHITECTURES[name]
    return getattr(importlib.import_module(module), cls)


def kernel_sources(config: dict):
    """What a checkout without a built library has to compile to step this model."""
    model_class(config)
    return COMMON_SOURCES + SOURCES[architecture_of(config)]


def synthetic_config(name: str, *args):
    module, cls, factory = SYNTHETIC[name]
    return getattr(getattr(importlib.import_module(module), cls), factory)(*args)


def load_model(folder: str, dtype, device, max_context: int):
    """Configuration and weights of a checkpoint folder -> the model, ready for an engine."""
    from ..model_loader import load_config, load_weights

    config = load_config(folder)
    cls = model_class(config)
    weights = load_weights(folder, dtype, device)
    model = cls(config, weights, dtype, device, max_context)
    weights.check_all_used()
    return model
