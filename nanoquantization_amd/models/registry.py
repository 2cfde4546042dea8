"""Which model class, weights and engine a checkpoint directory stands for, by its config.json."""
from __future__ import annotations

import json
import os
from dataclasses import dataclass
from typing import Callable, List

import torch


@dataclass(frozen=True)
class Architecture:
    name: str
    matches: Callable[[dict], bool]
    load: Callable[[str, dict, torch.dtype], "torch.nn.Module"]      # (directory, config, dtype) -> model on the CPU
    engine: Callable[[], type]                                       # the EngineCore subclass that runs it
    step_kernels: str                                                # the native library its engine needs


def _load_hybrid(cls, spec_from_config, path: str, cfg: dict, dtype: torch.dtype):
    from ..utils.loader import load_views, tensor_shapes
    model = cls(spec_from_config(cfg, tensor_shapes(path))).to(dtype)
    load_views(model, path)
    return model


def _load_gafulix(path: str, cfg: dict, dtype: torch.dtype):
    from .gafulix import GafulixForCausalLM, spec_from_config
    return _load_hybrid(GafulixForCausalLM, spec_from_config, path, cfg, dtype)


def _load_roletar(path: str, cfg: dict, dtype: torch.dtype):
    from .roletar import RoletarForCausalLM, spec_from_config
    return _load_hybrid(RoletarForCausalLM, spec_from_config, path, cfg, dtype)


def _load_qwen3(path: str, cfg: dict, dtype: torch.dtype):
    from ..utils.loader import load_model
    from .qwen3_quantized import Qwen3QuantizedForCausalLM
    q = cfg["quantization_config"]
    model = Qwen3QuantizedForCausalLM(
        num_hidden_layers=cfg["num_hidden_layers"], vocab_size=cfg["vocab_size"], hidden_size=cfg["hidden_size"],
        total_num_heads=cfg["num_attention_heads"], total_num_kv_heads=cfg["num_key_value_heads"],
        max_position_embeddings=cfg["max_position_embeddings"], intermediate_size=cfg["intermediate_size"],
        w_bits=q["w_bits"], group_size=q["group_size"], head_dim=cfg.get("head_dim"),
        tie_word_embeddings=cfg.get("tie_word_embeddings", False), rope_theta=cfg.get("rope_theta", 10000),
        rms_norm_eps=cfg.get("rms_norm_eps", 1e-6))
    model = model.to(dtype)
    load_model(model, path)
    return model


def _hybrid_engine():
    from ..engine.hybrid_engine import HybridEngine
    return HybridEngine


def _awq_engine():
    from ..engine.llm_engine import LLMEngine
    return LLMEngine


ARCHITECTURES: List[Architecture] = [
    Architecture("Gafulix", lambda c: c.get("architecture") == "Gafulix", _load_gafulix, _hybrid_engine, "hybrid"),
    Architecture("Roletar", lambda c: c.get("architecture") == "Roletar", _load_roletar, _hybrid_engine, "hybrid"),
    # Qwen3 with AWQ linears: the reference's checkpoints carry a quantization_config and no further mark
    Architecture("Qwen3Quantized", lambda c: "quantization_config" in c and "architecture" not in c, _load_qwen3,
                 _awq_engine, "awq"),
]


def read_config(path: str) -> dict:
    with open(os.path.join(path, "config.json")) as f:
        return json.load(f)


def find_architecture(cfg: dict) -> Architecture:
    for arch in ARCHITECTURES:
        if arch.matches(cfg):
            return arch
    raise ValueError("config.json names no known architecture (known: " + ", ".join(a.name for a in ARCHITECTURES) + ")")


def load_pretrained(path: str, device="cpu", dtype: torch.dtype = torch.bfloat16):
    """The model of a checkpoint directory, its weights loaded."""
    cfg = read_config(path)
    return find_architecture(cfg).load(path, cfg, dtype).to(device)


def engine_for(model):
    """The engine class that runs a model made by this package."""
    from .hybrid import HybridDecoder
    return _hybrid_engine() if isinstance(model, HybridDecoder) else _awq_engine()
