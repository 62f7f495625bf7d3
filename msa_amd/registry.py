"""Model registry: architecture name of a folder's ``config.json`` -> configuration and model class."""
from __future__ import annotations

import json
import os
from typing import Callable, Dict

import torch

from .config import HybridConfig, MSAConfig, PostNormConfig
from .weights import load_tensors


def _build_hybrid(config: dict, tensors, dtype, device):
    from .hybrid import HybridForCausalLM
    return HybridForCausalLM.from_tensors(HybridConfig.from_dict(config), tensors, dtype, device)


def _build_postnorm(config: dict, tensors, dtype, device):
    from .postnorm import PostNormForCausalLM
    return PostNormForCausalLM.from_tensors(PostNormConfig.from_dict(config), tensors, dtype, device)


def _build_msa(config: dict, tensors, dtype, device):
    from .model import MSAForCausalLM
    names = set(MSAConfig.__dataclass_fields__)
    with torch.device(device):
        model = MSAForCausalLM(MSAConfig(**{k: v for k, v in config.items() if k in names})).to(dtype)
    if "lm_head.weight" not in tensors and config.get("tie_word_embeddings"):
        tensors["lm_head.weight"] = tensors["model.embed_tokens.weight"]
    model.load_state_dict(tensors)
    return model.eval()


# architecture -> builder(config dict, {name: tensor}, dtype, device)
ARCHITECTURES: Dict[str, Callable] = {"Gevonex": _build_hybrid, "Sugizen": _build_postnorm, "MSAForCausalLM": _build_msa}


def architecture(config: dict) -> str:
    name = config.get("architecture") or (config.get("architectures") or [None])[0]
    if name not in ARCHITECTURES:
        raise NotImplementedError(f"unknown architecture {name!r} (known: {sorted(ARCHITECTURES)})")
    return name


def read_config(model_dir: str) -> dict:
    with open(os.path.join(model_dir, "config.json")) as f:
        return json.load(f)


def load_model(model_dir: str, dtype: torch.dtype = torch.bfloat16, device="cuda:0"):
    """The model a folder's ``config.json`` names, with its weights on ``device``."""
    config = read_config(model_dir)
    return ARCHITECTURES[architecture(config)](config, load_tensors(model_dir), dtype, device)
