"""Model registry: the architecture a checkpoint folder's config.json names -> how to load it.

Folders with a HuggingFace config (`architectures`) go through transformers and init_engine's layer
replacement; native designs (`architecture`) are built directly."""
import json
import os
from typing import Callable, Dict, Type

import torch

from ...engineconfig import MuiEngineConfig
from .native import MuiNativeForCausalLM
from .salepel.config import ARCHITECTURE as SALEPEL
from .salepel.model import MuiSalepelForCausalLM
from .zufadra.config import ARCHITECTURE as ZUFADRA
from .zufadra.model import MuiZufadraForCausalLM


def _load_hf(path: str, dtype, device, engine_config: MuiEngineConfig):
    from transformers import AutoModelForCausalLM

    from ...engine import init_engine

    model = AutoModelForCausalLM.from_pretrained(path, torch_dtype=dtype, local_files_only=True)
    return init_engine(model, device=device, engine_config=engine_config)


def _native(cls: Type[MuiNativeForCausalLM]) -> Callable:
    def load(path: str, dtype, device, engine_config: MuiEngineConfig):
        return cls.from_pretrained(path, dtype=dtype, device=device, engine_config=engine_config)

    return load


MODEL_LOADERS: Dict[str, Callable] = {
    "LlamaForCausalLM": _load_hf,
    "MistralForCausalLM": _load_hf,
    SALEPEL: _native(MuiSalepelForCausalLM),
    ZUFADRA: _native(MuiZufadraForCausalLM),
}


def architecture_of(path: str) -> str:
    with open(os.path.join(path, "config.json")) as f:
        cfg = json.load(f)
    name = cfg.get("architecture") or (cfg.get("architectures") or [None])[0]
    if name not in MODEL_LOADERS:
        raise ValueError(f"{path}: architecture {name!r} is none of {sorted(MODEL_LOADERS)}")
    return name


def load_model(path: str, dtype: torch.dtype = torch.bfloat16, device="cuda", engine_config: MuiEngineConfig = None):
    """The causal LM of a checkpoint folder, ready for generate() or step-by-step forward()."""
    loader = MODEL_LOADERS[architecture_of(path)]
    return loader(path, dtype, device, engine_config or MuiEngineConfig())
