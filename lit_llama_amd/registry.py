"""Model families and how a checkpoint finds its own.

A folder with config.json names its family under `architecture`; a bare lit-llama checkpoint (`.pth`) is a LLaMA of the size its
embedding says (utils.llama_model_lookup).  `load_model` returns a model on the GPU that `generate` and `batching.generate_batch` serve.
"""
from __future__ import annotations

import json
from pathlib import Path
from typing import Callable, Dict, Optional

import torch

from .checkpoint import lazy_load


def _hybrid(config: dict, dtype: torch.dtype, device):
    from .hybrid import HybridConfig, HybridLM

    return HybridLM(HybridConfig.from_dict(config), dtype=dtype, device=device)


def _llama(config: dict, dtype: torch.dtype, device, quantize: Optional[str] = None):
    from .model import LLaMA, LLaMAConfig
    from .utils import EmptyInitOnDevice

    kw = {k: v for k, v in config.items() if k in LLaMAConfig.__dataclass_fields__}
    with EmptyInitOnDevice(device=device, dtype=dtype, quantization_mode=quantize):
        return LLaMA(LLaMAConfig(**kw)).eval()


FAMILIES: Dict[str, Callable] = {"LLaMA": _llama, "Sekulorn": _hybrid, "Kovalorn": _hybrid, "Kudazen": _hybrid, "Gurolix": _hybrid}


def build_model(config: dict, dtype: torch.dtype = torch.bfloat16, device="cuda", **kw):
    """An empty model of the family `config["architecture"]` names."""
    name = config.get("architecture")
    if name not in FAMILIES:
        raise ValueError(f"unknown architecture {name!r} (known: {sorted(FAMILIES)})")
    return FAMILIES[name](config, dtype, device, **kw)


def load_model(path, dtype: torch.dtype = torch.bfloat16, device="cuda", quantize: Optional[str] = None):
    """`path`: a folder with config.json and model.safetensors, or a lit-llama checkpoint file."""
    path = Path(path)
    kw = {"quantize": quantize} if quantize else {}
    if path.is_dir():
        config = json.loads((path / "config.json").read_text())
        model = build_model(config, dtype, device, **kw)
        weights = path / "model.safetensors"
    else:
        from .model import llama_configs
        from .utils import llama_model_lookup

        with lazy_load(path) as sd:
            name = llama_model_lookup(sd)
        model = build_model({"architecture": "LLaMA", **llama_configs[name]}, dtype, device, **kw)
        weights = path
    with lazy_load(weights) as sd:
        model.load_state_dict(sd)
    return model
