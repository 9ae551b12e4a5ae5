"""Which model class a folder of weights holds, and how to load it.

A folder with a config.json names its design there ("architecture"); one without is a nanochat checkpoint (model_*.pt, meta_*.json)."""
import importlib
import os

import torch

from .checkpoint import read_config

# architecture -> (module, class); a class has load(model_dir, dtype, device)
ARCHITECTURES = {"Palilix": ("palilix", "Palilix"), "Zodirax": ("zodirax", "Zodirax")}


def model_class(architecture):
    if architecture not in ARCHITECTURES:
        raise ValueError(f"unknown architecture {architecture!r}; known: {', '.join(sorted(ARCHITECTURES))}")
    module, name = ARCHITECTURES[architecture]
    return getattr(importlib.import_module(f".{module}", __package__), name)


def load_model(model_dir, dtype=torch.bfloat16, device="cuda", step=None):
    """(model, info) of any folder this package can serve."""
    if os.path.exists(os.path.join(model_dir, "config.json")):
        cfg = read_config(model_dir)
        return model_class(cfg.get("architecture")).load(model_dir, dtype=dtype, device=device), {"model_config": cfg, "step": None}
    if dtype != torch.bfloat16:
        raise ValueError("a nanochat checkpoint runs with FP8 linears and bfloat16 activations only")
    from .checkpoint import build_model
    return build_model(model_dir, step, device)
