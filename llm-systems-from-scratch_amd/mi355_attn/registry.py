"""Model registry: which class serves a model folder."""
from __future__ import annotations

import json
import os

from .model import CachedLM, CachedTransformerLM
from .weights import load_state_dict
from .zomipel import ZomipelLM
from .zuzelorn import ZuzelornLM

# config.json's "architecture" -> class; a configuration without the key is the reference decoder's
# (llm-core/llm_core/model.py:238-256 stores only the constructor arguments)
ARCHITECTURES: dict[str, type[CachedLM]] = {"TransformerLM": CachedTransformerLM, "Zuzelorn": ZuzelornLM,
                                          "Zomipel": ZomipelLM}
CHECKPOINT_NAMES = ("model.safetensors", "model.pt", "checkpoint.pt")


class UnsupportedDtype(ValueError):
    """The model's class does not compute in the requested type."""


def model_class(config: dict) -> type[CachedLM]:
    name = config.get("architecture", "TransformerLM")
    if name not in ARCHITECTURES:
        raise ValueError(f"unknown architecture {name!r} (known: {', '.join(sorted(ARCHITECTURES))})")
    return ARCHITECTURES[name]


def load_model(model_dir: str, *, dtype: str = "bfloat16", **kwargs) -> CachedLM:
    """The model of a folder with config.json and a checkpoint (one of CHECKPOINT_NAMES), ready to serve."""
    with open(os.path.join(model_dir, "config.json")) as f:
        config = json.load(f)
    cls = model_class(config)
    if dtype not in cls.DTYPES:
        raise UnsupportedDtype(f"{cls.__name__} computes in {', '.join(cls.DTYPES)}, not in {dtype}")
    if len(cls.DTYPES) > 1:
        kwargs["dtype"] = dtype
    for name in CHECKPOINT_NAMES:
        path = os.path.join(model_dir, name)
        if os.path.exists(path):
            return cls(config, load_state_dict(path), **kwargs)
    raise FileNotFoundError(f"{model_dir} holds none of {', '.join(CHECKPOINT_NAMES)}")
