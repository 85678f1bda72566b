"""Checkpoint files: state dicts out of safetensors or torch files, nothing in them executed."""
from __future__ import annotations

import torch


def load_state_dict(path: str) -> dict:
    """A .safetensors file, or a torch file that is a state_dict or {"model": state_dict}
    (llm-core/llm_core/model.py:245-251), on the CPU."""
    if path.endswith(".safetensors"):
        from safetensors.torch import load_file
        return load_file(path)
    sd = torch.load(path, map_location="cpu", weights_only=True)
    return sd["model"] if "model" in sd else sd
