"""Checkpoint files -- state dicts out of safetensors or torch files, nothing in them executed -- and the reshaping of their
tensors for the kernels."""
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


class Checkpoint:
    """A state dict's tensors, with their shapes checked against what the configuration says."""

    def __init__(self, state_dict: dict, dtype: torch.dtype, device):
        self.tensors, self.dtype, self.device = state_dict, dtype, device

    def raw(self, name, *shape):
        if name not in self.tensors:
            raise KeyError(f"the checkpoint has no tensor {name}")
        t = self.tensors[name].detach()
        if tuple(t.shape) != shape:
            raise ValueError(f"{name} is {tuple(t.shape)}, the configuration says {shape}")
        return t

    def matrix(self, t):
        """A tensor in the computing type on the device."""
        return t.to(device=self.device, dtype=self.dtype).contiguous()

    def vector(self, name, *shape):
        """A named parameter in fp32 on the device."""
        return self.raw(name, *shape).to(device=self.device, dtype=torch.float32).contiguous()


def pad_heads(t, heads, size, to):
    """(heads * size, ...) -> (heads * to, ...) with zero rows behind every head."""
    if size == to:
        return t
    t = t.view(heads, size, *t.shape[1:])
    return torch.cat((t, t.new_zeros(heads, to - size, *t.shape[2:])), 1).flatten(0, 1)


def stack_rows(parts):
    """Rows of several matrices (or entries of vectors), each part starting at a multiple of 8 rows (zero rows between),
    so that every part of a product's row is 16-byte aligned.  Returns the stack and the parts' first rows."""
    out, starts, at = [], [], 0
    for t in parts:
        starts.append(at)
        pad = -t.shape[0] % 8
        out += [t, t.new_zeros(pad, *t.shape[1:])] if pad else [t]
        at += t.shape[0] + pad
    return torch.cat(out).contiguous(), starts


def pad_to(t, dim, multiple):
    """Zeros behind dimension `dim` up to a multiple."""
    pad = -t.shape[dim] % multiple
    if not pad:
        return t
    shape = list(t.shape)
    shape[dim] = pad
    return torch.cat((t, t.new_zeros(shape)), dim)


def pair_halves(t, heads, size, dims):
    """Rows of a query or key projection whose rotation pairs entry i of a head with entry i + dims / 2, reordered so that the
    pairs are adjacent (which changes no score when queries and keys are reordered alike)."""
    order = torch.arange(size)
    order[:dims] = torch.stack((torch.arange(dims // 2), torch.arange(dims // 2, dims)), 1).flatten()
    return t.view(heads, size, *t.shape[1:])[:, order].flatten(0, 1)
