"""Where a model's tensors come from: a folder with safetensors files, or a seeded random initialisation.

Both sources answer take(name, shape, kind) with a device tensor in the model's dtype; a model asks for each of its tensors
once, under the checkpoint's name.  shape_of(name) is the shape that the source holds, or None where it makes tensors of any
shape: for sizes that the configuration leaves to the tensors.  `kind` only matters to the random source:
  linear (std fan_in^-0.5) | embed (std 0.02, or `std`) | norm (around one) | norm_offset (around zero) | vector (std 0.1)
"""
from __future__ import annotations

import json
import mmap
import sys
from pathlib import Path

import torch

_TYPES = {"BF16": torch.bfloat16, "F32": torch.float32, "F16": torch.float16, "I32": torch.int32, "I64": torch.int64}


def read_safetensors(path) -> dict:
    """name -> CPU tensor of one safetensors file (an 8-byte little-endian length, that many bytes of JSON, the data)."""
    with open(path, "rb") as f:
        buf = mmap.mmap(f.fileno(), 0, access=mmap.ACCESS_COPY)
    n = int.from_bytes(buf[:8], "little")
    if n > len(buf) - 8:
        raise ValueError(f"{path}: the header is longer than the file")
    out = {}
    for name, entry in json.loads(buf[8:8 + n]).items():
        if name == "__metadata__":
            continue
        dtype = _TYPES.get(entry["dtype"])
        if dtype is None:
            raise ValueError(f"{path}: {name} has the unsupported type {entry['dtype']}")
        begin, end = entry["data_offsets"]
        shape = entry["shape"]
        count = 1
        for s in shape:
            count *= s
        if end - begin != count * torch.empty((), dtype=dtype).element_size() or end > len(buf) - 8 - n:
            raise ValueError(f"{path}: the offsets of {name} do not fit its shape or the file")
        t = torch.frombuffer(buf, dtype=torch.uint8, count=end - begin, offset=8 + n + begin) if count else torch.empty(0, dtype=torch.uint8)
        if (8 + n + begin) % 8:
            t = t.clone()
        out[name] = t.view(dtype).reshape(shape)
    return out


class CheckpointWeights:
    """Tensors of every *.safetensors file of a folder."""

    def __init__(self, folder, dtype=torch.bfloat16, device="cuda:0"):
        self.dtype, self.device = dtype, torch.device(device)
        files = sorted(Path(folder).glob("*.safetensors"))
        if not files:
            raise FileNotFoundError(f"{folder} holds no safetensors file")
        self._tensors = {}
        for f in files:
            self._tensors.update(read_safetensors(f))

    def take(self, name: str, shape, kind: str = "linear", std: float = None) -> torch.Tensor:
        t = self._tensors.pop(name, None)
        if t is None:
            raise KeyError(f"the checkpoint has no tensor {name}")
        if tuple(t.shape) != tuple(shape):
            raise ValueError(f"{name} has the shape {tuple(t.shape)}, the configuration asks for {tuple(shape)}")
        if t.is_floating_point():
            return t.to(device=self.device, dtype=self.dtype)
        return t.to(self.device)

    def shape_of(self, name: str):
        t = self._tensors.get(name)
        if t is None:
            raise KeyError(f"the checkpoint has no tensor {name}")
        return tuple(t.shape)

    def finish(self) -> None:
        if self._tensors:
            print(f"tensors of the checkpoint that the model does not use: {', '.join(sorted(self._tensors))}", file=sys.stderr)


class RandomWeights:
    """Seeded random tensors, drawn in the order in which the model asks for them."""

    def __init__(self, seed: int = 0, dtype=torch.bfloat16, device="cuda:0"):
        self.dtype, self.device = dtype, torch.device(device)
        self._g = torch.Generator(device=self.device).manual_seed(seed)

    def take(self, name: str, shape, kind: str = "linear", std: float = None) -> torch.Tensor:
        if std is None:
            std = {"linear": shape[-1] ** -0.5, "embed": 0.02, "norm": 0.05, "norm_offset": 0.05, "vector": 0.1}[kind]
        t = torch.randn(tuple(shape), generator=self._g, device=self.device, dtype=torch.float32) * std
        return ((1.0 + t) if kind == "norm" else t).to(torch.bfloat16).to(self.dtype)

    def shape_of(self, name: str):
        return None

    def finish(self) -> None:
        pass


class TensorWeights(CheckpointWeights):
    """A dict of tensors under the checkpoint's names."""

    def __init__(self, tensors: dict, dtype=torch.bfloat16, device="cuda:0"):
        self.dtype, self.device = dtype, torch.device(device)
        self._tensors = dict(tensors)
