"""Weight files: a memory-mapped safetensors reader (8-byte little-endian header length, JSON header
``name -> {dtype, shape, data_offsets}``, raw data) that executes nothing from the file."""
from __future__ import annotations

import json
import mmap
import os
from typing import Dict, Iterator

import torch

_DTYPES = {"BF16": torch.bfloat16, "F32": torch.float32, "F16": torch.float16, "I32": torch.int32, "I64": torch.int64,
           "U8": torch.uint8, "F64": torch.float64}


class SafetensorsFile:
    """Read-only mapping of one file; tensors are copied out of the mapping when asked for."""

    def __init__(self, path: str):
        self.path = path
        with open(path, "rb") as f:
            self._map = mmap.mmap(f.fileno(), 0, access=mmap.ACCESS_READ)
        n = int.from_bytes(self._map[:8], "little")
        if n <= 0 or 8 + n > len(self._map):
            raise ValueError(f"{path}: not a safetensors file")
        header = json.loads(self._map[8:8 + n].decode("utf-8"))
        header.pop("__metadata__", None)
        self._base, self._entries = 8 + n, header

    def names(self) -> Iterator[str]:
        return iter(self._entries)

    def __contains__(self, name: str) -> bool:
        return name in self._entries

    def __getitem__(self, name: str) -> torch.Tensor:
        if name not in self._entries:
            raise KeyError(f"{self.path}: no tensor {name!r}")
        e = self._entries[name]
        lo, hi = e["data_offsets"]
        dtype, shape = _DTYPES[e["dtype"]], e["shape"]
        n = 1
        for s in shape:
            n *= s
        if hi - lo != n * torch.empty((), dtype=dtype).element_size() or self._base + hi > len(self._map):
            raise ValueError(f"{self.path}: {name} has {hi - lo} bytes for shape {shape}")
        return torch.frombuffer(bytearray(self._map[self._base + lo:self._base + hi]), dtype=dtype).view(shape) if n else \
            torch.empty(shape, dtype=dtype)


def load_tensors(model_dir: str) -> Dict[str, torch.Tensor]:
    """Every tensor of a model folder: ``model.safetensors``, or the shards ``model.safetensors.index.json`` lists."""
    index = os.path.join(model_dir, "model.safetensors.index.json")
    if os.path.exists(index):
        with open(index) as f:
            files = sorted(set(json.load(f)["weight_map"].values()))
    else:
        files = ["model.safetensors"]
    out: Dict[str, torch.Tensor] = {}
    for name in files:
        st = SafetensorsFile(os.path.join(model_dir, name))
        out.update((n, st[n]) for n in st.names())
    return out
