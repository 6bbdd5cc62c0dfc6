"""Reader of safetensors files: an 8-byte little-endian header length, a JSON
header (name -> dtype, shape, data_offsets), then the raw tensor data.  The
file is mapped, so a tensor's pages are read when it is asked for."""

from __future__ import annotations

import json
import mmap
import os
import struct
from typing import Dict, List, Tuple

import torch

_DTYPES = {"BF16": torch.bfloat16, "F16": torch.float16, "F32": torch.float32,
           "F64": torch.float64, "I32": torch.int32, "I64": torch.int64,
           "I16": torch.int16, "I8": torch.int8, "U8": torch.uint8}


class Checkpoint:
    def __init__(self, path: str):
        self.path = path
        with open(path, "rb") as f:
            head = f.read(8)
            if len(head) < 8:
                raise ValueError(f"{path}: no safetensors header")
            (n,) = struct.unpack("<Q", head)
            if n > os.path.getsize(path) - 8:
                raise ValueError(f"{path}: header longer than the file")
            self._entries: Dict[str, dict] = json.loads(f.read(n))
            self._entries.pop("__metadata__", None)
            self._map = mmap.mmap(f.fileno(), 0, access=mmap.ACCESS_READ)
        self._data = 8 + n

    def names(self) -> List[str]:
        return list(self._entries)

    def shape(self, name: str) -> Tuple[int, ...]:
        return tuple(self._entry(name)["shape"])

    def _entry(self, name: str) -> dict:
        if name not in self._entries:
            raise KeyError(f"{self.path}: no tensor {name!r}")
        return self._entries[name]

    def get(self, name: str) -> torch.Tensor:
        """A copy of the tensor, on the CPU, in the file's dtype."""
        e = self._entry(name)
        dtype = _DTYPES.get(e["dtype"])
        if dtype is None:
            raise ValueError(f"{name}: unsupported dtype {e['dtype']}")
        lo, hi = e["data_offsets"]
        raw = bytearray(self._map[self._data + lo:self._data + hi])
        count = 1
        for s in e["shape"]:
            count *= s
        if len(raw) != count * torch.empty((), dtype=dtype).element_size():
            raise ValueError(f"{name}: data does not fit its shape")
        if not raw:
            return torch.empty(e["shape"], dtype=dtype)
        return torch.frombuffer(raw, dtype=dtype).view(e["shape"])


def open_checkpoint(folder: str) -> Checkpoint:
    return Checkpoint(os.path.join(folder, "model.safetensors"))
