"""Checkpoint reading: a memory-mapped safetensors file.

The format is an 8-byte little-endian header length, that many bytes of
JSON (name -> dtype, shape, data_offsets) and the tensor data."""

from __future__ import annotations

import json
import mmap
import os
from typing import Dict, Iterator, Tuple

import torch

_DTYPES = {
    "BF16": torch.bfloat16, "F16": torch.float16, "F32": torch.float32,
    "F64": torch.float64, "I64": torch.int64, "I32": torch.int32,
    "I16": torch.int16, "I8": torch.int8, "U8": torch.uint8, "BOOL": torch.bool,
}


class SafetensorsFile:
    """Tensors of one file by name; each is copied out of the map when it
    is asked for, so a large file is never held twice in host memory."""

    def __init__(self, path: str):
        with open(path, "rb") as f:
            self._map = mmap.mmap(f.fileno(), 0, access=mmap.ACCESS_READ)
        n = int.from_bytes(self._map[:8], "little")
        header = json.loads(self._map[8 : 8 + n])
        header.pop("__metadata__", None)
        self._base = 8 + n
        self._entries: Dict[str, dict] = header

    def names(self) -> Iterator[str]:
        return iter(self._entries)

    def shape(self, name: str) -> Tuple[int, ...]:
        return tuple(self._entries[name]["shape"])

    def tensor(self, name: str) -> torch.Tensor:
        e = self._entries[name]
        lo, hi = e["data_offsets"]
        data = bytearray(self._map[self._base + lo : self._base + hi])
        dtype = _DTYPES[e["dtype"]]
        if not data:
            return torch.empty(e["shape"], dtype=dtype)
        return torch.frombuffer(data, dtype=dtype).reshape(e["shape"])


def open_checkpoint(folder: str) -> SafetensorsFile:
    return SafetensorsFile(os.path.join(folder, "model.safetensors"))
