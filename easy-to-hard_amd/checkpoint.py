"""Checkpoint folders: config.json plus model.safetensors.

A safetensors file is an 8-byte little-endian header length, that many bytes of JSON (name -> dtype, shape,
data_offsets) and the raw tensor data; it is memory-mapped and read tensor by tensor.
"""

import json
import mmap
import struct
from pathlib import Path

import torch

_DTYPES = {"BF16": torch.bfloat16, "F16": torch.float16, "F32": torch.float32, "F64": torch.float64, "I8": torch.int8, "U8": torch.uint8,
           "I16": torch.int16, "I32": torch.int32, "I64": torch.int64, "BOOL": torch.bool}


class SafetensorsFile:
    def __init__(self, path):
        self.path = Path(path)
        with open(self.path, "rb") as f:
            self._map = mmap.mmap(f.fileno(), 0, access=mmap.ACCESS_COPY)  # private pages: torch wants writable memory
        if len(self._map) < 8:
            raise ValueError(f"{path}: too short for a safetensors file")
        (n,) = struct.unpack("<Q", self._map[:8])
        if 8 + n > len(self._map):
            raise ValueError(f"{path}: header of {n} bytes exceeds the file")
        header = json.loads(self._map[8: 8 + n])
        header.pop("__metadata__", None)
        self._entries, self._base = header, 8 + n

    def keys(self):
        return self._entries.keys()

    def __contains__(self, name):
        return name in self._entries

    def get(self, name) -> torch.Tensor:
        """The tensor as a view of the mapped file."""
        if name not in self._entries:
            raise KeyError(f"{self.path}: no tensor named {name}")
        e = self._entries[name]
        dtype, shape, (lo, hi) = _DTYPES[e["dtype"]], tuple(e["shape"]), e["data_offsets"]
        count = 1
        for s in shape:
            count *= s
        size = count * torch.empty((), dtype=dtype).element_size()
        if hi - lo != size or self._base + hi > len(self._map):
            raise ValueError(f"{self.path}: {name} spans {hi - lo} bytes, {shape} of {e['dtype']} needs {size}")
        if count == 0:
            return torch.empty(shape, dtype=dtype)
        start = self._base + lo
        if start % torch.empty((), dtype=dtype).element_size():
            return torch.frombuffer(bytearray(self._map[start: start + size]), dtype=dtype).view(shape)
        return torch.frombuffer(self._map, dtype=dtype, count=count, offset=start).view(shape)


def read_config(folder) -> dict:
    with open(Path(folder) / "config.json") as f:
        return json.load(f)
