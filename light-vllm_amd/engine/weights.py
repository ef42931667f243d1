"""Checkpoint files: a safetensors reader (8-byte little-endian header length, a JSON header of name -> dtype, shape,
data_offsets, then the data), memory-mapped so that only the tensors taken are read."""
import json
import mmap
import os
import struct
from typing import Dict

import torch

_DTYPES = {"BF16": torch.bfloat16, "F16": torch.float16, "F32": torch.float32, "F64": torch.float64,
           "I64": torch.int64, "I32": torch.int32, "I16": torch.int16, "I8": torch.int8, "U8": torch.uint8,
           "BOOL": torch.bool}


class SafetensorsFile:

    def __init__(self, path: str):
        self.path = path
        size = os.path.getsize(path)
        self._file = open(path, "rb")
        self._map = mmap.mmap(self._file.fileno(), 0, access=mmap.ACCESS_COPY)
        n = struct.unpack("<Q", self._map[:8])[0]
        if 8 + n > size:
            raise ValueError(f"{path}: the header does not fit the file")
        header = json.loads(self._map[8:8 + n])
        header.pop("__metadata__", None)
        self._base, self._header = 8 + n, header
        for name, h in header.items():
            a, b = h["data_offsets"]
            numel = 1
            for d in h["shape"]:
                numel *= d
            if h["dtype"] not in _DTYPES:
                raise ValueError(f"{path}: tensor {name} has dtype {h['dtype']}")
            if not 0 <= a <= b <= size - self._base or b - a != numel * torch.empty((), dtype=_DTYPES[h["dtype"]]).element_size():
                raise ValueError(f"{path}: tensor {name} does not fit the file")

    def keys(self):
        return self._header.keys()

    def __contains__(self, name: str) -> bool:
        return name in self._header

    def __getitem__(self, name: str) -> torch.Tensor:
        """A CPU tensor of its own memory."""
        h = self._header[name]
        a, b = h["data_offsets"]
        if a == b:
            return torch.empty(h["shape"], dtype=_DTYPES[h["dtype"]])
        raw = bytearray(self._map[self._base + a:self._base + b])
        return torch.frombuffer(raw, dtype=_DTYPES[h["dtype"]]).reshape(h["shape"])


def load_checkpoint(model_dir: str) -> SafetensorsFile:
    return SafetensorsFile(os.path.join(model_dir, "model.safetensors"))
