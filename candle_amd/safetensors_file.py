"""Reader of safetensors files: an 8-byte little-endian length, that many bytes of JSON ({name: {dtype, shape, data_offsets}}), then the
data.  The file is memory-mapped; tensors are views of it until they are copied to the device."""
from __future__ import annotations

import json
import mmap
import os
import struct
from typing import Dict, List, Tuple

import torch

_DTYPES = {"BF16": torch.bfloat16, "F16": torch.float16, "F32": torch.float32, "F64": torch.float64, "I64": torch.int64, "I32": torch.int32,
           "I16": torch.int16, "I8": torch.int8, "U8": torch.uint8, "BOOL": torch.bool}


class SafetensorsError(ValueError):
    """The file is not a safetensors file, or lacks a tensor."""


class SafetensorsFile:
    def __init__(self, path: str):
        self.path = path
        size = os.path.getsize(path)
        with open(path, "rb") as f:
            head = f.read(8)
            if len(head) != 8:
                raise SafetensorsError(f"{path}: too short")
            n = struct.unpack("<Q", head)[0]
            if n > size - 8:
                raise SafetensorsError(f"{path}: header of {n} bytes in a file of {size}")
            try:
                header = json.loads(f.read(n))
            except ValueError as e:
                raise SafetensorsError(f"{path}: header is not JSON ({e})") from None
            self._map = mmap.mmap(f.fileno(), 0, access=mmap.ACCESS_COPY)
        self._data = 8 + n
        self._infos: Dict[str, Tuple[torch.dtype, List[int], int, int]] = {}
        for name, info in header.items():
            if name == "__metadata__":
                continue
            dtype = _DTYPES.get(info["dtype"])
            if dtype is None:
                raise SafetensorsError(f"{path}: {name} has the unknown dtype {info['dtype']}")
            lo, hi = info["data_offsets"]
            count = 1
            for d in info["shape"]:
                count *= d
            if not 0 <= lo <= hi <= size - self._data or hi - lo != count * dtype.itemsize:
                raise SafetensorsError(f"{path}: {name} has inconsistent offsets")
            self._infos[name] = (dtype, list(info["shape"]), lo, hi)

    def names(self) -> List[str]:
        return list(self._infos)

    def __contains__(self, name: str) -> bool:
        return name in self._infos

    def tensor(self, name: str) -> torch.Tensor:
        """The tensor on the host, as stored."""
        if name not in self._infos:
            raise SafetensorsError(f"{self.path}: no tensor {name}")
        dtype, shape, lo, hi = self._infos[name]
        if lo == hi:
            return torch.empty(shape, dtype=dtype)
        return torch.frombuffer(self._map, dtype=torch.uint8, count=hi - lo, offset=self._data + lo).clone().view(dtype).reshape(shape)
