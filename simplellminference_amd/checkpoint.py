"""Reading a model folder: ``config.json`` and ``model.safetensors`` (an 8-byte little-endian header length, the JSON
header ``name -> {dtype, shape, data_offsets}``, then the tensor data), memory-mapped. Tensors come out as fp32 arrays
(the form every ``set_weight`` / ``set_tensor`` takes); bfloat16 and fp16 widen exactly."""
from __future__ import annotations

import json
import os
import struct

import numpy as np

_PLAIN = {"F32": np.float32, "F16": np.float16, "I32": np.int32, "I64": np.int64, "U8": np.uint8, "I8": np.int8}


def read_config(model_dir: str) -> dict:
    with open(os.path.join(model_dir, "config.json"), encoding="utf-8") as f:
        return json.load(f)


class SafeTensors:
    """The tensors of one safetensors file by name."""

    def __init__(self, path: str):
        size = os.path.getsize(path)
        with open(path, "rb") as f:
            head = f.read(8)
            n = struct.unpack("<Q", head)[0] if len(head) == 8 else size
            if 8 + n > size:
                raise ValueError(f"{path}: not a safetensors file")
            self._header = json.loads(f.read(n))
        self._header.pop("__metadata__", None)
        self._data = np.memmap(path, np.uint8, "r", offset=8 + n) if size > 8 + n else np.empty(0, np.uint8)
        self.path = path

    def names(self) -> list[str]:
        return list(self._header)

    def shape(self, name: str) -> tuple[int, ...]:
        return tuple(self._header[name]["shape"])

    def get(self, name: str) -> np.ndarray:
        h = self._header[name]
        lo, hi = h["data_offsets"]
        shape = tuple(h["shape"])
        raw = self._data[lo:hi]
        itemsize = 2 if h["dtype"] == "BF16" else np.dtype(_PLAIN[h["dtype"]]).itemsize if h["dtype"] in _PLAIN else 0
        if not itemsize:
            raise ValueError(f"{self.path}: tensor {name} has unsupported dtype {h['dtype']}")
        if hi > self._data.size or hi - lo != itemsize * int(np.prod(shape, dtype=np.int64)):
            raise ValueError(f"{self.path}: tensor {name} does not fit its shape")
        if h["dtype"] == "BF16":
            return (np.frombuffer(raw, "<u2").astype(np.uint32) << 16).view(np.float32).reshape(shape)
        return np.frombuffer(raw, _PLAIN[h["dtype"]]).reshape(shape).astype(np.float32)
