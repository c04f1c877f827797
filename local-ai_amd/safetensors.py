"""Safetensors reader: an 8-byte little-endian length, that many bytes of JSON (name -> dtype, shape, data_offsets), then
the data.  Tensors are read-only views of a memory map of the file."""
from __future__ import annotations

import json
import mmap
import struct
from typing import Dict, Tuple

import numpy as np

from . import Io
from .gguf import InvalidFormat

# bf16 has no numpy type: its raw bits
_NUMPY = {"F64": np.float64, "F32": np.float32, "F16": np.float16, "BF16": np.uint16, "I64": np.int64, "I32": np.int32,
          "I16": np.int16, "I8": np.int8, "U8": np.uint8, "BOOL": np.uint8}


class SafetensorsFile:
    def __init__(self, path: str):
        try:
            with open(path, "rb") as f:
                self._map = mmap.mmap(f.fileno(), 0, access=mmap.ACCESS_READ)
        except (OSError, ValueError) as e:
            raise Io(f"{path}: {e}") from e
        if len(self._map) < 8:
            raise InvalidFormat(f"{path}: no header")
        n = struct.unpack("<Q", self._map[:8])[0]
        if n > len(self._map) - 8:
            raise InvalidFormat(f"{path}: header of {n} bytes exceeds the file")
        try:
            header = json.loads(self._map[8:8 + n])
        except ValueError as e:
            raise InvalidFormat(f"{path}: header is not JSON") from e
        header.pop("__metadata__", None)
        self.path, self._data, self._entries = path, 8 + n, header

    def __contains__(self, name: str) -> bool:
        return name in self._entries

    def names(self):
        return list(self._entries)

    def shape(self, name: str) -> Tuple[int, ...]:
        return tuple(self._entry(name)["shape"])

    def _entry(self, name: str) -> Dict:
        if name not in self._entries:
            raise InvalidFormat(f"{self.path}: no tensor {name}")
        return self._entries[name]

    def raw(self, name: str) -> Tuple[str, np.ndarray]:
        """(dtype name, array): the stored values, bf16 as uint16 bits."""
        e = self._entry(name)
        if e["dtype"] not in _NUMPY:
            raise InvalidFormat(f"{self.path}: {name} has dtype {e['dtype']}")
        dt = np.dtype(_NUMPY[e["dtype"]])
        a, b = e["data_offsets"]
        count = int(np.prod(e["shape"], dtype=np.int64))
        if b - a != count * dt.itemsize or self._data + b > len(self._map):
            raise InvalidFormat(f"{self.path}: {name} has {b - a} bytes for shape {e['shape']}")
        return e["dtype"], np.frombuffer(self._map, dt, count, self._data + a).reshape(e["shape"])

    def bf16(self, name: str, shape=None) -> np.ndarray:
        """The tensor as bf16 bits; f32 and f16 values are rounded to nearest even."""
        dtype, a = self.raw(name)
        self._check_shape(name, a, shape)
        if dtype == "BF16":
            return a
        return round_to_bf16(a.astype(np.float32))

    def f32(self, name: str, shape=None) -> np.ndarray:
        dtype, a = self.raw(name)
        self._check_shape(name, a, shape)
        if dtype == "BF16":
            return (a.astype(np.uint32) << 16).view(np.float32)
        return a.astype(np.float32)

    def _check_shape(self, name, a, shape) -> None:
        if shape is not None and tuple(a.shape) != tuple(shape):
            raise InvalidFormat(f"{self.path}: {name} is {list(a.shape)}, the configuration says {list(shape)}")


def round_to_bf16(x: np.ndarray) -> np.ndarray:
    """f32 -> bf16 bits, nearest even (NaN stays NaN)."""
    u = np.ascontiguousarray(x, np.float32).view(np.uint32)
    r = ((u + 0x7FFF + ((u >> 16) & 1)) >> 16).astype(np.uint16)
    return np.where(np.isnan(x), np.uint16(0x7FC0), r)


def write(path: str, tensors: Dict[str, np.ndarray]) -> None:
    """Writes `tensors`; uint16 arrays are taken for bf16 bits."""
    names = {np.dtype(np.float32): "F32", np.dtype(np.uint16): "BF16", np.dtype(np.int32): "I32", np.dtype(np.float16): "F16"}
    header, off = {}, 0
    for n, a in tensors.items():
        header[n] = {"dtype": names[a.dtype], "shape": list(a.shape), "data_offsets": [off, off + a.nbytes]}
        off += a.nbytes
    text = json.dumps(header).encode()
    text += b" " * (-len(text) % 8)
    with open(path, "wb") as f:
        f.write(struct.pack("<Q", len(text)) + text)
        for a in tensors.values():
            f.write(np.ascontiguousarray(a).tobytes())
