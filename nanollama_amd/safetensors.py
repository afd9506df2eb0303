"""Reading and writing safetensors files: an 8-byte little-endian length, that many bytes of JSON {name: {dtype, shape,
data_offsets}}, then the data.  Nothing in such a file is executed; offsets and sizes are checked before use."""
from __future__ import annotations

import json
import mmap
import struct
from typing import Dict, Iterator, Tuple

import numpy as np

_ITEM = {"F64": 8, "I64": 8, "U64": 8, "F32": 4, "I32": 4, "U32": 4, "BF16": 2, "F16": 2, "I16": 2, "U16": 2, "I8": 1, "U8": 1, "BOOL": 1}
_RAW = {8: np.uint64, 4: np.uint32, 2: np.uint16, 1: np.uint8}


class SafetensorsFile:
    """names() and get(name) -> (dtype tag, array): float32 / int32 as such, other types as raw unsigned words of their size."""

    def __init__(self, path: str):
        with open(path, "rb") as f:
            self._map = mmap.mmap(f.fileno(), 0, access=mmap.ACCESS_READ)
        size = len(self._map)
        if size < 8:
            raise ValueError(f"{path}: not a safetensors file")
        n = struct.unpack("<Q", self._map[:8])[0]
        if n > size - 8:
            raise ValueError(f"{path}: header of {n} bytes in a file of {size}")
        head = json.loads(self._map[8:8 + n].decode("utf-8"))
        head.pop("__metadata__", None)
        self._base = 8 + n
        self._info: Dict[str, dict] = head
        for name, t in head.items():
            a, b = t["data_offsets"]
            count = int(np.prod(t["shape"], dtype=np.int64)) if t["shape"] else 1
            if t["dtype"] not in _ITEM or not 0 <= a <= b <= size - self._base or b - a != count * _ITEM[t["dtype"]]:
                raise ValueError(f"{path}: tensor {name} has a bad type or bad offsets")

    def names(self) -> Iterator[str]:
        return iter(self._info)

    def __contains__(self, name: str) -> bool:
        return name in self._info

    def shape(self, name: str) -> Tuple[int, ...]:
        return tuple(self._info[name]["shape"])

    def nbytes(self, name: str) -> int:
        a, b = self._info[name]["data_offsets"]
        return b - a

    def get(self, name: str):
        t = self._info[name]
        a, b = t["data_offsets"]
        dt = {"F32": np.float32, "I32": np.int32}.get(t["dtype"], _RAW[_ITEM[t["dtype"]]])
        return t["dtype"], np.frombuffer(self._map, dtype=dt, count=(b - a) // np.dtype(dt).itemsize, offset=self._base + a).reshape(t["shape"])


def to_bf16(x: np.ndarray) -> np.ndarray:
    """float32 -> bfloat16 bits, round to nearest even."""
    u = np.ascontiguousarray(x, dtype=np.float32).view(np.uint32)
    return ((u + 0x7FFF + ((u >> 16) & 1)) >> 16).astype(np.uint16)


def from_bf16(x: np.ndarray) -> np.ndarray:
    return (np.ascontiguousarray(x).astype(np.uint32) << 16).view(np.float32)


def save(path: str, tensors: Dict[str, np.ndarray]) -> None:
    """tensors: uint16 arrays are stored as BF16, float32 as F32, int32 as I32."""
    tag = {np.dtype(np.uint16): "BF16", np.dtype(np.float32): "F32", np.dtype(np.int32): "I32"}
    head, at = {}, 0
    for name, x in tensors.items():
        head[name] = {"dtype": tag[x.dtype], "shape": list(x.shape), "data_offsets": [at, at + x.nbytes]}
        at += x.nbytes
    raw = json.dumps(head).encode()
    raw += b" " * (-len(raw) % 8)
    with open(path, "wb") as f:
        f.write(struct.pack("<Q", len(raw)) + raw)
        for x in tensors.values():
            f.write(np.ascontiguousarray(x).tobytes())
