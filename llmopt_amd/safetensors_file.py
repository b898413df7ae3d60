"""Safetensors weight files: an 8-byte little-endian header length, that many bytes of JSON
(name -> dtype, shape, data_offsets), then the data.  Read without copies (memory-mapped), with
every range checked against the file before a tensor is handed out.
"""
from __future__ import annotations

import json
import os
import struct
from typing import Mapping, Sequence

import numpy as np

# bfloat16 has no numpy type: its tensors are handed out as their 16-bit patterns
_NUMPY = {"BF16": np.uint16, "F16": np.float16, "F32": np.float32, "I32": np.int32, "I64": np.int64, "U8": np.uint8}


class SafetensorsError(ValueError):
    """The file does not decode."""


class SafetensorsFile:
    def __init__(self, path: str):
        self.path = path
        size = os.path.getsize(path)
        with open(path, "rb") as handle:
            prefix = handle.read(8)
            if len(prefix) < 8:
                raise SafetensorsError(f"{path} is too short for a safetensors file")
            length = struct.unpack("<Q", prefix)[0]
            if length > size - 8:
                raise SafetensorsError(f"{path}: the header extends beyond the file")
            header = json.loads(handle.read(length))
        self._start = 8 + length
        self._data = np.memmap(path, dtype=np.uint8, mode="r") if size > self._start else np.zeros(0, np.uint8)
        self._entries = {}
        for name, entry in header.items():
            if name == "__metadata__":
                continue
            dtype, shape, (begin, end) = entry["dtype"], tuple(entry["shape"]), entry["data_offsets"]
            if dtype not in _NUMPY:
                raise SafetensorsError(f"tensor {name} has unsupported dtype {dtype}")
            count = int(np.prod(shape, dtype=np.int64))
            if not 0 <= begin <= end <= size - self._start or end - begin != count * np.dtype(_NUMPY[dtype]).itemsize:
                raise SafetensorsError(f"tensor {name}: data range disagrees with its dtype and shape")
            self._entries[name] = (dtype, shape, begin, end)

    def names(self) -> Sequence[str]:
        return list(self._entries)

    def __contains__(self, name: str) -> bool:
        return name in self._entries

    def dtype(self, name: str) -> str:
        return self._entries[name][0]

    def numpy(self, name: str) -> np.ndarray:
        if name not in self._entries:
            raise SafetensorsError(f"{self.path} has no tensor {name}")
        dtype, shape, begin, end = self._entries[name]
        return self._data[self._start + begin:self._start + end].view(_NUMPY[dtype]).reshape(shape)

    def bfloat16(self, name: str, shape: Sequence[int]) -> np.ndarray:
        """The 16-bit patterns of a bfloat16 tensor, after checking its shape."""
        array = self.numpy(name)
        if self.dtype(name) != "BF16":
            raise SafetensorsError(f"tensor {name} is {self.dtype(name)}, expected BF16")
        if tuple(array.shape) != tuple(shape):
            raise SafetensorsError(f"tensor {name} has shape {list(array.shape)}, expected {list(shape)}")
        return array


def write_safetensors(path: str, tensors: Mapping[str, np.ndarray]) -> None:
    """Writes `tensors`; uint16 arrays are stored as the bfloat16 patterns they hold."""
    names = {np.dtype(v): k for k, v in _NUMPY.items()}
    header, offset, arrays = {}, 0, []
    for name, tensor in tensors.items():
        array = np.asarray(tensor, order="C")  # (keeps rank 0, which ascontiguousarray does not)
        header[name] = {"dtype": names[array.dtype], "shape": list(array.shape),
                        "data_offsets": [offset, offset + array.nbytes]}
        offset += array.nbytes
        arrays.append(array)
    encoded = json.dumps(header).encode()
    encoded += b" " * (-len(encoded) % 8)
    with open(path, "wb") as handle:
        handle.write(struct.pack("<Q", len(encoded)) + encoded)
        for array in arrays:
            handle.write(array.tobytes())


def to_bfloat16(values) -> np.ndarray:
    """float32 values rounded to nearest even, as 16-bit patterns."""
    bits = np.asarray(values, dtype=np.float32).view(np.uint32)
    return ((bits + 0x7FFF + ((bits >> 16) & 1)) >> 16).astype(np.uint16)


def from_bfloat16(patterns) -> np.ndarray:
    return (np.asarray(patterns, dtype=np.uint16).astype(np.uint32) << 16).view(np.float32)
