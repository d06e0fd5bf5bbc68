"""Reader of safetensors files: tensors as read-only numpy views of the mapped file.

Format: an 8-byte little-endian length, that many bytes of JSON (name -> dtype, shape,
data_offsets; offsets count from the end of the JSON), then the data.  Nothing in the file is
executed; sizes and offsets are checked against the file before a view is made.  numpy has no
bfloat16: such tensors come as uint16 bit patterns.
"""
from __future__ import annotations

import json
import mmap
from pathlib import Path

import numpy as np

_DTYPES = {"BF16": np.uint16, "F16": np.float16, "F32": np.float32, "F64": np.float64, "I8": np.int8, "U8": np.uint8,
           "I16": np.int16, "I32": np.int32, "I64": np.int64}


class SafeTensorsError(ValueError):
    """The file is not a valid safetensors file, or lacks what is asked of it."""


class SafeTensors:
    def __init__(self, path):
        self.path = Path(path)
        with open(self.path, "rb") as f:
            size = f.seek(0, 2)
            if size < 8:
                raise SafeTensorsError(f"{self.path}: too short")
            self._map = mmap.mmap(f.fileno(), 0, access=mmap.ACCESS_READ)
        n = int.from_bytes(self._map[:8], "little")
        if n > size - 8:
            raise SafeTensorsError(f"{self.path}: header of {n} bytes in a file of {size}")
        try:
            header = json.loads(self._map[8:8 + n])
        except ValueError as e:
            raise SafeTensorsError(f"{self.path}: header is not JSON ({e})") from None
        if not isinstance(header, dict):
            raise SafeTensorsError(f"{self.path}: header is not an object")
        self._entries = {}
        room = size - 8 - n
        for name, t in header.items():
            if name == "__metadata__":
                continue
            try:
                dtype, shape, (lo, hi) = np.dtype(_DTYPES[t["dtype"]]), tuple(int(d) for d in t["shape"]), t["data_offsets"]
            except (KeyError, TypeError, ValueError):
                raise SafeTensorsError(f"{self.path}: tensor {name!r} has an unsupported description") from None
            count = 1
            for d in shape:
                count *= d
            if min(shape, default=0) < 0 or not (0 <= lo <= hi <= room) or hi - lo != count * dtype.itemsize:
                raise SafeTensorsError(f"{self.path}: tensor {name!r} does not fit its data")
            self._entries[name] = (t["dtype"], dtype, shape, 8 + n + lo, count)

    def __contains__(self, name: str) -> bool:
        return name in self._entries

    def names(self) -> list[str]:
        return list(self._entries)

    def raw(self, name: str, dtype: str | None = None, shape=None) -> np.ndarray:
        """View of a tensor, checked against the dtype and shape the caller expects."""
        if name not in self._entries:
            raise SafeTensorsError(f"{self.path}: tensor {name!r} is missing")
        kind, np_dtype, have, at, count = self._entries[name]
        if dtype is not None and kind != dtype:
            raise SafeTensorsError(f"{self.path}: tensor {name!r} is {kind}, expected {dtype}")
        if shape is not None and tuple(shape) != have:
            raise SafeTensorsError(f"{self.path}: tensor {name!r} has shape {list(have)}, expected {list(shape)}")
        return np.frombuffer(self._map, np_dtype, count, at).reshape(have)

    def bf16(self, name: str, shape) -> np.ndarray:
        """A bfloat16 tensor's bit patterns."""
        return self.raw(name, "BF16", shape)


def write(path, tensors: dict[str, np.ndarray]) -> None:
    """Write arrays as a safetensors file (uint16 arrays as bfloat16)."""
    kinds = {np.dtype(v): k for k, v in _DTYPES.items()}
    header, at = {}, 0
    for name, t in tensors.items():
        header[name] = {"dtype": kinds[t.dtype], "shape": list(t.shape), "data_offsets": [at, at + t.nbytes]}
        at += t.nbytes
    text = json.dumps(header).encode()
    text += b" " * (-len(text) % 8)
    with open(path, "wb") as f:
        f.write(len(text).to_bytes(8, "little"))
        f.write(text)
        for t in tensors.values():
            f.write(np.ascontiguousarray(t).tobytes())
