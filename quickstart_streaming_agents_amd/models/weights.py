"""Checkpoint reading: the safetensors container, without executing anything.

A file is an 8-byte little-endian header length, that many bytes of JSON
({name: {dtype, shape, data_offsets}}), then the tensor data.  Tensors are
copied from a read-only memory map one at a time, so loading needs host
memory for one tensor, not for the file.
"""

from __future__ import annotations

import json
import mmap
import os
import struct

import torch

_DTYPES = {"BF16": torch.bfloat16, "F16": torch.float16,
           "F32": torch.float32, "F64": torch.float64,
           "I64": torch.int64, "I32": torch.int32, "I16": torch.int16,
           "I8": torch.int8, "U8": torch.uint8, "BOOL": torch.bool}


class SafetensorsFile:
    def __init__(self, path: str):
        self._fh = open(path, "rb")
        size = os.fstat(self._fh.fileno()).st_size
        if size < 8:
            raise ValueError(f"{path}: not a safetensors file")
        (n,) = struct.unpack("<Q", self._fh.read(8))
        if n > size - 8:
            raise ValueError(f"{path}: header exceeds the file")
        head = json.loads(self._fh.read(n).decode("utf-8"))
        head.pop("__metadata__", None)
        self._head = head
        self._base = 8 + n
        self._size = size
        self._map = mmap.mmap(self._fh.fileno(), 0, access=mmap.ACCESS_READ)

    def keys(self) -> list[str]:
        return list(self._head)

    def __contains__(self, name: str) -> bool:
        return name in self._head

    def shape(self, name: str) -> tuple[int, ...]:
        return tuple(self._head[name]["shape"])

    def get(self, name: str) -> torch.Tensor | None:
        """A host copy of one tensor in its stored type (None: not there)."""
        info = self._head.get(name)
        if info is None:
            return None
        dtype = _DTYPES[info["dtype"]]
        a, b = info["data_offsets"]
        count = 1
        for s in info["shape"]:
            count *= s
        itemsize = torch.empty(0, dtype=dtype).element_size()
        if b - a != count * itemsize or self._base + b > self._size:
            raise ValueError(f"{name}: data offsets do not fit the shape")
        if count == 0:
            return torch.empty(info["shape"], dtype=dtype)
        raw = bytearray(self._map[self._base + a:self._base + b])
        return torch.frombuffer(raw, dtype=dtype).reshape(info["shape"])

    def close(self) -> None:
        self._map.close()
        self._fh.close()


def write_safetensors(path: str, tensors: dict[str, torch.Tensor]) -> None:
    """Write host tensors in the same container."""
    names = {v: k for k, v in _DTYPES.items()}
    head, at = {}, 0
    for name, t in tensors.items():
        n = t.numel() * t.element_size()
        head[name] = {"dtype": names[t.dtype], "shape": list(t.shape),
                      "data_offsets": [at, at + n]}
        at += n
    blob = json.dumps(head).encode("utf-8")
    blob += b" " * (-len(blob) % 8)
    with open(path, "wb") as fh:
        fh.write(struct.pack("<Q", len(blob)))
        fh.write(blob)
        for t in tensors.values():
            fh.write(t.detach().cpu().contiguous().view(torch.uint8)
                     .reshape(-1).numpy().tobytes())
