"""safetensors reader / writer: an 8-byte little-endian header length, a JSON header
(name -> dtype, shape, data_offsets), then the data. Tensors are zero-copy views of the mapped file."""
from __future__ import annotations

import json
import mmap
import os
import struct
import warnings
from typing import Dict

import torch

DTYPES = {"BF16": torch.bfloat16, "F16": torch.float16, "F32": torch.float32, "F64": torch.float64,
          "I32": torch.int32, "I64": torch.int64, "I16": torch.int16, "I8": torch.int8, "U8": torch.uint8,
          "BOOL": torch.bool}
_NAMES = {v: k for k, v in DTYPES.items()}


class SafetensorsReader:
    def __init__(self, path: str):
        self.path = path
        size = os.path.getsize(path)
        with open(path, "rb") as f:
            if size < 8:
                raise ValueError(f"{path}: not a safetensors file")
            n = struct.unpack("<Q", f.read(8))[0]
            if n > size - 8 or n > (1 << 28):
                raise ValueError(f"{path}: bad safetensors header length {n}")
            head = json.loads(f.read(n).decode("utf-8"))
            self._map = mmap.mmap(f.fileno(), 0, access=mmap.ACCESS_READ)
        self.metadata = head.pop("__metadata__", {})
        self._base = 8 + n
        self._dir: Dict[str, tuple] = {}
        for name, d in head.items():
            if d["dtype"] not in DTYPES:
                raise ValueError(f"{path}: {name}: dtype {d['dtype']} not supported")
            dt, shape = DTYPES[d["dtype"]], tuple(int(v) for v in d["shape"])
            lo, hi = (int(v) for v in d["data_offsets"])
            numel = 1
            for v in shape:
                numel *= v
            if lo < 0 or hi - lo != numel * dt.itemsize or self._base + hi > size:
                raise ValueError(f"{path}: {name}: data_offsets do not fit its shape or the file")
            self._dir[name] = (dt, shape, lo, numel)

    def __contains__(self, name: str) -> bool:
        return name in self._dir

    def keys(self):
        return self._dir.keys()

    def shape(self, name: str) -> tuple:
        return self._dir[name][1]

    def tensor(self, name: str) -> torch.Tensor:
        """A read-only view of the file (copy or move it before writing)."""
        dt, shape, lo, numel = self._dir[name]
        if numel == 0:
            return torch.empty(shape, dtype=dt)
        with warnings.catch_warnings():
            warnings.simplefilter("ignore", UserWarning)     # the mapping is read-only
            return torch.frombuffer(self._map, dtype=dt, count=numel, offset=self._base + lo).view(shape)


def write_safetensors(path: str, tensors: Dict[str, torch.Tensor]):
    head, off = {}, 0
    for k, t in tensors.items():
        n = t.numel() * t.element_size()
        head[k] = {"dtype": _NAMES[t.dtype], "shape": list(t.shape), "data_offsets": [off, off + n]}
        off += n
    h = json.dumps(head).encode()
    h += b" " * (-len(h) % 8)
    with open(path, "wb") as f:
        f.write(struct.pack("<Q", len(h)))
        f.write(h)
        for t in tensors.values():
            f.write(t.detach().cpu().contiguous().reshape(-1).view(torch.uint8).numpy().tobytes())
