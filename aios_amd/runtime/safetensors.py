"""Memory-mapped reader of safetensors files: an 8-byte little-endian header length, that many bytes of
JSON (name -> dtype, shape, data_offsets into what follows), then the tensor data.

Raw bytes only (numpy has no bfloat16); nothing in the file is executed.
"""
from __future__ import annotations

import json
import mmap
import os
from typing import Dict, NamedTuple, Tuple

import numpy as np

_ITEM = {"BF16": 2, "F16": 2, "F32": 4, "F64": 8, "I64": 8, "I32": 4, "I16": 2, "I8": 1, "U8": 1, "BOOL": 1}


class TensorInfo(NamedTuple):
    dtype: str
    shape: Tuple[int, ...]
    begin: int
    end: int


class SafetensorsReader:
    def __init__(self, path: str):
        self.path = path
        with open(path, "rb") as f:
            size = os.fstat(f.fileno()).st_size
            head = f.read(8)
            if len(head) != 8:
                raise ValueError(f"{path}: not a safetensors file")
            n = int.from_bytes(head, "little")
            if n <= 0 or 8 + n > size:
                raise ValueError(f"{path}: bad safetensors header length")
            meta = json.loads(f.read(n))
            self._mm = mmap.mmap(f.fileno(), 0, access=mmap.ACCESS_READ)
        base = 8 + n
        self.tensors: Dict[str, TensorInfo] = {}
        for name, t in meta.items():
            if name == "__metadata__":
                continue
            shape = tuple(int(x) for x in t["shape"])
            b, e = (base + int(x) for x in t["data_offsets"])
            count = 1
            for x in shape:
                count *= x
            if t["dtype"] not in _ITEM or not base <= b <= e <= size or e - b != count * _ITEM[t["dtype"]]:
                raise ValueError(f"{path}: tensor {name}: offsets do not fit its shape")
            self.tensors[name] = TensorInfo(t["dtype"], shape, b, e)

    def raw(self, name: str) -> np.ndarray:
        """The tensor's bytes (uint8 view of the mapping)."""
        t = self.tensors[name]
        return np.frombuffer(self._mm, np.uint8, t.end - t.begin, t.begin)


def write(path: str, tensors: Dict[str, Tuple[str, Tuple[int, ...], bytes]]):
    """Write {name: (dtype, shape, bytes)}."""
    meta, off = {}, 0
    for name, (dtype, shape, data) in tensors.items():
        meta[name] = {"dtype": dtype, "shape": list(shape), "data_offsets": [off, off + len(data)]}
        off += len(data)
    head = json.dumps(meta).encode()
    head += b" " * (-len(head) % 8)
    with open(path, "wb") as f:
        f.write(len(head).to_bytes(8, "little"))
        f.write(head)
        for _, _, data in tensors.values():
            f.write(data)
