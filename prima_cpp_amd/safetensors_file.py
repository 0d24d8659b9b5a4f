"""Read-only view of a .safetensors file: 8-byte little-endian header length, JSON header (name -> dtype, shape, data_offsets), then the data, which is mapped and handed
to the weight uploader as it lies."""
import json
import mmap
import os
import struct

import numpy as np

from .lib import BF16, F32, PM355Error

_ITEM = {"F64": 8, "F32": 4, "F16": 2, "BF16": 2, "I64": 8, "I32": 4, "I16": 2, "I8": 1, "U8": 1, "BOOL": 1}
_TYPE = {"BF16": BF16, "F32": F32}


class SafetensorsFile:
    """.tensors: name -> (dtype string, shape tuple, uint8 view)"""

    def __init__(self, path):
        self.path = path
        size = os.path.getsize(path)
        with open(path, "rb") as f:
            if size < 8:
                raise PM355Error(f"{path}: too short for a safetensors file")
            (n,) = struct.unpack("<Q", f.read(8))
            if n > size - 8:
                raise PM355Error(f"{path}: header length {n} exceeds the file")
            header = json.loads(f.read(n))
            self._mm = mmap.mmap(f.fileno(), 0, access=mmap.ACCESS_READ)
        buf = np.frombuffer(self._mm, dtype=np.uint8)
        self.tensors = {}
        for name, t in header.items():
            if name == "__metadata__":
                continue
            lo, hi = t["data_offsets"]
            want = int(np.prod(t["shape"], dtype=np.int64)) * _ITEM.get(t["dtype"], 0)
            if not 0 <= lo <= hi <= size - 8 - n or hi - lo != want:
                raise PM355Error(f"{path}: tensor {name}: data_offsets do not fit dtype and shape")
            self.tensors[name] = (t["dtype"], tuple(t["shape"]), buf[8 + n + lo:8 + n + hi])

    def get(self, name, shape):
        """(pm355 type, bytes) of a tensor that must have this shape"""
        if name not in self.tensors:
            raise PM355Error(f"{self.path}: tensor {name} is missing")
        dtype, have, data = self.tensors[name]
        if have != tuple(shape):
            raise PM355Error(f"{self.path}: tensor {name} is {list(have)}, expected {list(shape)}")
        if dtype not in _TYPE:
            raise PM355Error(f"{self.path}: tensor {name}: dtype {dtype} is not served (BF16, F32)")
        return _TYPE[dtype], data
