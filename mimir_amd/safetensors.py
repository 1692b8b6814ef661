"""Reader for safetensors files: an 8-byte little-endian length, that many bytes
of JSON (name -> dtype, shape, data_offsets), then the tensors' bytes. The
file is mapped, so a tensor's bytes are read when it is uploaded."""
from __future__ import annotations

import json
import struct

import numpy as np

# numpy has no bfloat16: its bits
_DTYPES = {"BF16": np.dtype("<u2"), "F16": np.dtype("<f2"), "F32": np.dtype("<f4"), "I32": np.dtype("<i4"), "I64": np.dtype("<i8"), "U8": np.dtype("u1")}


class SafetensorsError(ValueError):
    pass


class SafetensorsFile:
    """tensors: name -> (dtype name, array of the tensor's shape)."""

    def __init__(self, path: str):
        self.path = path
        with open(path, "rb") as f:
            head = f.read(8)
            if len(head) != 8:
                raise SafetensorsError(f"{path}: not a safetensors file")
            n = struct.unpack("<Q", head)[0]
            raw = f.read(n) if n < 1 << 30 else b""
            if len(raw) != n:
                raise SafetensorsError(f"{path}: header of {n} bytes is cut short")
            f.seek(0, 2)
            size = f.tell() - 8 - n
        try:
            index = json.loads(raw)
        except ValueError as e:
            raise SafetensorsError(f"{path}: header: {e}") from e
        data = np.memmap(path, np.uint8, "r", 8 + n, (size,)) if size else np.empty(0, np.uint8)
        self.tensors: dict[str, tuple[str, np.ndarray]] = {}
        for name, t in index.items():
            if name == "__metadata__":
                continue
            dt, shape, (lo, hi) = t["dtype"], tuple(t["shape"]), t["data_offsets"]
            if dt not in _DTYPES:
                raise SafetensorsError(f"{path}: {name}: dtype {dt}")
            if not 0 <= lo <= hi <= size or hi - lo != int(np.prod(shape, dtype=np.int64)) * _DTYPES[dt].itemsize:
                raise SafetensorsError(f"{path}: {name}: bytes {lo}..{hi} of {size} for {shape} {dt}")
            self.tensors[name] = (dt, data[lo:hi].view(_DTYPES[dt]).reshape(shape))
