"""safetensors files: an 8-byte little-endian header length, a JSON header {name: {dtype, shape, data_offsets}}, the data.

The reader maps the file and hands tensors out as numpy arrays; bfloat16, which numpy does not have, comes as its raw
16-bit patterns (`bits`) or widened (`f32`).  A small writer produces files of the same layout.
"""
from __future__ import annotations

import json
import struct

import numpy as np

DTYPES = {"BF16": np.dtype("<u2"), "F16": np.dtype("<f2"), "F32": np.dtype("<f4"), "F64": np.dtype("<f8"),
          "I8": np.dtype("<i1"), "U8": np.dtype("<u1"), "I16": np.dtype("<i2"), "I32": np.dtype("<i4"),
          "I64": np.dtype("<i8"), "BOOL": np.dtype("?")}


class SafetensorsError(ValueError):
    pass


class SafetensorsFile:
    def __init__(self, path: str):
        self.data = np.memmap(path, np.uint8, "r")
        if self.data.size < 8:
            raise SafetensorsError("file ends inside the header length")
        (n,) = struct.unpack("<Q", self.data[:8].tobytes())
        if 8 + n > self.data.size:
            raise SafetensorsError("file ends inside the header")
        try:
            header = json.loads(self.data[8:8 + n].tobytes().decode("utf-8"))
        except (UnicodeDecodeError, json.JSONDecodeError) as e:
            raise SafetensorsError(f"header is not JSON: {e}") from None
        header.pop("__metadata__", None)
        self.start, self.tensors = 8 + n, {}
        for name, t in header.items():
            if t["dtype"] not in DTYPES:
                raise SafetensorsError(f"tensor {name}: unknown dtype {t['dtype']}")
            begin, end = t["data_offsets"]
            shape = tuple(int(d) for d in t["shape"])
            want = int(np.prod(shape, dtype=np.int64)) * DTYPES[t["dtype"]].itemsize
            if begin < 0 or end - begin != want or self.start + end > self.data.size:
                raise SafetensorsError(f"tensor {name}: {end - begin} bytes for shape {shape} of {t['dtype']}")
            self.tensors[name] = (t["dtype"], shape, begin, end)

    def __contains__(self, name: str) -> bool:
        return name in self.tensors

    def raw(self, name: str):
        """(dtype name, array); BF16 as its 16-bit patterns."""
        if name not in self.tensors:
            raise SafetensorsError(f"no tensor named {name}")
        dtype, shape, begin, end = self.tensors[name]
        return dtype, np.frombuffer(self.data[self.start + begin:self.start + end].tobytes(), DTYPES[dtype]).reshape(shape)

    def bits(self, name: str) -> np.ndarray:
        """A bfloat16 tensor's 16-bit patterns."""
        dtype, a = self.raw(name)
        if dtype != "BF16":
            raise SafetensorsError(f"tensor {name} is {dtype}, not BF16")
        return a

    def f32(self, name: str) -> np.ndarray:
        dtype, a = self.raw(name)
        if dtype == "BF16":
            return (a.astype(np.uint32) << 16).view(np.float32)
        return a.astype(np.float32)


def write(path: str, tensors: dict) -> None:
    """tensors: {name: (dtype name, array)}; BF16 arrays are uint16 patterns."""
    header, offset, parts = {}, 0, []
    for name, (dtype, a) in tensors.items():
        a = np.ascontiguousarray(a)
        if a.dtype != DTYPES[dtype]:
            raise SafetensorsError(f"tensor {name}: array of {a.dtype} for {dtype}")
        header[name] = {"dtype": dtype, "shape": list(a.shape), "data_offsets": [offset, offset + a.nbytes]}
        offset += a.nbytes
        parts.append(a.tobytes())
    head = json.dumps(header).encode("utf-8")
    head += b" " * (-len(head) % 8)
    with open(path, "wb") as f:
        f.write(struct.pack("<Q", len(head)) + head)
        for p in parts:
            f.write(p)
