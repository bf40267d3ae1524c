"""safetensors files: an 8-byte little-endian length, that many bytes of JSON (name -> dtype, shape, data_offsets), the data.

Memory-mapped; a tensor comes back in its stored type (bfloat16 as uint16 bit patterns) with `bf16_to_f32` beside it.
"""
import json
import mmap
import os
import struct

import numpy as np

_NP = {"F32": np.float32, "F16": np.float16, "BF16": np.uint16, "I32": np.int32, "I64": np.int64, "F64": np.float64,
       "U8": np.uint8, "I8": np.int8}


def bf16_to_f32(bits):
    return (np.ascontiguousarray(bits).astype(np.uint32) << 16).view(np.float32)


def f32_to_bf16(x):
    """Bit patterns, rounded to nearest, ties to even."""
    u = np.ascontiguousarray(x, np.float32).view(np.uint32)
    r = ((u + 0x7FFF + ((u >> 16) & 1)) >> 16).astype(np.uint16)
    return np.where(np.isnan(x), np.uint16(0x7FC0), r)


class SafetensorsFile:
    def __init__(self, path):
        self._f = open(path, "rb")
        size = os.fstat(self._f.fileno()).st_size
        if size < 8:
            raise ValueError(f"{path}: not a safetensors file")
        self._mm = mmap.mmap(self._f.fileno(), 0, access=mmap.ACCESS_READ)
        n = struct.unpack("<Q", self._mm[:8])[0]
        if n > size - 8:
            raise ValueError(f"{path}: header length {n} exceeds the file")
        head = json.loads(self._mm[8:8 + n].decode("utf-8"))
        self._at = 8 + n
        self.entries = {k: v for k, v in head.items() if k != "__metadata__"}
        for k, v in self.entries.items():
            lo, hi = v["data_offsets"]
            if v["dtype"] not in _NP:
                raise ValueError(f"{path}: tensor {k} has type {v['dtype']}, which is not supported")
            want = int(np.prod(v["shape"], dtype=np.int64)) * np.dtype(_NP[v["dtype"]]).itemsize
            if not (0 <= lo <= hi <= size - self._at) or hi - lo != want:
                raise ValueError(f"{path}: tensor {k} does not fit its data range")

    def __contains__(self, name):
        return name in self.entries

    def names(self):
        return list(self.entries)

    def shape(self, name):
        return tuple(self.entries[name]["shape"])

    def raw(self, name):
        """The stored values (bfloat16: bit patterns), without a copy."""
        e = self.entries[name]
        lo, hi = e["data_offsets"]
        dt = np.dtype(_NP[e["dtype"]])
        if hi == lo:
            return np.zeros(e["shape"], dt)
        return np.frombuffer(self._mm, dt, count=(hi - lo) // dt.itemsize, offset=self._at + lo).reshape(e["shape"])

    def f32(self, name):
        r = self.raw(name)
        return bf16_to_f32(r) if self.entries[name]["dtype"] == "BF16" else r.astype(np.float32)

    def bf16(self, name):
        """bfloat16 bit patterns; float types are rounded."""
        e = self.entries[name]
        return self.raw(name) if e["dtype"] == "BF16" else f32_to_bf16(self.raw(name).astype(np.float32))

    def is_bf16_exact(self, name):
        return self.entries[name]["dtype"] == "BF16"


class TensorDict:
    """The same access over arrays in memory (float arrays, or uint16 bit patterns for bfloat16)."""

    def __init__(self, tensors):
        self.tensors = dict(tensors)

    def __contains__(self, name):
        return name in self.tensors

    def names(self):
        return list(self.tensors)

    def shape(self, name):
        return tuple(self.tensors[name].shape)

    def f32(self, name):
        t = self.tensors[name]
        return bf16_to_f32(t) if t.dtype == np.uint16 else np.ascontiguousarray(t, np.float32)

    def bf16(self, name):
        t = self.tensors[name]
        return t if t.dtype == np.uint16 else f32_to_bf16(t)

    def is_bf16_exact(self, name):
        t = self.tensors[name]
        return t.dtype == np.uint16 or np.array_equal(bf16_to_f32(f32_to_bf16(t)), np.asarray(t, np.float32))
