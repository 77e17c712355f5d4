"""Checkpoint folders: config.json beside model.safetensors.

A safetensors file is an 8-byte little-endian length, that many bytes of JSON (name -> dtype, shape, data_offsets) and the data.
bf16 values are handled as numpy uint16 (their bit patterns)."""
import json
import os
import struct

import numpy as np

_NP = {"BF16": np.uint16, "F16": np.float16, "F32": np.float32, "I32": np.int32}
_NAME = {np.dtype(v): k for k, v in _NP.items()}


def read_config(folder):
    with open(os.path.join(folder, "config.json"), encoding="utf-8") as f:
        return json.load(f)


def read_safetensors(path):
    """name -> numpy view onto a read-only memory map."""
    mm = np.memmap(path, np.uint8, "r")
    if mm.size < 8:
        raise ValueError(f"{path}: not a safetensors file")
    n = struct.unpack("<Q", mm[:8].tobytes())[0]
    if n > mm.size - 8:
        raise ValueError(f"{path}: the header runs past the end of the file")
    head, out = json.loads(mm[8:8 + n].tobytes()), {}
    for name, info in head.items():
        if name == "__metadata__":
            continue
        if info["dtype"] not in _NP:
            raise ValueError(f"{path}: tensor {name} has unsupported type {info['dtype']}")
        lo, hi = info["data_offsets"]
        dt, shape = np.dtype(_NP[info["dtype"]]), tuple(info["shape"])
        if not 0 <= lo <= hi <= mm.size - 8 - n or hi - lo != dt.itemsize * int(np.prod(shape)):
            raise ValueError(f"{path}: tensor {name} does not fit its place in the file")
        raw = mm[8 + n + lo:8 + n + hi]
        if (8 + n + lo) % dt.itemsize:
            raw = raw.copy()
        out[name] = raw.view(dt).reshape(shape)
    return out


def write_safetensors(path, tensors):
    head, blobs, off = {}, [], 0
    for name, a in tensors.items():
        a = np.ascontiguousarray(a)
        head[name] = {"dtype": _NAME[a.dtype], "shape": list(a.shape), "data_offsets": [off, off + a.nbytes]}
        blobs.append(a)
        off += a.nbytes
    raw = json.dumps(head).encode()
    raw += b" " * (-len(raw) % 8)
    with open(path, "wb") as f:
        f.write(struct.pack("<Q", len(raw)))
        f.write(raw)
        for a in blobs:
            f.write(a.tobytes())


def bf16_bits(x):
    """float32 -> bf16 bit patterns, round to nearest even."""
    u = np.ascontiguousarray(x, np.float32).view(np.uint32)
    return ((u + 0x7FFF + ((u >> 16) & 1)) >> 16).astype(np.uint16)


def bf16_floats(bits):
    return (np.ascontiguousarray(bits, np.uint16).astype(np.uint32) << 16).view(np.float32)


def as_f32(a):
    return bf16_floats(a) if a.dtype == np.uint16 else np.asarray(a, np.float32)


def as_bf16(a):
    return np.ascontiguousarray(a) if a.dtype == np.uint16 else bf16_bits(a)
