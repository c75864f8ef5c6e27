"""Reader and writer of the safetensors file format (an 8-byte little-endian
header length, a JSON header ``name -> {dtype, shape, data_offsets}``, then the
data). Tensors are views of one memory-mapped file: nothing is copied until a
caller moves them to a device."""
from __future__ import annotations

import json
import mmap
import struct
from pathlib import Path

import torch

DTYPES = {"F64": torch.float64, "F32": torch.float32, "F16": torch.float16, "BF16": torch.bfloat16,
          "I64": torch.int64, "I32": torch.int32, "I16": torch.int16, "I8": torch.int8, "U8": torch.uint8,
          "BOOL": torch.bool}
MAX_HEADER = 100 << 20


def load_file(path) -> dict[str, torch.Tensor]:
    path = Path(path)
    size = path.stat().st_size
    with open(path, "rb") as f:
        if size < 8:
            raise ValueError(f"{path}: too short for a safetensors file")
        (n,) = struct.unpack("<Q", f.read(8))
        if n > min(MAX_HEADER, size - 8):
            raise ValueError(f"{path}: bad header length {n}")
        header = json.loads(f.read(n))
        data = mmap.mmap(f.fileno(), 0, access=mmap.ACCESS_COPY)  # private: writable views, file untouched
    base, out = 8 + n, {}
    for name, d in header.items():
        if name == "__metadata__":
            continue
        dt = DTYPES.get(d["dtype"])
        if dt is None:
            raise ValueError(f"{path}: tensor {name} has unsupported dtype {d['dtype']}")
        lo, hi = d["data_offsets"]
        count = 1
        for s in d["shape"]:
            count *= s
        if lo < 0 or hi - lo != count * dt.itemsize or base + hi > size:
            raise ValueError(f"{path}: tensor {name} does not fit the file")
        if count == 0:
            out[name] = torch.empty(d["shape"], dtype=dt)
            continue
        out[name] = torch.frombuffer(data, dtype=dt, count=count, offset=base + lo).reshape(d["shape"])
    return out


def save_file(tensors: dict[str, torch.Tensor], path) -> None:
    names = {v: k for k, v in DTYPES.items()}
    header, blobs, off = {}, [], 0
    for name, t in tensors.items():
        t = t.detach().cpu().contiguous()
        raw = t.reshape(-1).view(torch.uint8).numpy().tobytes() if t.numel() else b""
        header[name] = {"dtype": names[t.dtype], "shape": list(t.shape), "data_offsets": [off, off + len(raw)]}
        blobs.append(raw)
        off += len(raw)
    h = json.dumps(header).encode()
    h += b" " * (-len(h) % 8)
    with open(path, "wb") as f:
        f.write(struct.pack("<Q", len(h)))
        f.write(h)
        for b in blobs:
            f.write(b)
