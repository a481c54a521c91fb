"""Reading checkpoints: a folder with config.json and model.safetensors.

A safetensors file is an 8-byte little-endian header length, that many bytes of JSON (name -> dtype, shape,
data_offsets) and the data.  The file is mapped, not read: a tensor costs memory when it is copied to where it is used.
"""
from __future__ import annotations

import json
import math
import mmap
import os
import struct
from typing import Dict

import torch

from ._capi import TahDuoError

_DTYPES = {"BF16": torch.bfloat16, "F16": torch.float16, "F32": torch.float32, "F64": torch.float64, "I8": torch.int8, "U8": torch.uint8,
           "I16": torch.int16, "I32": torch.int32, "I64": torch.int64, "BOOL": torch.bool}


def read_config(folder: str) -> dict:
    with open(os.path.join(folder, "config.json")) as f:
        return json.load(f)


def read_safetensors(path: str) -> Dict[str, torch.Tensor]:
    """The file's tensors as views of a private mapping of it (pages are copied when written to)."""
    with open(path, "rb") as f:
        m = mmap.mmap(f.fileno(), 0, access=mmap.ACCESS_COPY)
    if len(m) < 8:
        raise TahDuoError(f"{path}: not a safetensors file")
    n = struct.unpack("<Q", m[:8])[0]
    if n > len(m) - 8:
        raise TahDuoError(f"{path}: the header is longer than the file")
    header, out = json.loads(m[8:8 + n]), {}
    for name, e in header.items():
        if name == "__metadata__":
            continue
        if e["dtype"] not in _DTYPES:
            raise TahDuoError(f"{path}: tensor {name} has the unknown type {e['dtype']}")
        dt, shape, (a, b) = _DTYPES[e["dtype"]], e["shape"], e["data_offsets"]
        count = math.prod(shape)
        size = torch.empty(0, dtype=dt).element_size()
        if a < 0 or b > len(m) - 8 - n or b - a != count * size:
            raise TahDuoError(f"{path}: tensor {name} does not fit the file")
        if count == 0:
            out[name] = torch.empty(shape, dtype=dt)
        elif (8 + n + a) % size:  # (a view needs an aligned start)
            out[name] = torch.frombuffer(bytearray(m[8 + n + a:8 + n + b]), dtype=dt).view(shape)
        else:
            out[name] = torch.frombuffer(m, dtype=dt, count=count, offset=8 + n + a).view(shape)
    return out


def write_safetensors(path: str, tensors: Dict[str, torch.Tensor]) -> None:
    names = {v: k for k, v in _DTYPES.items()}
    header, at, data = {}, 0, []
    for name, t in tensors.items():
        raw = t.detach().cpu().contiguous().reshape(-1).view(torch.uint8).numpy().tobytes()
        header[name] = {"dtype": names[t.dtype], "shape": list(t.shape), "data_offsets": [at, at + len(raw)]}
        at += len(raw)
        data.append(raw)
    text = json.dumps(header).encode()
    text += b" " * (-len(text) % 8)
    with open(path, "wb") as f:
        f.write(struct.pack("<Q", len(text)) + text)
        for raw in data:
            f.write(raw)


def read_tensors(folder: str) -> Dict[str, torch.Tensor]:
    return read_safetensors(os.path.join(folder, "model.safetensors"))
