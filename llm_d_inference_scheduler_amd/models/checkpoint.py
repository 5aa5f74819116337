"""Safetensors reader: maps the file and hands out tensors without copies.

The format is an 8-byte little-endian header length, a JSON header
(name -> dtype, shape, data_offsets) and the raw tensor bytes.
"""
import json
import math
import os
from typing import Dict

import torch

_DTYPES = {"F64": torch.float64, "F32": torch.float32, "F16": torch.float16,
           "BF16": torch.bfloat16, "I64": torch.int64, "I32": torch.int32,
           "I16": torch.int16, "I8": torch.int8, "U8": torch.uint8,
           "BOOL": torch.bool}


def read_safetensors(path: str) -> Dict[str, torch.Tensor]:
    """-> {name: CPU tensor}, copy-on-write views of the mapped file."""
    size = os.path.getsize(path)
    if size < 8:
        raise ValueError(f"{path}: not a safetensors file")
    raw = torch.from_file(path, shared=False, size=size, dtype=torch.uint8)
    n = int.from_bytes(bytes(raw[:8].tolist()), "little")
    if n > size - 8:
        raise ValueError(f"{path}: header of {n} bytes in {size}")
    header = json.loads(bytes(raw[8:8 + n].tolist()).decode("utf-8"))
    data = raw[8 + n:]
    out = {}
    for name, info in header.items():
        if name == "__metadata__":
            continue
        dtype = _DTYPES[info["dtype"]]
        lo, hi = info["data_offsets"]
        shape = info["shape"]
        if hi - lo != math.prod(shape) * dtype.itemsize or \
                not 0 <= lo <= hi <= data.numel():
            raise ValueError(f"{path}: bad extent of {name}")
        piece = data[lo:hi]
        if piece.data_ptr() % dtype.itemsize:
            piece = piece.clone()
        out[name] = piece.view(dtype).view(shape)
    return out
