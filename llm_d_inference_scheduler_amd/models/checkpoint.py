"""Named weights: from a safetensors file, or drawn at random.

The file is mapped and its tensors are handed out without copies. The format
is an 8-byte little-endian header length, a JSON header (name -> dtype, shape,
data_offsets) and the raw tensor bytes.
"""
import json
import math
import os
from typing import Callable, Dict

import torch

from ..utils.logging import get_logger

log = get_logger("models.checkpoint")

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


def weights(folder: str, shapes: Dict[str, tuple], random_tensor: Callable,
            device: torch.device, seed: int) -> Callable[[str], torch.Tensor]:
    """-> take(name): the tensor in its stored precision on `device`, from
    the checkpoint folder or, without one, random_tensor(name, shape, fill)
    where fill(shape, std) draws normal values."""
    if folder:
        files = read_safetensors(os.path.join(folder, "model.safetensors"))
        missing = sorted(set(shapes) - set(files))
        if missing:
            raise ValueError(f"{folder}: missing tensors {missing}")
        if len(files) > len(shapes):
            log.warning("unused tensors", names=sorted(set(files)
                                                       - set(shapes)))

        def take(name):
            t = files[name]
            if tuple(t.shape) != shapes[name]:
                raise ValueError(f"{name}: shape {tuple(t.shape)}, expected "
                                 f"{shapes[name]}")
            return t.to(device)
        return take
    # drawn on the device itself: a checkpoint-sized CPU init would dominate
    # start-up. One seed gives every rank the same weights.
    gen = torch.Generator(device=device).manual_seed(seed)

    def take(name):
        def fill(shape, std):
            return torch.empty(shape, dtype=torch.float32,
                               device=device).normal_(0.0, std,
                                                      generator=gen)
        return random_tensor(name, shapes[name], fill).to(torch.bfloat16)
    return take
