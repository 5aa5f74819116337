"""Checkpoint folders for the tests, and token ids."""
import json
import os

import torch


def write_safetensors(path, tensors):
    names = {torch.bfloat16: "BF16", torch.float32: "F32",
             torch.int32: "I32"}
    header, blobs, at = {}, [], 0
    for k, t in tensors.items():
        raw = t.contiguous().view(torch.uint8).numpy().tobytes() \
            if t.dim() else b""
        header[k] = {"dtype": names[t.dtype], "shape": list(t.shape),
                     "data_offsets": [at, at + len(raw)]}
        blobs.append(raw)
        at += len(raw)
    head = json.dumps(header).encode()
    with open(path, "wb") as f:
        f.write(len(head).to_bytes(8, "little") + head + b"".join(blobs))


def write_model(folder, cfg, weights):
    """-> (folder path, weights)."""
    os.makedirs(folder, exist_ok=True)
    with open(os.path.join(folder, "config.json"), "w") as f:
        json.dump(cfg, f)
    write_safetensors(os.path.join(folder, "model.safetensors"), weights)
    return str(folder), weights


def tokens(cfg, n, seed=0):
    g = torch.Generator().manual_seed(1000 + seed)
    return torch.randint(0, cfg["vocab"], (n,), generator=g).tolist()
