"""Reader of safetensors folders: an 8-byte little-endian header length, a JSON table of names,
dtypes, shapes and byte ranges, then the data.  Tensors are views of the mapped file until a model
copies them to its device."""
from __future__ import annotations

import json
import os

import torch

_DTYPES = {"BF16": torch.bfloat16, "F16": torch.float16, "F32": torch.float32, "F64": torch.float64,
           "I64": torch.int64, "I32": torch.int32, "I16": torch.int16, "I8": torch.int8,
           "U8": torch.uint8, "BOOL": torch.bool}


def read_safetensors(path: str) -> dict[str, torch.Tensor]:
    size = os.path.getsize(path)
    with open(path, "rb") as f:
        head_len = int.from_bytes(f.read(8), "little")
        if not 0 < head_len <= size - 8:
            raise ValueError(f"{path}: not a safetensors file")
        table = json.loads(f.read(head_len))
    base = 8 + head_len
    data = torch.from_file(path, shared=False, size=size, dtype=torch.uint8)
    out = {}
    for name, t in table.items():
        if name == "__metadata__":
            continue
        dtype = _DTYPES[t["dtype"]]
        lo, hi = t["data_offsets"]
        count = 1
        for n in t["shape"]:
            count *= n
        if not 0 <= lo <= hi <= size - base or hi - lo != count * dtype.itemsize:
            raise ValueError(f"{path}: {name} does not fit its byte range")
        raw = data[base + lo:base + hi]
        if (base + lo) % dtype.itemsize:
            raw = raw.clone()
        out[name] = raw.view(dtype).reshape(t["shape"])
    return out


def read_folder(folder: str) -> dict[str, torch.Tensor]:
    """All tensors of a model folder (one file, or several shards)."""
    files = sorted(f for f in os.listdir(folder) if f.endswith(".safetensors"))
    if not files:
        raise FileNotFoundError(f"{folder} holds no .safetensors file")
    out: dict[str, torch.Tensor] = {}
    for f in files:
        out.update(read_safetensors(os.path.join(folder, f)))
    return out


def write_safetensors(path: str, tensors: dict[str, torch.Tensor]) -> None:
    """The inverse, for exported and generated models."""
    names = {v: k for k, v in _DTYPES.items()}
    table, blobs, at = {}, [], 0
    for name, t in tensors.items():
        t = t.detach().cpu().contiguous()
        blob = t.reshape(-1).view(torch.uint8).numpy().tobytes()
        table[name] = {"dtype": names[t.dtype], "shape": list(t.shape), "data_offsets": [at, at + len(blob)]}
        blobs.append(blob)
        at += len(blob)
    head = json.dumps(table).encode()
    head += b" " * (-len(head) % 8)
    with open(path, "wb") as f:
        f.write(len(head).to_bytes(8, "little") + head)
        for b in blobs:
            f.write(b)
