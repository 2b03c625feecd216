"""Checkpoint folders: config.json and safetensors files, read without executing anything from them."""
from __future__ import annotations

import glob
import json
import mmap
import os
import struct
from typing import Dict, Iterable

import torch

_DTYPES = {"BF16": torch.bfloat16, "F16": torch.float16, "F32": torch.float32, "F64": torch.float64,
           "I8": torch.int8, "U8": torch.uint8, "I16": torch.int16, "I32": torch.int32, "I64": torch.int64, "BOOL": torch.bool}


def read_config(path: str) -> dict:
    with open(os.path.join(path, "config.json")) as f:
        return json.load(f)


def read_safetensors(path: str) -> Dict[str, torch.Tensor]:
    """The tensors of one file, as views of the mapped file (copy before the mapping is to go away)."""
    with open(path, "rb") as f:
        size = os.fstat(f.fileno()).st_size
        head = f.read(8)
        if len(head) != 8:
            raise ValueError(f"{path}: not a safetensors file")
        n = struct.unpack("<Q", head)[0]
        if n > size - 8:
            raise ValueError(f"{path}: header of {n} bytes in a file of {size}")
        header = json.loads(f.read(n))
        data = mmap.mmap(f.fileno(), 0, access=mmap.ACCESS_COPY)
    out = {}
    for name, t in header.items():
        if name == "__metadata__":
            continue
        dtype, shape, (a, b) = _DTYPES[t["dtype"]], t["shape"], t["data_offsets"]
        count = 1
        for s in shape:
            count *= s
        if not 0 <= a <= b <= size - 8 - n or b - a != count * torch.empty(0, dtype=dtype).element_size():
            raise ValueError(f"{path}: tensor {name} does not fit its place in the file")
        if count == 0:
            out[name] = torch.empty(shape, dtype=dtype)
        elif (8 + n + a) % torch.empty(0, dtype=dtype).element_size():
            out[name] = torch.frombuffer(bytearray(data[8 + n + a:8 + n + b]), dtype=dtype).reshape(shape)
        else:
            out[name] = torch.frombuffer(data, dtype=dtype, count=count, offset=8 + n + a).reshape(shape)
    return out


def read_weights(path: str) -> Dict[str, torch.Tensor]:
    """All tensors of a checkpoint folder (one safetensors file or several)."""
    files = sorted(glob.glob(os.path.join(path, "*.safetensors")))
    if not files:
        raise FileNotFoundError(f"no safetensors file in {path}")
    out: Dict[str, torch.Tensor] = {}
    for f in files:
        out.update(read_safetensors(f))
    return out


def take(weights: Dict[str, torch.Tensor], name: str, shape: Iterable[int]) -> torch.Tensor:
    """The named tensor, with the shape it has to have."""
    if name not in weights:
        raise ValueError(f"checkpoint: tensor {name} is missing")
    shape = tuple(shape)
    t = weights[name]
    if tuple(t.shape) != shape:
        raise ValueError(f"checkpoint: tensor {name} has shape {tuple(t.shape)}, expected {shape}")
    return t


def write_safetensors(path: str, tensors: Dict[str, torch.Tensor]) -> None:
    """Writes contiguous CPU tensors in the same format."""
    names = {v: k for k, v in _DTYPES.items()}
    header: Dict[str, dict] = {}
    off = 0
    for name, t in tensors.items():
        n = t.numel() * t.element_size()
        header[name] = {"dtype": names[t.dtype], "shape": list(t.shape), "data_offsets": [off, off + n]}
        off += n
    head = json.dumps(header).encode()
    head += b" " * (-len(head) % 8)
    with open(path, "wb") as f:
        f.write(struct.pack("<Q", len(head)))
        f.write(head)
        for t in tensors.values():
            t = t.detach().cpu().contiguous()
            f.write(t.reshape(-1).view(torch.uint8).numpy().tobytes() if t.numel() else b"")


