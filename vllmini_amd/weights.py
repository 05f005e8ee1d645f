"""Checkpoints in the safetensors format: 8 bytes of length, a JSON header (name -> dtype, shape, data_offsets), the data."""
from __future__ import annotations

import json
import mmap
import os
from typing import Dict, Optional

import numpy as np
import torch

_TYPES = {"BF16": (np.uint16, torch.bfloat16), "F16": (np.float16, None), "F32": (np.float32, None), "F64": (np.float64, None),
          "I64": (np.int64, None), "I32": (np.int32, None), "I16": (np.int16, None), "I8": (np.int8, None), "U8": (np.uint8, None),
          "BOOL": (np.bool_, None)}


def read_safetensors(path: str, device: Optional[torch.device] = None) -> Dict[str, torch.Tensor]:
    """Every tensor of one file, as stored, on `device` (default: CPU)."""
    with open(path, "rb") as f:
        size = os.fstat(f.fileno()).st_size
        n = int.from_bytes(f.read(8), "little")
        if size < 8 or n > size - 8:
            raise ValueError(f"{path}: the header is longer than the file")
        header = json.loads(f.read(n))
        base, out = 8 + n, {}
        data = mmap.mmap(f.fileno(), 0, access=mmap.ACCESS_READ) if size > base else b""
        for name, info in header.items():
            if name == "__metadata__":
                continue
            if info["dtype"] not in _TYPES:
                raise ValueError(f"{path}: {name} has type {info['dtype']}")
            np_type, view = _TYPES[info["dtype"]]
            a, b = info["data_offsets"]
            shape = [int(x) for x in info["shape"]]
            count = int(np.prod(shape, dtype=np.int64))
            if a < 0 or b - a != count * np.dtype(np_type).itemsize or base + b > size:
                raise ValueError(f"{path}: the extent of {name} does not fit its shape or the file")
            arr = np.frombuffer(data, dtype=np_type, count=count, offset=base + a).copy() if count else np.zeros(0, np_type)
            t = torch.from_numpy(arr)
            t = (t.view(view) if view is not None else t).view(shape)
            out[name] = t.to(device) if device is not None else t
    return out


def load_checkpoint(model_dir: str, device: Optional[torch.device] = None) -> Dict[str, torch.Tensor]:
    """The tensors of every *.safetensors file of a folder."""
    files = sorted(f for f in os.listdir(model_dir) if f.endswith(".safetensors"))
    if not files:
        raise FileNotFoundError(f"no *.safetensors file in {model_dir}")
    out: Dict[str, torch.Tensor] = {}
    for f in files:
        out.update(read_safetensors(os.path.join(model_dir, f), device))
    return out
