"""Language models from a folder: config.json + model.safetensors.

The model class is chosen by config.json: "architecture" (Fasovik, Fogorax) or "model_type" (nano, qwen2).  A model names its
checkpoint tensors in `checkpoint_tensors()` — views into its (possibly stacked) parameters — or, without that method, by
its parameter names.  Loading is strict: every tensor of the file has one place, every place is filled, shapes agree."""
from __future__ import annotations

import json
import math
import mmap
import os
import struct
from pathlib import Path
from typing import Dict, Iterator, Tuple

import torch

_DTYPES = {"BF16": torch.bfloat16, "F16": torch.float16, "F32": torch.float32, "F64": torch.float64, "I64": torch.int64,
           "I32": torch.int32, "I16": torch.int16, "I8": torch.int8, "U8": torch.uint8, "BOOL": torch.bool}


def read_safetensors(path) -> Iterator[Tuple[str, torch.Tensor]]:
    """(name, CPU tensor) of every tensor of the file: an 8-byte little-endian header length, a JSON header (name -> dtype,
    shape, byte range), the data.  The file is mapped, one tensor is copied at a time."""
    size = os.path.getsize(path)
    with open(path, "rb") as f:
        n = struct.unpack("<Q", f.read(8))[0]
        if n > size - 8:
            raise ValueError(f"{path}: header of {n} bytes in a file of {size}")
        header = json.loads(f.read(n))
        with mmap.mmap(f.fileno(), 0, access=mmap.ACCESS_READ) as m:
            for name, t in header.items():
                if name == "__metadata__":
                    continue
                lo, hi = (8 + n + int(o) for o in t["data_offsets"])
                dt, shape = _DTYPES[t["dtype"]], tuple(t["shape"])
                if not 8 + n <= lo <= hi <= size or hi - lo != math.prod(shape) * dt.itemsize:
                    raise ValueError(f"{path}: bad byte range of {name}")
                raw = bytearray(m[lo:hi])
                yield name, (torch.frombuffer(raw, dtype=dt) if raw else torch.empty(0, dtype=dt)).view(shape)


@torch.no_grad()
def load_weights(model, path) -> None:
    places: Dict[str, torch.Tensor] = dict(model.checkpoint_tensors() if hasattr(model, "checkpoint_tensors")
                                           else model.state_dict(keep_vars=True))
    for name, t in read_safetensors(path):
        dst = places.pop(name, None)
        if dst is None:
            raise ValueError(f"{path}: no place for tensor {name} in {type(model).__name__}")
        if tuple(dst.shape) != tuple(t.shape):
            raise ValueError(f"{path}: {name} is {tuple(t.shape)}, the configuration says {tuple(dst.shape)}")
        dst.copy_(t)
    if places:
        raise ValueError(f"{path}: missing tensors {sorted(places)[:8]}")


def load_llm(folder, dtype=torch.bfloat16, device=None):
    """The causal LM of a checkpoint folder, ready for inference (`GenericLLMBackbone.llm`)."""
    from .llm_factory import config_from_dict, llm_class
    folder = Path(folder)
    config = config_from_dict(json.loads((folder / "config.json").read_text()))
    device = torch.device(device if device is not None else "cuda")
    with torch.device("meta"):
        model = llm_class(config)(config)
    model = model.to(dtype).to_empty(device=device)
    load_weights(model, folder / "model.safetensors")
    return model.requires_grad_(False).eval()
