"""Model registry and checkpoint loading: a folder with config.json (its "architecture" chooses the class) and *.safetensors.

A registered class has ``config_class`` (with ``from_dict``), takes the config, and may map its parameter names to the
checkpoint's with ``checkpoint_name``: a name, or a list of names whose tensors are stacked (a mixture's experts).
"""
from __future__ import annotations

import glob
import json
import mmap
import os
import struct
from typing import Callable, Dict

import torch
import torch.nn as nn

MODELS: Dict[str, type] = {}

_DTYPES = {"F64": torch.float64, "F32": torch.float32, "F16": torch.float16, "BF16": torch.bfloat16, "I64": torch.int64,
           "I32": torch.int32, "I16": torch.int16, "I8": torch.int8, "U8": torch.uint8, "BOOL": torch.bool}


def register_model(name: str) -> Callable[[type], type]:
    def add(cls: type) -> type:
        MODELS[name] = cls
        return cls
    return add


def model_class(architecture: str) -> type:
    from . import biruvik, gisitar, padulorn, rivudra  # noqa: F401  (they register themselves)
    if architecture not in MODELS:
        raise ValueError(f"architecture {architecture!r} is not registered (known: {sorted(MODELS)})")
    return MODELS[architecture]


def read_safetensors(path: str) -> Dict[str, torch.Tensor]:
    """{name: tensor} of one file, views of a private memory map (copied when they move to the device)."""
    with open(path, "rb") as f:
        size = os.fstat(f.fileno()).st_size
        head = f.read(8)
        n = struct.unpack("<Q", head)[0] if len(head) == 8 else size
        if 8 + n > size:
            raise ValueError(f"{path}: not a safetensors file")
        header = json.loads(f.read(n))
        data = mmap.mmap(f.fileno(), 0, access=mmap.ACCESS_COPY)
    out = {}
    for name, t in header.items():
        if name == "__metadata__":
            continue
        a, b = t["data_offsets"]
        dt, shape = _DTYPES[t["dtype"]], t["shape"]
        count = 1
        for s in shape:
            count *= s
        if b - a != count * dt.itemsize or 8 + n + b > size or a < 0:
            raise ValueError(f"{path}: tensor {name!r} does not fit its place in the file")
        flat = torch.frombuffer(data, dtype=torch.uint8, count=b - a, offset=8 + n + a) if count else torch.empty(0, dtype=torch.uint8)
        if (8 + n + a) % dt.itemsize:
            flat = flat.clone()
        out[name] = flat.view(dt).view(shape)
    return out


def load_checkpoint(model: nn.Module, tensors: Dict[str, torch.Tensor], dtype: torch.dtype, device) -> None:
    """Put every parameter of `model` (which may live on the meta device) in place; names, shapes and completeness checked."""
    rename = getattr(model, "checkpoint_name", lambda n: n)
    left = set(tensors)
    for name, p in list(model.named_parameters()):
        keys = rename(name)
        stacked = isinstance(keys, list)
        parts = []
        for key in keys if stacked else [keys]:
            if key not in tensors:
                raise KeyError(f"the checkpoint lacks {key!r}")
            t, want = tensors[key], tuple(p.shape[1:] if stacked else p.shape)
            if tuple(t.shape) != want:
                raise ValueError(f"{key}: shape {tuple(t.shape)} in the checkpoint, {want} in the model")
            left.discard(key)
            parts.append(t)
        if stacked:
            full = torch.empty(p.shape, dtype=dtype, device=device)
            for i, t in enumerate(parts):
                full[i].copy_(t)
        else:
            full = parts[0].to(device=device, dtype=dtype)
        owner, _, leaf = name.rpartition(".")
        setattr(model.get_submodule(owner), leaf, nn.Parameter(full, requires_grad=p.requires_grad))
    if left:
        raise KeyError(f"the model has no place for {sorted(left)[:4]}{' ...' if len(left) > 4 else ''}")


def load_pretrained(folder: str, dtype: torch.dtype = torch.bfloat16, device="cuda") -> nn.Module:
    """Model of the class that folder/config.json names, with the weights of folder/*.safetensors, in eval mode."""
    with open(os.path.join(folder, "config.json")) as f:
        config = json.load(f)
    cls = model_class(config["architecture"])
    files = sorted(glob.glob(os.path.join(folder, "*.safetensors")))
    if not files:
        raise FileNotFoundError(f"no *.safetensors in {folder}")
    tensors: Dict[str, torch.Tensor] = {}
    for f in files:
        tensors.update(read_safetensors(f))
    with torch.device("meta"):
        model = cls(cls.config_class.from_dict(config))
    load_checkpoint(model, tensors, dtype, device)
    return model.eval()
