"""Checkpoint folders: ``config.json`` and ``*.safetensors``, memory-mapped (nothing in them is executed)."""
from __future__ import annotations

import json
from pathlib import Path

import numpy as np
import torch

_DTYPES = {"BF16": (np.uint16, torch.bfloat16), "F16": (np.float16, torch.float16), "F32": (np.float32, torch.float32),
           "F64": (np.float64, torch.float64), "I64": (np.int64, torch.int64), "I32": (np.int32, torch.int32),
           "I16": (np.int16, torch.int16), "I8": (np.int8, torch.int8), "U8": (np.uint8, torch.uint8),
           "BOOL": (np.bool_, torch.bool)}


def is_checkpoint(path) -> bool:
    return (Path(path) / "config.json").is_file()


def read_config(path) -> dict:
    with open(Path(path) / "config.json") as f:
        return json.load(f)


def _open(path):
    """(mapped bytes, offset of the data, header) of one file: an 8-byte little-endian header length, the JSON
    header (name -> dtype, shape, data_offsets) and the data."""
    raw = np.memmap(path, dtype=np.uint8, mode="r")
    if raw.size < 8:
        raise ValueError(f"{path}: not a safetensors file")
    n = int(raw[:8].view("<u8")[0])
    if n > raw.size - 8:
        raise ValueError(f"{path}: header of {n} bytes in a file of {raw.size}")
    head = json.loads(raw[8:8 + n].tobytes())
    head.pop("__metadata__", None)
    return raw, 8 + n, head


def tensor_shapes(path) -> dict[str, tuple]:
    """Name -> shape of every tensor of a checkpoint folder (headers only)."""
    return {name: tuple(t["shape"]) for f in _files(path) for name, t in _open(f)[2].items()}


def read_safetensors(path, device="cpu") -> dict[str, torch.Tensor]:
    """Every tensor of one file."""
    raw, data, head = _open(path)
    out = {}
    for name, t in head.items():
        if t["dtype"] not in _DTYPES:
            raise ValueError(f"{path}: {name} has dtype {t['dtype']}")
        np_dt, dt = _DTYPES[t["dtype"]]
        lo, hi = (data + o for o in t["data_offsets"])
        want = int(np.prod(t["shape"], dtype=np.int64)) * np.dtype(np_dt).itemsize
        if not data <= lo <= hi <= raw.size or hi - lo != want:
            raise ValueError(f"{path}: {name} has bad offsets")
        a = np.frombuffer(raw[lo:hi].tobytes(), dtype=np_dt).reshape(t["shape"])
        v = torch.from_numpy(a.copy())
        out[name] = (v.view(torch.bfloat16) if dt == torch.bfloat16 else v).to(device)
    return out


def _files(path) -> list[Path]:
    files = sorted(Path(path).glob("*.safetensors"))
    if not files:
        raise FileNotFoundError(f"no *.safetensors in {path}")
    return files


def load_weights(path, device="cpu") -> dict[str, torch.Tensor]:
    out: dict[str, torch.Tensor] = {}
    for f in _files(path):
        out.update(read_safetensors(f, device))
    return out
