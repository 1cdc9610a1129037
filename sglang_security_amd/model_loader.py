"""Checkpoints from a folder with config.json and *.safetensors.

A safetensors file is an 8-byte little-endian length, that many bytes of JSON (name -> dtype, shape, data_offsets), and
the tensors' bytes; it is mapped, and tensors are copied out one at a time."""
from __future__ import annotations

import glob
import json
import mmap
import os
import struct
from typing import Dict, Optional, Tuple

import torch

_DTYPES = {"F64": torch.float64, "F32": torch.float32, "F16": torch.float16, "BF16": torch.bfloat16, "I64": torch.int64,
           "I32": torch.int32, "I16": torch.int16, "I8": torch.int8, "U8": torch.uint8, "BOOL": torch.bool}


class SafetensorsFile:
    def __init__(self, path: str):
        self.path = path
        with open(path, "rb") as f:
            self._map = mmap.mmap(f.fileno(), 0, access=mmap.ACCESS_READ)
        if len(self._map) < 8:
            raise ValueError(f"{path}: not a safetensors file")
        n = struct.unpack("<Q", self._map[:8])[0]
        if n > len(self._map) - 8:
            raise ValueError(f"{path}: header longer than the file")
        self._data = 8 + n
        self.index = {k: v for k, v in json.loads(self._map[8: 8 + n].decode("utf-8")).items() if k != "__metadata__"}

    def get(self, name: str) -> torch.Tensor:
        e = self.index[name]
        if e["dtype"] not in _DTYPES:
            raise ValueError(f"{self.path}: {name} has unknown type {e['dtype']}")
        dt, shape = _DTYPES[e["dtype"]], list(e["shape"])
        lo, hi = e["data_offsets"]
        count = 1
        for s in shape:
            count *= s
        if not 0 <= lo <= hi <= len(self._map) - self._data or hi - lo != count * dt.itemsize:
            raise ValueError(f"{self.path}: {name} does not lie within the file")
        if count == 0:
            return torch.empty(shape, dtype=dt)
        return torch.frombuffer(bytearray(self._map[self._data + lo: self._data + hi]), dtype=dt).view(shape)


class Weights:
    """Tensors by name, on the device and in the activation type unless asked otherwise."""

    def __init__(self, tensors, dtype: torch.dtype, device):
        """tensors: a folder's files (load_weights) or a mapping name -> tensor."""
        self._tensors, self.dtype, self.device = tensors, dtype, device
        self.used = set()

    def __contains__(self, name):
        return name in self._tensors

    def get(self, name: str, shape: Tuple[Optional[int], ...], dtype: torch.dtype = None) -> torch.Tensor:
        """shape: None where the tensor itself gives the size."""
        if name not in self._tensors:
            raise ValueError(f"the checkpoint has no tensor {name}")
        t = self._tensors[name]
        t = t() if callable(t) else t
        if len(t.shape) != len(shape) or any(want is not None and n != want for n, want in zip(t.shape, shape)):
            raise ValueError(f"{name}: shape {tuple(t.shape)}, the configuration asks for {tuple(shape)}")
        self.used.add(name)
        return t.to(device=self.device, dtype=dtype or self.dtype)

    def check_all_used(self):
        left = sorted(set(self._tensors) - self.used)
        if left:
            raise ValueError(f"tensors the model does not know: {', '.join(left[:8])}{' ...' if len(left) > 8 else ''}")


def load_config(folder: str) -> dict:
    with open(os.path.join(folder, "config.json")) as f:
        return json.load(f)


def load_weights(folder: str, dtype: torch.dtype, device) -> Weights:
    tensors: Dict[str, object] = {}
    files = sorted(glob.glob(os.path.join(folder, "*.safetensors")))
    if not files:
        raise FileNotFoundError(f"no *.safetensors in {folder}")
    for path in files:
        f = SafetensorsFile(path)
        for name in f.index:
            tensors[name] = lambda f=f, name=name: f.get(name)
    return Weights(tensors, dtype, device)
