"""safetensors files: an 8-byte little-endian header length, a JSON header
(name -> dtype, shape, data_offsets) and the tensors' bytes."""
from __future__ import annotations

import json
import os

import numpy as np
import torch

_DTYPES = {"BF16": torch.bfloat16, "F16": torch.float16, "F32": torch.float32, "F64": torch.float64,
           "I8": torch.int8, "I16": torch.int16, "I32": torch.int32, "I64": torch.int64, "U8": torch.uint8,
           "BOOL": torch.bool}
_NAMES = {v: k for k, v in _DTYPES.items()}


def read_safetensors(path: str) -> dict[str, torch.Tensor]:
  """All tensors of the file, in host memory."""
  size = os.path.getsize(path)
  with open(path, "rb") as f:
    head = f.read(8)
    n = int.from_bytes(head, "little")
    if len(head) != 8 or n > size - 8:
      raise ValueError(f"{path}: not a safetensors file")
    index = json.loads(f.read(n))
  raw = np.memmap(path, dtype=np.uint8, mode="r") if size > 8 + n else np.zeros(size, dtype=np.uint8)
  out = {}
  for name, meta in index.items():
    if name == "__metadata__":
      continue
    dtype, shape = _DTYPES.get(meta["dtype"]), tuple(meta["shape"])
    if dtype is None:
      raise ValueError(f"{path}: tensor {name} has the unknown dtype {meta['dtype']}")
    a, b = meta["data_offsets"]
    count = int(np.prod(shape, dtype=np.int64)) * torch.empty(0, dtype=dtype).element_size()
    if not 0 <= a <= b <= size - 8 - n or b - a != count:
      raise ValueError(f"{path}: tensor {name} does not fit the file")
    if count == 0:
      out[name] = torch.empty(shape, dtype=dtype)
      continue
    out[name] = torch.from_numpy(np.array(raw[8 + n + a: 8 + n + b])).view(dtype).reshape(shape)
  return out


def write_safetensors(path: str, tensors: dict[str, torch.Tensor]) -> None:
  index, at, parts = {}, 0, []
  for name, t in tensors.items():
    data = t.detach().cpu().contiguous().reshape(-1).view(torch.uint8).numpy().tobytes()
    index[name] = {"dtype": _NAMES[t.dtype], "shape": list(t.shape), "data_offsets": [at, at + len(data)]}
    at += len(data)
    parts.append(data)
  head = json.dumps(index).encode()
  head += b" " * (-len(head) % 8)
  with open(path, "wb") as f:
    f.write(len(head).to_bytes(8, "little"))
    f.write(head)
    for p in parts:
      f.write(p)
