"""Architectures by name: how a model folder (config.json + model.safetensors) becomes a
configuration and a model on the GPU."""
from __future__ import annotations

import dataclasses
import json
import os
from typing import Callable

import torch

from . import config
from .checkpoint import read_safetensors
from .model import QLoRAModel
from .stack_model import StackModel


@dataclasses.dataclass(frozen=True)
class Architecture:
  read_config: Callable[[dict], object]
  build: Callable[..., object]          # (cfg, weights, device, dtype) -> model
  dtypes: tuple = (torch.bfloat16,)


def _qlora_config(d: dict) -> config.ModelConfig:
  """config.json of the quantised families: the fields of ModelConfig, "architecture" naming the family."""
  kw = {k: tuple(v) if isinstance(v, list) else v for k, v in d.items() if k != "architecture"}
  return config.ModelConfig(family=d["architecture"], **kw)


_QLORA = Architecture(_qlora_config, lambda cfg, w, device, dtype: QLoRAModel(cfg, w, device))


def _stack(reader) -> Architecture:
  """A decoder given layer by layer."""
  return Architecture(reader, lambda cfg, w, device, dtype: StackModel(cfg, w, device, dtype), (torch.bfloat16, torch.float32))


ARCHITECTURES: dict[str, Architecture] = {
    "llama3": _QLORA,
    "qwen3": _QLORA,
    "gemma3": _QLORA,
    "Nunezen": _stack(config.nunezen_from_dict),
    "Lapevik": _stack(config.lapevik_from_dict),
    "Kuzezen": _stack(config.kuzezen_from_dict),
    "Kezolix": _stack(config.kezolix_from_dict),
}


def architecture_of(d: dict) -> Architecture:
  name = d.get("architecture")
  if name not in ARCHITECTURES:
    raise ValueError(f"unknown architecture {name!r}; known: {sorted(ARCHITECTURES)}")
  return ARCHITECTURES[name]


def read_config(folder: str):
  """(architecture entry, configuration) of a model folder."""
  with open(os.path.join(folder, "config.json")) as f:
    d = json.load(f)
  arch = architecture_of(d)
  return arch, arch.read_config(d)


def load_model(folder: str, device="cuda", dtype=torch.bfloat16):
  """The model of a folder, on the GPU."""
  arch, cfg = read_config(folder)
  if dtype not in arch.dtypes:
    raise ValueError(f"this architecture runs in {[str(t) for t in arch.dtypes]}, not in {dtype}")
  return arch.build(cfg, read_safetensors(os.path.join(folder, "model.safetensors")), device, dtype)
