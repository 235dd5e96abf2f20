"""Small Kezolix configurations and random weights for the tests."""
import json
import os

import torch

from oracle import kezolix_ref as R
from tests.nunezen_cases import tokens  # noqa: F401  (random ids for a configuration)
from tunix_amd import checkpoint


def dense(ff):
  return {"kind": "dense", "ff": ff}


def moe(ff, experts, top, shared, scale=1.0):
  return {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top, "scale": scale}, "shared": {"ff": shared}}


def attention(heads, kv_heads, dim, vdim, chunk, mlp=None, scale=None, kv_from=None):
  m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "mask": {"size": chunk}, "scale": dim ** -0.5 if scale is None else scale}
  if kv_from is not None:
    m["kv_from"] = kv_from
  return {"type": "attention", "mixer": m, "mlp": mlp}


def state(heads, dim, vdim, mlp=None):
  return {"type": "hgrn2", "mixer": {"heads": heads, "dim": dim, "vdim": vdim}, "mlp": mlp}


def config(vocab, width, layers, eps=1e-6, mult=0.7, positions=320):
  return {"architecture": "Kezolix", "vocab": vocab, "width": width, "norm": {"eps": eps}, "layers": layers, "max_positions": positions, "residual_mult": mult}


CONFIGS = {
    # every kind of layer and feed-forward, with and without one; keys borrowed twice, over a layer of the same sizes
    "mixed": config(320, 128, [state(3, 32, 48, dense(160)), attention(6, 2, 32, 48, 20, moe(48, 9, 3, 80, 1.7)), state(2, 64, 40),
                               attention(6, 2, 32, 48, 33, None, 0.3), attention(6, 2, 32, 48, 50, moe(64, 4, 1, 64, 0.6), 0.25, kv_from=1),
                               attention(6, 2, 32, 48, 17, dense(96), kv_from=1)]),
    # every expert of every token: nothing hangs on a close call of a router
    "all": config(320, 128, [attention(4, 1, 64, 24, 40, moe(48, 6, 6, 96, 2.5)), state(5, 16, 32, moe(80, 2, 2, 80)), attention(4, 1, 64, 24, 9, dense(200), kv_from=0),
                             state(2, 128, 64, moe(32, 1, 1, 40, 0.4))], mult=0.5),
    # nothing a multiple of eight
    "odd": config(211, 100, [attention(3, 3, 21, 13, 7, moe(33, 5, 2, 99, 3.0)), state(3, 11, 9, dense(70)), attention(3, 3, 21, 13, 1000, kv_from=0, scale=0.31),
                             state(1, 20, 30, moe(20, 6, 1, 20)), attention(10, 5, 12, 45, 1)], eps=1e-3, mult=1.0, positions=200),
    # wide heads and many of them
    "wide": config(512, 192, [state(1, 200, 136, dense(256)), attention(16, 2, 136, 200, 64, moe(128, 3, 3, 128)), state(2, 256, 264),
                              attention(20, 5, 64, 96, 130, dense(64)), attention(16, 2, 136, 200, 45, kv_from=1), state(4, 96, 24)], eps=1e-4, mult=0.4, positions=400),
    # one recurrent layer
    "one": config(96, 72, [state(9, 8, 8, dense(40))], mult=1.3, positions=64),
}


def random_weights(d: dict, seed: int, sharp: float = 2.5) -> dict:
  """bf16 weights.  `sharp` scales the queries' norm weights so that scores stand out of the average; forget gates reach from
  a few tokens to hundreds; no layer's result drops out of the average over depth."""
  g = torch.Generator().manual_seed(seed)
  out = {}
  for name, shape in R.tensor_shapes(d).items():
    t = torch.randn(*shape, generator=g)
    if name.endswith("f.b"):
      t = 2.0 + 2.0 * t
    elif name.endswith(".lower"):
      t = (0.3 + 0.4 * t).clamp(0.0, 0.98)
    elif name.endswith(".dwa"):
      t = 0.4 * t
      t[-1] += 0.8
    elif name.endswith("mlp.act"):
      t = 0.5 * t + 0.3
    elif name.endswith(".correction"):
      t = 0.2 * t
    elif name.endswith("q.norm"):
      t = sharp * (1.0 + 0.3 * t)
    elif len(shape) == 1:
      t = 1.0 + 0.3 * t
    elif name in ("embed", "pos"):
      t = 0.8 * t
    else:
      t = t * shape[1] ** -0.5 * (2.0 if name.endswith("router") else 1.0)
    out[name] = t.to(torch.bfloat16)
  return out


def write_model(folder, name: str, seed: int) -> tuple:
  d = CONFIGS[name]
  w = random_weights(d, seed)
  with open(os.path.join(folder, "config.json"), "w") as f:
    json.dump(d, f)
  checkpoint.write_safetensors(os.path.join(folder, "model.safetensors"), w)
  return d, w
