"""Small Nunezen configurations and random weights for the tests."""
import json
import os

import numpy as np
import torch

from oracle import nunezen_ref as R
from tunix_amd import checkpoint


def attention(heads, kv_heads, dim, vdim, rot, base=10_000.0, scale=None, ff=None):
  return {"type": "attention", "mlp": None if ff is None else {"kind": "dense", "ff": ff},
          "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim,
                    "rot": {"base": base, "dims": rot}, "scale": dim ** -0.5 if scale is None else scale}}


def lightning(heads, dim, vdim, decay, ff=None):
  return {"type": "lightning", "mlp": None if ff is None else {"kind": "dense", "ff": ff},
          "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "decay": list(decay)}}


def config(vocab, width, layers, eps=1e-6, loop=None):
  d = {"architecture": "Nunezen", "vocab": vocab, "width": width, "norm": {"eps": eps}, "layers": layers}
  if loop is not None:
    d["loop"] = dict(zip(("start", "stop", "times"), loop))
  return d


CONFIGS = {
    # both mixers with and without a feed-forward, loop over the first layers, every kernel's aligned path
    "mixed": config(320, 128, [attention(6, 2, 48, 64, 32, ff=160), lightning(4, 16, 40, [0.5, 0.9, 0.99, 1.0], ff=96),
                               attention(4, 4, 64, 32, 64, base=500.0, scale=0.2), lightning(2, 64, 128, [0.0, 0.97])],
                    loop=(0, 2, 3)),
    # nothing a multiple of eight: vocabulary, width, heads, feed-forward, rotated dimensions
    "odd": config(211, 100, [lightning(3, 20, 36, [0.8, 0.95, 0.999]), attention(10, 5, 21, 45, 6, scale=0.31, ff=70),
                             lightning(5, 12, 10, [0.3, 0.6, 0.9, 0.99, 0.7], ff=33)], eps=1e-5, loop=(1, 3, 2)),
    # wide heads, one kv head, a head group that is no power of two, no loop
    "wide": config(512, 192, [attention(5, 1, 136, 200, 2, ff=384), lightning(2, 160, 136, [0.9, 0.996]),
                              attention(3, 3, 256, 96, 128, scale=-0.05)]),
    "attention": config(96, 64, [attention(4, 2, 32, 32, 0, ff=64)], loop=(0, 1, 2)),
    "lightning": config(96, 64, [lightning(2, 32, 32, [0.9, 0.98]), lightning(1, 8, 264, [0.95])], eps=1e-3),
}


def random_weights(d: dict, seed: int, sharp: float = 2.0) -> dict:
  """bf16 weights; `sharp` scales the attention queries so that scores stand out of the average."""
  g = torch.Generator().manual_seed(seed)
  out = {}
  for name, shape in R.tensor_shapes(d).items():
    t = torch.randn(*shape, generator=g)
    if name.endswith("mix.norm"):
      t = 1.0 + 0.3 * t
    elif name.endswith("sink"):
      t = 1.5 * t
    elif len(shape) == 1:
      t = 0.3 * t
    elif name == "embed":
      t = 0.8 * t
    else:
      t = t * shape[1] ** -0.5 * (sharp if name.endswith("mix.q") else 1.0)
    out[name] = t.to(torch.bfloat16)
  return out


def tokens(d: dict, n: int, seed: int) -> list:
  """Random ids, 0 and the last one among them."""
  t = np.random.Generator(np.random.PCG64(seed)).integers(0, d["vocab"], size=n)
  if n > 4:
    t[1], t[3] = 0, d["vocab"] - 1
  return [int(x) for x in t]


def write_model(folder, name: str, seed: int) -> tuple:
  d = CONFIGS[name]
  w = random_weights(d, seed)
  with open(os.path.join(folder, "config.json"), "w") as f:
    json.dump(d, f)
  checkpoint.write_safetensors(os.path.join(folder, "model.safetensors"), w)
  return d, w
