"""Small Kuzezen configurations and random weights for the tests."""
import json
import os

import torch

from oracle import kuzezen_ref as R
from tests.nunezen_cases import tokens  # noqa: F401  (random ids for a configuration)
from tunix_amd import checkpoint


def left(heads, kv_heads, dim, vdim, conv=4, scale=None, coef=0.2, every=16):
  return {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": conv, "scale": dim ** -0.5 if scale is None else scale,
          "q_temp": {"coef": coef, "every": every}}


def right(heads, dim, vdim, cap=8.0):
  return {"heads": heads, "dim": dim, "vdim": vdim, "gate_cap": cap}


def layer(a, b, ff=None):
  return {"type": "parallel", "mixer": {"left": a, "right": b}, "mlp": None if ff is None else {"kind": "dense", "ff": ff}}


def config(vocab, width, layers, taps=3, eps=1e-6, loop=None, mult=0.7, scale=3.0, cap=20.0):
  d = {"architecture": "Kuzezen", "vocab": vocab, "width": width, "norm": {"eps": eps}, "layers": layers, "canon": {"taps": taps},
       "embedding": {"scale": scale}, "residual_mult": mult, "logit_softcap": cap}
  if loop is not None:
    d["loop"] = dict(zip(("start", "stop", "times"), loop))
  return d


CONFIGS = {
    # unlike layers with and without a feed-forward, a loop in the middle, the statistics head
    "mixed": config(320, 128, [layer(left(6, 2, 32, 48, conv=3), right(3, 16, 40), 160), layer(left(4, 4, 64, 24, conv=2, scale=0.2, coef=0.5, every=7), right(2, 64, 128, 4.0)),
                               layer(left(8, 1, 24, 64), right(5, 40, 16), 96)], taps=4, loop=(1, 3, 2)),
    # nothing a multiple of eight
    "odd": config(211, 100, [layer(left(3, 3, 21, 13, conv=5, coef=-0.1, every=3), right(2, 11, 9), 33), layer(left(10, 5, 12, 45, conv=1, scale=0.31), right(3, 20, 30, 2.5), 70)],
                  taps=6, eps=1e-4, loop=(0, 1, 3), mult=1.0, scale=1.0, cap=5.0),
    # wide heads, many of them, one tap, no loop
    "wide": config(512, 192, [layer(left(16, 2, 136, 200, conv=4), right(2, 160, 136), 256), layer(left(20, 5, 64, 96, conv=2), right(4, 96, 24, 30.0), None),
                              layer(left(32, 8, 40, 48), right(1, 128, 264), 64)], taps=1, eps=1e-3, mult=0.4),
    # heads that no MFMA kernel of a prompt takes, one layer, run twice
    "heads": config(96, 72, [layer(left(40, 8, 16, 8, conv=2), right(9, 8, 8), 40)], taps=2, loop=(0, 1, 2), mult=1.3),
}


def random_weights(d: dict, seed: int, sharp: float = 2.0) -> dict:
  """bf16 weights.  `sharp` scales the attention's queries so that scores stand out of the average; the memory's forget
  gates reach from a few tokens to hundreds; the heads' mixture has large parts off its diagonal, of both signs."""
  g = torch.Generator().manual_seed(seed)
  out = {}
  for name, shape in R.tensor_shapes(d).items():
    t = torch.randn(*shape, generator=g)
    if name.endswith("f.b"):
      t = 2.0 + 2.0 * t
    elif name.endswith(".talk"):
      t = torch.eye(shape[0]) + 0.6 * shape[0] ** -0.5 * t
    elif "canon" in name or name.endswith(".conv"):
      t = t * shape[1] ** -0.5
    elif len(shape) == 1:
      t = t if name.endswith("i.b") else 1.0 + 0.3 * t
    elif name in ("embed", "loop.step"):
      t = 0.8 * t
    else:
      t = t * shape[1] ** -0.5 * (sharp if name.endswith("left.q") else 1.0)
    out[name] = t.to(torch.bfloat16)
  return out


def write_model(folder, name: str, seed: int) -> tuple:
  d = CONFIGS[name]
  w = random_weights(d, seed)
  with open(os.path.join(folder, "config.json"), "w") as f:
    json.dump(d, f)
  checkpoint.write_safetensors(os.path.join(folder, "model.safetensors"), w)
  return d, w
