"""Small Lapevik configurations and random weights for the tests."""
import json
import os

import torch

from oracle import lapevik_ref as R
from tests.nunezen_cases import tokens  # noqa: F401  (random ids for a configuration)
from tunix_amd import checkpoint


def moe(ff, experts, top):
  return {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top}}


def ssd(heads, vdim, state, groups=1, conv=4, norm_groups=1, mlp=None, kind="mamba2"):
  return {"type": kind, "mlp": mlp, "mixer": {"heads": heads, "vdim": vdim, "state": state, "groups": groups, "conv": conv,
                                              "norm_groups": norm_groups}}


def latent(heads, dim, rot, vdim, q_rank, kv_rank, base=10_000.0, scale=None, mlp=None):
  return {"type": "latent_attention", "mlp": mlp,
          "mixer": {"heads": heads, "dim": dim, "rot_dim": rot, "vdim": vdim, "q_rank": q_rank, "kv_rank": kv_rank,
                    "rot": {"base": base, "dims": rot}, "scale": (dim + rot) ** -0.5 if scale is None else scale}}


def config(vocab, width, layers, eps=1e-6, groups=1):
  return {"architecture": "Lapevik", "vocab": vocab, "width": width, "norm": {"eps": eps, "groups": groups}, "layers": layers}


CONFIGS = {
    # every mechanism on its aligned kernels; layers with and without a feed-forward
    "mixed": config(320, 128, [latent(5, 32, 16, 48, 64, 80, mlp=moe(48, 9, 3)), ssd(6, 32, 16, 2, 4, 3, moe(64, 4, 1)),
                               ssd(4, 16, 64, 1, 2, 2, None, "mamba2_2"), latent(2, 64, 64, 32, 96, 128, base=500.0, scale=0.2)],
                    groups=4),
    # every expert of every token: nothing hangs on a close call of a router
    "all": config(320, 128, [latent(5, 32, 16, 48, 64, 80, mlp=moe(48, 6, 6)), ssd(6, 32, 16, 2, 4, 3, moe(64, 2, 2)),
                             ssd(4, 16, 64, 1, 2, 2, moe(32, 1, 1), "mamba2_2"), latent(2, 64, 64, 32, 96, 128, base=500.0, scale=0.2)],
                  groups=2),
    # nothing a multiple of eight
    "odd": config(211, 100, [ssd(3, 20, 12, 3, 3, 1, moe(33, 5, 5)), latent(3, 21, 6, 45, 37, 50, scale=0.31, mlp=moe(70, 3, 2)),
                             ssd(4, 10, 7, 2, 5, 4, None, "mamba2_2"), latent(1, 9, 2, 11, 13, 17, mlp=moe(20, 6, 1))], eps=1e-4, groups=5),
    # long latents (the widest cache rows), wide states, one norm group
    "wide": config(512, 192, [latent(3, 128, 64, 128, 160, 320), ssd(2, 136, 160, 2, 4, 1, moe(128, 3, 2)),
                              latent(2, 96, 32, 200, 64, 224, mlp=moe(96, 17, 6)), ssd(2, 64, 256, 1, 3, 2)], eps=1e-3),
    # a latent that no MFMA kernel takes, nothing rotated, a single head
    "latent": config(96, 64, [latent(1, 32, 0, 32, 32, 600), latent(2, 16, 4, 16, 8, 16, base=7.0, mlp=moe(16, 2, 2))], groups=2),
    # a convolution of one tap, one head, several heads of 24 values in a group
    "ssd": config(96, 64, [ssd(1, 32, 32, conv=1), ssd(8, 24, 8, 1, 4, 8, moe(24, 4, 4))], eps=1e-3, groups=8),
}


def random_weights(d: dict, seed: int, sharp: float = 2.0) -> dict:
  """bf16 weights.  `sharp` scales the latent queries so that scores stand out of the average; decays reach from
  a few tokens to hundreds; the router's logits are spread."""
  g = torch.Generator().manual_seed(seed)
  out = {}
  for name, shape in R.tensor_shapes(d).items():
    t = torch.randn(*shape, generator=g)
    if name.endswith("A_log"):
      t = 1.5 * t - 1.0
    elif name.endswith("dt_bias"):
      t = t - 1.5
    elif name.endswith(".shift"):
      t = 0.5 + 0.4 * t
    elif name.endswith("conv.b"):
      t = 0.3 * t
    elif len(shape) == 1:
      t = 1.0 + 0.3 * t
    elif name == "embed":
      t = 0.8 * t
    elif name.endswith("mix.conv"):
      t = t * shape[1] ** -0.5
    else:
      t = t * shape[1] ** -0.5 * (sharp if name.endswith(("mix.uq", "router")) else 1.0)
    out[name] = t.to(torch.bfloat16)
  return out


def write_model(folder, name: str, seed: int) -> tuple:
  d = CONFIGS[name]
  w = random_weights(d, seed)
  with open(os.path.join(folder, "config.json"), "w") as f:
    json.dump(d, f)
  checkpoint.write_safetensors(os.path.join(folder, "model.safetensors"), w)
  return d, w
