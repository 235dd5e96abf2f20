"""Nunezen without a GPU: reading a configuration, the order of looped layers, file formats, the registry and
the command line's errors, and the plain implementation's mechanisms against closed forms."""
import json
import math

import numpy as np
import pytest
import torch

from oracle import nunezen_ref as R
from tests import nunezen_cases as C
from tunix_amd import checkpoint, cli, config, registry
from tunix_amd.cache import KVSpec, SequenceCache, StateSpec


@pytest.mark.parametrize("name", sorted(C.CONFIGS))
def test_config_reader_names_every_tensor(name):
  d = C.CONFIGS[name]
  cfg = config.nunezen_from_dict(d)
  assert cfg.weight_shapes() == R.tensor_shapes(d)
  assert cfg.layer_runs == R.layer_order(d)
  assert cfg.norm_eps == d["norm"]["eps"]
  for ly, src in zip(cfg.layers, d["layers"]):
    m = src["mixer"]
    assert (ly.mixer.heads, ly.mixer.dim, ly.mixer.vdim) == (m["heads"], m["dim"], m["vdim"])
    if src["type"] == "attention":
      assert (ly.mixer.scale, ly.mixer.rot_base, ly.mixer.rot_dims) == (m["scale"], m["rot"]["base"], m["rot"]["dims"])
    else:
      assert list(ly.mixer.decay) == m["decay"]
    assert (ly.mlp is None) == (src["mlp"] is None)


def test_loop_order():
  d = dict(C.CONFIGS["mixed"])
  n = len(d["layers"])
  d["loop"] = {"start": 1, "stop": 3, "times": 3}
  order = config.nunezen_from_dict(d).layer_runs
  assert order == [(0, False)] + [(1, True), (2, False)] * 3 + [(i, False) for i in range(3, n)]
  d["loop"] = {"start": 0, "stop": n, "times": 1}
  assert config.nunezen_from_dict(d).layer_runs == [(i, i == 0) for i in range(n)]
  d.pop("loop")
  assert config.nunezen_from_dict(d).layer_runs == [(i, False) for i in range(n)]
  d["loop"] = {"start": 2, "stop": n + 1, "times": 2}
  with pytest.raises(ValueError, match="does not fit"):
    config.nunezen_from_dict(d)


@pytest.mark.parametrize("change", [
    lambda d: d["layers"][0].update(type="convolution"),
    lambda d: d["layers"][0]["mlp"].update(kind="experts"),
    lambda d: d["layers"][0]["mixer"].update(kv_heads=4),
    lambda d: d["layers"][0]["mixer"]["rot"].update(dims=7),
    lambda d: d["layers"][1]["mixer"].update(decay=[0.5]),
])
def test_config_reader_rejects_what_the_design_does_not_have(change):
  d = json.loads(json.dumps(C.CONFIGS["mixed"]))
  change(d)
  with pytest.raises(ValueError):
    config.nunezen_from_dict(d)


def test_safetensors_round_trip(tmp_path):
  t = {"a": torch.randn(3, 5).to(torch.bfloat16), "b.c": torch.arange(7, dtype=torch.int32), "s": torch.randn(2, 0, 3),
       "f": torch.randn(4)}
  path = str(tmp_path / "x.safetensors")
  checkpoint.write_safetensors(path, t)
  back = checkpoint.read_safetensors(path)
  assert set(back) == set(t)
  for k in t:
    assert back[k].dtype == t[k].dtype and back[k].shape == t[k].shape and torch.equal(back[k], t[k])
  from safetensors.torch import load_file
  lib = load_file(path)
  assert all(torch.equal(lib[k], t[k]) for k in t)
  raw = open(path, "rb").read()
  open(path, "wb").write(raw[:-4])
  with pytest.raises(ValueError, match="does not fit"):
    checkpoint.read_safetensors(path)


def test_registry_and_command_line(tmp_path):
  C.write_model(tmp_path, "mixed", seed=1)
  arch, cfg = registry.read_config(str(tmp_path))
  assert isinstance(cfg, config.StackConfig) and torch.float32 in arch.dtypes
  q = {"architecture": "llama3", "num_layers": 2, "vocab_size": 64, "embed_dim": 128, "hidden_dim": 256, "num_heads": 2,
       "num_kv_heads": 1, "head_dim": 64}
  (tmp_path / "config.json").write_text(json.dumps(q))
  arch, cfg = registry.read_config(str(tmp_path))
  assert isinstance(cfg, config.ModelConfig) and cfg.family == "llama3" and arch.dtypes == (torch.bfloat16,)
  with pytest.raises(SystemExit) as e:      # a quantised family does not run in fp32: said before anything is loaded
    cli.main(["trace", "--model", str(tmp_path), "--dtype", "float32", "--out", str(tmp_path)])
  assert e.value.code == 3
  with pytest.raises(ValueError, match="unknown architecture"):
    registry.architecture_of({"architecture": "none"})


def test_cache_entries_rows_and_growth():
  specs = [KVSpec(2, 4, 8), StateSpec(3, 4, 5), KVSpec(2, 4, 8)]
  c = SequenceCache(specs, 3, 6, "cpu")
  assert len(c.entries) == 3 and c.entries[0] is not c.entries[2] and len(c.kcache) == 2
  c.entries[0].k.normal_()
  c.entries[1].s.normal_()
  view = c.rows(1, 2)
  assert view.entries[0].k.data_ptr() == c.entries[0].k[1:].data_ptr() and view.entries[1].s.shape[0] == 2
  k, s = c.entries[0].k.clone(), c.entries[1].s.clone()
  c.grow(16)
  assert c.S == 16 and c.entries[0].k.shape == (3, 2, 16, 4) and torch.equal(c.entries[0].k[:, :, :6], k)
  assert not c.entries[0].k[:, :, 6:].any() and torch.equal(c.entries[1].s, s)
  shared = SequenceCache(specs, 1, 4, "cpu", shared=True)
  assert shared.entries[0] is shared.entries[2]


# ---- the plain implementation -------------------------------------------------------------------
def test_oracle_rotation_is_a_rotation_of_its_dimensions_only():
  x = torch.randn(5, 2, 10, dtype=torch.float64)
  y = R.rotate(x, torch.arange(5), 6, 100.0)
  assert torch.equal(y[..., 6:], x[..., 6:]) and torch.equal(y[0], x[0])
  torch.testing.assert_close(y.norm(dim=-1), x.norm(dim=-1))
  z = torch.complex(x[3, 0, 1], x[3, 0, 4]) * torch.exp(torch.tensor(1j * 3 * 100.0 ** (-2 / 6)))
  torch.testing.assert_close(torch.complex(y[3, 0, 1], y[3, 0, 4]), z.to(torch.complex128), rtol=1e-6, atol=1e-6)


def test_oracle_sink_only_enlarges_the_denominator():
  s = torch.tensor([[0.5, -1.0, -math.inf]], dtype=torch.float64)
  p = R.sink_softmax(s, torch.tensor(0.25, dtype=torch.float64))
  den = math.exp(0.5) + math.exp(-1.0) + math.exp(0.25)
  torch.testing.assert_close(p, torch.tensor([[math.exp(0.5) / den, math.exp(-1.0) / den, 0.0]], dtype=torch.float64))


def test_oracle_recurrence_equals_the_weighted_sum():
  g = torch.Generator().manual_seed(0)
  T, H, dk, dv = 9, 2, 3, 4
  q, k, v = (torch.randn(T, H, n, generator=g, dtype=torch.float64) for n in (dk, dk, dv))
  decay = [0.7, 1.0]
  o, S = R.lightning_recurrence(q, k, v, decay)
  for t in range(T):
    for h in range(H):
      want = sum(decay[h] ** (t - j) * (q[t, h] @ k[j, h]) * v[j, h] for j in range(t + 1))
      torch.testing.assert_close(o[t, h], want)
  first, mid = R.lightning_recurrence(q[:4], k[:4], v[:4], decay)
  rest, end = R.lightning_recurrence(q[4:], k[4:], v[4:], decay, mid)
  torch.testing.assert_close(torch.cat([first, rest]), o)
  torch.testing.assert_close(end, S)


def test_oracle_norm_and_gelu():
  x = torch.tensor([[3.0, 4.0]], dtype=torch.float64)
  w = torch.tensor([0.0, 1.0], dtype=torch.float64)
  r = 1.0 / math.sqrt(12.5 + 0.1)
  torch.testing.assert_close(R.rms_norm(x, w, 0.1), torch.tensor([[3 * r, 8 * r]], dtype=torch.float64))
  torch.testing.assert_close(R.rms_norm(x, w, 0.1, around_zero=False), torch.tensor([[0.0, 4 * r]], dtype=torch.float64))
  z = torch.linspace(-4, 4, 33)
  torch.testing.assert_close(R.gelu_tanh(z), torch.nn.functional.gelu(z, approximate="tanh"))


def test_oracle_is_causal():
  d = C.CONFIGS["mixed"]
  w = C.random_weights(d, 3)
  toks = C.tokens(d, 20, 4)
  a = R.forward(d, w, toks, torch.float64)
  other = list(toks)
  other[12] = (other[12] + 1) % d["vocab"]
  b = R.forward(d, w, other, torch.float64)
  assert torch.allclose(a[:12], b[:12], atol=1e-5) and not torch.allclose(a[12:], b[12:], atol=1e-3)
  np.testing.assert_allclose(a[:7].numpy(), R.forward(d, w, toks[:7], torch.float64).numpy(), atol=1e-8)
