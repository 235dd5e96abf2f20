"""Lapevik without a GPU: reading a configuration, the cache's entries, the registry, and the plain implementation's
mechanisms against closed forms."""
import json
import math

import pytest
import torch

from oracle import lapevik_ref as R
from tests import lapevik_cases as C
from tunix_amd import config, dummy_model, registry
from tunix_amd.cache import LatentSpec, PartsSpec, RingSpec, SequenceCache, StateSpec


@pytest.mark.parametrize("name", sorted(C.CONFIGS))
def test_config_reader_names_every_tensor(name):
  d = C.CONFIGS[name]
  cfg = config.lapevik_from_dict(d)
  assert cfg.weight_shapes() == R.tensor_shapes(d)
  assert (cfg.norm_eps, cfg.norm_groups, cfg.norm_offset) == (d["norm"]["eps"], d["norm"]["groups"], 0.0)
  assert cfg.token_shift and cfg.embed_norm and not cfg.pre_norm and cfg.loop is None
  for ly, src in zip(cfg.layers, d["layers"]):
    m = src["mixer"]
    if src["type"] in R.RECURRENT:
      assert isinstance(ly.mixer, config.SsdMixer)
      assert all(getattr(ly.mixer, k) == m[k] for k in ("heads", "vdim", "state", "groups", "conv", "norm_groups"))
    else:
      assert all(getattr(ly.mixer, k) == m[k] for k in ("heads", "dim", "rot_dim", "vdim", "q_rank", "kv_rank", "scale"))
      assert not m["rot_dim"] or ly.mixer.rot_base == m["rot"]["base"]
    e = src["mlp"]
    assert (ly.mlp is None) == (e is None)
    if e is not None:
      assert (ly.mlp.ff, ly.mlp.experts, ly.mlp.top) == (e["expert"]["ff"], e["router"]["experts"], e["router"]["top"])


@pytest.mark.parametrize("change", [
    lambda d: d["layers"][0].update(type="attention"),
    lambda d: d["layers"][0]["mlp"].update(kind="dense"),
    lambda d: d["layers"][0]["mlp"]["router"].update(top=10),
    lambda d: d["layers"][0]["mixer"]["rot"].update(dims=8),
    lambda d: d["layers"][1]["mixer"].update(groups=4),
    lambda d: d["layers"][1]["mixer"].update(norm_groups=5),
    lambda d: d["layers"][1]["mixer"].update(conv=0),
    lambda d: d["norm"].update(groups=3),
])
def test_config_reader_rejects_what_the_design_does_not_have(change):
  d = json.loads(json.dumps(C.CONFIGS["mixed"]))
  change(d)
  with pytest.raises(ValueError):
    config.lapevik_from_dict(d)


def test_registry_and_benchmark_shapes(tmp_path):
  C.write_model(tmp_path, "odd", seed=1)
  arch, cfg = registry.read_config(str(tmp_path))
  assert isinstance(cfg, config.StackConfig) and cfg.family == "lapevik" and torch.float32 in arch.dtypes
  w = dummy_model.create_stack_weights(cfg, 3)
  assert {k: tuple(t.shape) for k, t in w.items()} == cfg.weight_shapes()


def test_cache_entries_of_several_parts():
  spec = PartsSpec((("mixer", PartsSpec((("state", StateSpec(2, 3, 4)), ("conv", RingSpec(4, 5))))), ("shift", RingSpec(1, 6, torch.float32))))
  c = SequenceCache([spec, LatentSpec(8), spec], 3, 6, "cpu")
  ring = c.entries[0]["mixer"]["conv"].r
  ring.normal_()
  c.entries[1].c.normal_()
  view = c.rows(1, 2)
  assert view.entries[0]["mixer"]["conv"].r.data_ptr() == ring[1:].data_ptr() and view.entries[0]["shift"].r.shape == (2, 1, 6)
  lat, keep = c.entries[1].c.clone(), ring.clone()
  c.grow(16)
  assert c.entries[1].c.shape == (3, 16, 8) and torch.equal(c.entries[1].c[:, :6], lat) and not c.entries[1].c[:, 6:].any()
  assert torch.equal(c.entries[0]["mixer"]["conv"].r, keep)
  shared = SequenceCache([spec, LatentSpec(8), spec], 1, 4, "cpu", shared=True)
  assert shared.entries[0] is shared.entries[2]


# ---- the plain implementation -------------------------------------------------------------------
def test_oracle_norm_in_groups():
  x = torch.tensor([[3.0, 4.0, 0.0, 2.0]], dtype=torch.float64)
  w = torch.tensor([1.0, 2.0, 1.0, 0.5], dtype=torch.float64)
  a, b = 1 / math.sqrt(12.5 + 0.1), 1 / math.sqrt(2.0 + 0.1)
  torch.testing.assert_close(R.group_norm(x, w, 0.1, 2), torch.tensor([[3 * a, 8 * a, 0.0, b]], dtype=torch.float64))


def test_oracle_shift_and_convolution_carry_over_a_cut():
  g = torch.Generator().manual_seed(1)
  x, mix = torch.randn(9, 4, generator=g), torch.randn(4, generator=g)
  y = R.token_shift(x, mix)
  torch.testing.assert_close(y[0], x[0] * (1 - mix))
  torch.testing.assert_close(y[5], x[5] + (x[4] - x[5]) * mix)
  torch.testing.assert_close(torch.cat([R.token_shift(x[:3], mix), R.token_shift(x[3:], mix, x[2])]), y)
  taps, bias = torch.randn(4, 3, generator=g), torch.randn(4, generator=g)
  c = R.short_conv(x, taps, bias)
  torch.testing.assert_close(c[0], bias + taps[:, 2] * x[0])
  torch.testing.assert_close(c[4], bias + taps[:, 2] * x[4] + taps[:, 1] * x[3] + taps[:, 0] * x[2])
  torch.testing.assert_close(torch.cat([R.short_conv(x[:4], taps, bias), R.short_conv(x[4:], taps, bias, x[2:4])]), c)


def test_oracle_recurrence_equals_the_weighted_sum():
  g = torch.Generator().manual_seed(0)
  T, H, P, G, N = 7, 4, 3, 2, 5
  x, B, Cm = (torch.randn(T, *s, generator=g, dtype=torch.float64) for s in ((H, P), (G, N), (G, N)))
  dt, A, D = torch.rand(T, H, generator=g, dtype=torch.float64), torch.randn(H, generator=g, dtype=torch.float64), torch.randn(H, generator=g, dtype=torch.float64)
  y, S = R.ssd_recurrence(x, B, Cm, dt, A, D)
  for t in range(T):
    for h in range(H):
      want = D[h] * x[t, h]
      for j in range(t + 1):
        decay = math.exp(-math.exp(A[h]) * float(dt[j + 1:t + 1, h].sum()))
        want = want + decay * dt[j, h] * (Cm[t, h // 2] @ B[j, h // 2]) * x[j, h]
      torch.testing.assert_close(y[t, h], want)
  a, mid = R.ssd_recurrence(x[:3], B[:3], Cm[:3], dt[:3], A, D)
  b, end = R.ssd_recurrence(x[3:], B[3:], Cm[3:], dt[3:], A, D, mid)
  torch.testing.assert_close(torch.cat([a, b]), y)
  torch.testing.assert_close(end, S)


def test_oracle_rotation_pairs_neighbours():
  x = torch.randn(5, 2, 6, dtype=torch.float64)
  y = R.rotate_interleaved(x, torch.arange(5), 100.0)
  assert torch.equal(y[0], x[0])
  z = torch.complex(x[3, 1, 2], x[3, 1, 3]) * torch.exp(torch.tensor(1j * 3 * 100.0 ** (-2 / 6)))
  torch.testing.assert_close(torch.complex(y[3, 1, 2], y[3, 1, 3]), z.to(torch.complex128), rtol=1e-6, atol=1e-6)


def test_oracle_routing_and_softplus():
  h, router = torch.tensor([[1.0, 0.0]]), torch.tensor([[0.5, 0.0], [2.0, 1.0], [1.0, 3.0]])
  idx, w = R.route(h, router, 2)
  assert idx.tolist() == [[1, 2]]
  torch.testing.assert_close(w, torch.softmax(torch.tensor([[2.0, 1.0]]), -1))
  z = torch.linspace(-30, 30, 61)
  torch.testing.assert_close(R.softplus(z), torch.nn.functional.softplus(z, threshold=100))


def test_oracle_is_causal_and_reads_the_shift():
  d = C.CONFIGS["mixed"]
  w = C.random_weights(d, 3)
  toks = C.tokens(d, 16, 4)
  a = R.forward(d, w, toks, torch.float64)
  other = list(toks)
  other[9] = (other[9] + 1) % d["vocab"]
  b = R.forward(d, w, other, torch.float64)
  assert torch.allclose(a[:9], b[:9], atol=1e-6) and not torch.allclose(a[9:], b[9:], atol=1e-3)
  assert torch.allclose(a[:6], R.forward(d, w, toks[:6], torch.float64), atol=1e-8)
