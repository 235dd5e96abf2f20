"""Kezolix without a GPU: reading a configuration, the registry, borrowed cache entries, and the plain implementation's
mechanisms against closed forms."""
import json
import math

import pytest
import torch

from oracle import kezolix_ref as R
from tests import kezolix_cases as C
from tunix_amd import config, dummy_model, registry
from tunix_amd.cache import BorrowedSpec, KVSpec, SequenceCache, StateSpec
from tunix_amd.generate.utils import check_positions


@pytest.mark.parametrize("name", sorted(C.CONFIGS))
def test_config_reader_names_every_tensor(name):
  d = C.CONFIGS[name]
  cfg = config.kezolix_from_dict(d)
  assert cfg.weight_shapes() == R.tensor_shapes(d)
  assert (cfg.norm_eps, cfg.residual_mult, cfg.max_positions, cfg.tied_head) == (d["norm"]["eps"], d["residual_mult"], d["max_positions"], False)
  for ly, src in zip(cfg.layers, d["layers"]):
    m, mlp = src["mixer"], src["mlp"]
    assert all(getattr(ly.mixer, k) == m[k] for k in ("heads", "dim", "vdim"))
    if src["type"] == "attention":
      assert (ly.mixer.kv_heads, ly.mixer.scale, ly.mixer.chunk, ly.mixer.kv_from) == (m["kv_heads"], m["scale"], m["mask"]["size"], m.get("kv_from"))
      assert list(ly.mixer.slopes) == R.slopes(m["heads"])
    if mlp is None:
      assert ly.mlp is None
    elif mlp["kind"] == "dense":
      assert ly.mlp == config.PolyNormMlp(mlp["ff"])
    else:
      r = mlp["router"]
      assert (ly.mlp.ff, ly.mlp.experts, ly.mlp.top, ly.mlp.scale, ly.mlp.shared_ff) == (mlp["expert"]["ff"], r["experts"], r["top"], r["scale"], mlp["shared"]["ff"])


@pytest.mark.parametrize("change", [
    lambda d: d["layers"][0].update(type="lightning"),
    lambda d: d["layers"][0]["mlp"].update(kind="gated"),
    lambda d: d["layers"][1]["mixer"].update(kv_heads=4),
    lambda d: d["layers"][1]["mixer"]["mask"].update(size=0),
    lambda d: d["layers"][1]["mlp"]["router"].update(top=10),
    lambda d: d["layers"][4]["mixer"].update(kv_from=0),      # a recurrent layer
    lambda d: d["layers"][5]["mixer"].update(kv_from=4),      # a layer that borrows itself
    lambda d: d["layers"][1]["mixer"].update(kv_from=3),      # a later layer
    lambda d: d["layers"][4]["mixer"].update(vdim=40),
])
def test_config_reader_rejects_what_the_design_does_not_have(change):
  d = json.loads(json.dumps(C.CONFIGS["mixed"]))
  change(d)
  with pytest.raises(ValueError):
    config.kezolix_from_dict(d)


def test_new_parts_do_not_mix_with_what_they_exclude():
  cfg = config.kezolix_from_dict(C.CONFIGS["one"])
  for kw in (dict(loop=config.LayerLoop(0, 1, 2)), dict(embed_norm=True), dict(norm_groups=2), dict(pre_norm=False)):
    with pytest.raises(ValueError, match="depth average"):
      config.StackConfig("x", 8, 8, cfg.layers, 1e-6, depth_average=True, **kw)
  with pytest.raises(ValueError, match="borrow"):
    config.AttentionMixer(2, 1, 8, 8, 0, 1.0, 1.0, kv_from=0)
  with pytest.raises(ValueError, match="slopes"):
    config.AttentionMixer(2, 1, 8, 8, 0, 1.0, 1.0, slopes=(0.5,))
  with pytest.raises(ValueError, match="shared"):
    config.ExpertsMlp(8, 4, 2, shared_ff=8)


def test_a_shared_expert_among_the_others():
  """As large as others together it is as many routes of a token; otherwise it runs apart."""
  make = lambda ff, shared: config.ExpertsMlp(ff, 8, 2, gated=False, corrected=True, shared_ff=shared)
  assert [make(*a).routes for a in ((16, 16), (16, 48), (16, 24), (16, 8), (16, 0), (16, 80))] == [3, 5, 2, 2, 2, 2]


def test_registry_and_benchmark_shapes(tmp_path):
  C.write_model(tmp_path, "odd", seed=1)
  arch, cfg = registry.read_config(str(tmp_path))
  assert isinstance(cfg, config.StackConfig) and cfg.family == "kezolix" and torch.float32 in arch.dtypes
  for c in (cfg, config.kezolix_shape(256, 4, 2, 128, 8, 2, 48, vocab=64)):
    w = dummy_model.create_stack_weights(c, 3)
    assert {k: tuple(t.shape) for k, t in w.items()} == c.weight_shapes()
    assert all(0.0 <= float(t.min()) and float(t.max()) <= 1.0 for n, t in w.items() if n.endswith(".lower"))
    assert all(abs(float(t.float().mean()) - 1.0) < 0.3 for n, t in w.items() if "norm" in n)


def test_borrowed_entries():
  """A borrowed entry is the lender's, through views and growth; in a scratch cache nobody overwrites what is lent."""
  kv, st = KVSpec(2, 8, 4, torch.float32), StateSpec(1, 2, 3)
  specs = [kv, kv, st, BorrowedSpec(0), kv, st, BorrowedSpec(0)]
  for shared in (False, True):
    c = SequenceCache(specs, 3, 5, "cpu", shared=shared)
    assert c.entries[3] is c.entries[0] and c.entries[6] is c.entries[0]
    assert c.entries[1] is not c.entries[0] and c.entries[4] is not c.entries[0]
    assert (c.entries[4] is c.entries[1]) == shared and (c.entries[5] is c.entries[2]) == shared
    c.entries[0].k[1, 0, 4] = 7.0
    assert float(c.rows(1, 1).entries[6].k[0, 0, 4, 0]) == 7.0
    c.grow(9)
    assert c.entries[3].k.shape[2] == 9 and c.entries[6] is c.entries[0] and float(c.entries[0].k[1, 0, 4, 0]) == 7.0


def test_positions_are_bounded():
  class Model:
    cfg = config.kezolix_from_dict(C.CONFIGS["one"])
  check_positions(Model, 64)
  with pytest.raises(ValueError, match="64 positions"):
    check_positions(Model, 65)


# ---- the plain implementation -------------------------------------------------------------------
def test_oracle_norms():
  g = torch.Generator().manual_seed(1)
  x, w = torch.randn(4, 10, generator=g) + 3.0, torch.randn(10, generator=g)
  torch.testing.assert_close(R.layer_norm(x, w, 0.1), torch.nn.functional.layer_norm(x, (10,), w, None, 0.1))
  z = torch.tensor([[1.0, -2.0, 0.5]])
  want = 2 * z / math.sqrt(5.25 / 3) - z ** 2 / math.sqrt(17.0625 / 3) + 3 * z ** 3 / math.sqrt((1 + 64 + 0.5 ** 6) / 3) + 0.25
  torch.testing.assert_close(R.poly_norm(z, torch.tensor([2.0, -1.0, 3.0, 0.25]), 0.0), want)


def test_oracle_chunks_and_slopes():
  assert R.slopes(4) == [0.25, 0.0625, 0.015625, 0.00390625]
  assert [[R.visible(i, j, 3) for j in range(5)] for i in (2, 3, 4)] == [[True] * 3 + [False] * 2, [False] * 3 + [True, False], [False] * 3 + [True] * 2]
  g = torch.Generator().manual_seed(2)
  q, k, v = torch.randn(7, 2, 3, generator=g), torch.randn(7, 1, 3, generator=g), torch.randn(7, 1, 5, generator=g)
  o = R.biased_attention(q, k, v, 0.6, 4)
  torch.testing.assert_close(o[4], v[4].expand(2, -1))                       # alone in its chunk
  s = torch.tensor([float(q[6, 1] @ k[j, 0]) * 0.6 - 2.0 ** -8 * (6 - j) for j in (4, 5, 6)])
  torch.testing.assert_close(o[6, 1], torch.softmax(s, 0) @ v[4:7, 0])


def test_oracle_recurrence_equals_the_weighted_sum():
  g = torch.Generator().manual_seed(0)
  T, H, n, m = 8, 2, 3, 4
  q, v = (torch.randn(T, H, s, generator=g, dtype=torch.float64) for s in (n, m))
  f = R.forget_gate(torch.randn(T, H, n, generator=g, dtype=torch.float64), torch.rand(H, n, generator=g, dtype=torch.float64))
  y, end = R.gated_recurrence(q, f, v)
  for t in range(T):
    for h in range(H):
      want = sum(float((q[t, h] * (1 - f[j, h]) * f[j + 1:t + 1, h].prod(0)).sum()) * v[j, h] for j in range(t + 1))
      torch.testing.assert_close(y[t, h], want)
  a, mid = R.gated_recurrence(q[:3], f[:3], v[:3])
  b, last = R.gated_recurrence(q[3:], f[3:], v[3:], mid)
  torch.testing.assert_close(torch.cat([a, b]), y)
  torch.testing.assert_close(last, end)
  torch.testing.assert_close(R.forget_gate(torch.tensor([-50.0, 0.0, 50.0]), torch.tensor(0.2)), torch.tensor([0.2, 0.6, 1.0]))


def test_oracle_router():
  z, c = torch.tensor([[0.0, 2.0, 1.0, -1.0]]), torch.tensor([0.9, 0.0, 0.0, -0.5])
  s = torch.softmax(z, -1)[0]
  ids, w = R.route(z, c, 2, 3.0)
  assert ids.tolist() == [[0, 1]]                                            # the correction lifts expert 0, and stays out of the weights
  torch.testing.assert_close(w[0], 3.0 * s[:2] / (s[0] + s[1]))
  assert R.route(z, torch.zeros(4), 2, 1.0)[0].tolist() == [[1, 2]]


def test_oracle_is_causal():
  d = C.CONFIGS["mixed"]
  w = C.random_weights(d, 3)
  toks = C.tokens(d, 26, 4)
  a = R.forward(d, w, toks, torch.float64)
  other = list(toks)
  other[9] = (other[9] + 1) % d["vocab"]
  b = R.forward(d, w, other, torch.float64)
  assert torch.allclose(a[:9], b[:9], atol=1e-6) and not torch.allclose(a[9:], b[9:], atol=1e-3)
  assert torch.allclose(a[:6], R.forward(d, w, toks[:6], torch.float64), atol=1e-8)
