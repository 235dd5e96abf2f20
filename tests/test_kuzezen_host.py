"""Kuzezen without a GPU: reading a configuration, the registry, and the plain implementation's mechanisms against
closed forms."""
import json
import math

import pytest
import torch

from oracle import kuzezen_ref as R
from tests import kuzezen_cases as C
from tunix_amd import config, dummy_model, registry


@pytest.mark.parametrize("name", sorted(C.CONFIGS))
def test_config_reader_names_every_tensor(name):
  d = C.CONFIGS[name]
  cfg = config.kuzezen_from_dict(d)
  assert cfg.weight_shapes() == R.tensor_shapes(d)
  assert (cfg.norm_eps, cfg.input_conv, cfg.embed_scale) == (d["norm"]["eps"], d["canon"]["taps"], d["embedding"]["scale"])
  assert (cfg.residual_mult, cfg.logit_softcap, cfg.tied_head) == (d["residual_mult"], d["logit_softcap"], False)
  assert [(i, b) for i, b in cfg.layer_runs] == [(i, t is not None) for i, t in R.running_order(d)]
  for ly, src in zip(cfg.layers, d["layers"]):
    a, b = src["mixer"]["left"], src["mixer"]["right"]
    assert all(getattr(ly.mixer.left, k) == a[k] for k in ("heads", "kv_heads", "dim", "vdim", "conv", "scale"))
    assert (ly.mixer.left.temp_coef, ly.mixer.left.temp_every) == (a["q_temp"]["coef"], a["q_temp"]["every"])
    assert all(getattr(ly.mixer.right, k) == b[k] for k in ("heads", "dim", "vdim", "gate_cap"))
    assert (ly.mlp is None) == (src["mlp"] is None) and (ly.mlp is None or ly.mlp.ff == src["mlp"]["ff"])


@pytest.mark.parametrize("change", [
    lambda d: d["layers"][0].update(type="attention"),
    lambda d: d["layers"][0]["mlp"].update(kind="moe"),
    lambda d: d["layers"][0]["mixer"]["left"].update(kv_heads=4),
    lambda d: d["layers"][0]["mixer"]["left"].update(conv=0),
    lambda d: d["layers"][0]["mixer"]["left"]["q_temp"].update(every=0),
    lambda d: d["layers"][0]["mixer"]["right"].update(gate_cap=0.0),
    lambda d: d["canon"].update(taps=0),
    lambda d: d["loop"].update(stop=4),
])
def test_config_reader_rejects_what_the_design_does_not_have(change):
  d = json.loads(json.dumps(C.CONFIGS["mixed"]))
  change(d)
  with pytest.raises(ValueError):
    config.kuzezen_from_dict(d)


def test_parallel_layers_do_not_mix_with_others():
  par = config.kuzezen_from_dict(C.CONFIGS["heads"])
  attn = config.LayerSpec(config.AttentionMixer(2, 1, 8, 8, 0, 1.0, 1.0), None)
  with pytest.raises(ValueError, match="parallel"):
    config.StackConfig("x", 8, 8, (par.layers[0], attn), 1e-6, norm_offset=0.0, parallel=True, input_conv=2)
  with pytest.raises(ValueError, match="parallel"):
    config.StackConfig("x", 8, 8, (attn, par.layers[0]), 1e-6)
  with pytest.raises(ValueError, match="loop"):
    config.StackConfig("x", 8, 8, par.layers, 1e-6, loop=config.LayerLoop(0, 1, 2), norm_offset=0.0, parallel=True, input_conv=2)


def test_registry_and_benchmark_shapes(tmp_path):
  C.write_model(tmp_path, "odd", seed=1)
  arch, cfg = registry.read_config(str(tmp_path))
  assert isinstance(cfg, config.StackConfig) and cfg.family == "kuzezen" and torch.float32 in arch.dtypes
  for c in (cfg, config.kuzezen_shape(256, 4, 2, 128, vocab=64)):
    w = dummy_model.create_stack_weights(c, 3)
    assert {k: tuple(t.shape) for k, t in w.items()} == c.weight_shapes()
    assert all(abs(float(t.float().mean()) - 1.0) < 0.3 for n, t in w.items() if n.endswith((".norm", ".norm1", ".out")))


# ---- the plain implementation -------------------------------------------------------------------
def test_oracle_convolution_carries_over_a_cut():
  g = torch.Generator().manual_seed(1)
  x, taps = torch.randn(9, 4, generator=g), torch.randn(4, 3, generator=g)
  y = R.causal_conv(x, taps)
  torch.testing.assert_close(y[0], taps[:, 2] * x[0])
  torch.testing.assert_close(y[4], taps[:, 2] * x[4] + taps[:, 1] * x[3] + taps[:, 0] * x[2])
  torch.testing.assert_close(torch.cat([R.causal_conv(x[:4], taps), R.causal_conv(x[4:], taps, x[2:4])]), y)


def test_oracle_query_temperature_steps():
  t = R.query_temperature(torch.arange(9), 0.5, 4)
  want = [1.0] * 3 + [1 + 0.5 * math.log(2)] * 4 + [1 + 0.5 * math.log(3)] * 2
  torch.testing.assert_close(t, torch.tensor(want, dtype=torch.float64))


def test_oracle_mixture_of_heads():
  """The identity is plain attention; a permutation gives a head another one's weights on its own values."""
  g = torch.Generator().manual_seed(2)
  q, k, v = torch.randn(5, 4, 3, generator=g), torch.randn(5, 2, 3, generator=g), torch.randn(5, 2, 6, generator=g)
  plain = R.mixed_attention(q, k, v, 0.7, torch.eye(4))
  for h in range(4):
    s = (q[:, h] @ k[:, h // 2].T * 0.7).masked_fill(torch.triu(torch.ones(5, 5, dtype=torch.bool), 1), -math.inf)
    torch.testing.assert_close(plain[:, h], torch.softmax(s, -1) @ v[:, h // 2])
  perm = torch.tensor([2, 0, 3, 1])
  moved = R.mixed_attention(q, k, v, 0.7, torch.eye(4)[perm])
  other = R.mixed_attention(q, k, v.flip(1), 0.7, torch.eye(4))
  torch.testing.assert_close(moved[:, 0], other[:, 2])   # head 2's weights on the values of head 0
  torch.testing.assert_close(moved[:, 1], plain[:, 0])


def test_oracle_memory_equals_the_weighted_sum():
  g = torch.Generator().manual_seed(0)
  T, H, n, m = 8, 2, 3, 4
  q, k, v = (torch.randn(T, H, s, generator=g, dtype=torch.float64) for s in (n, n, m))
  li, lf = 3 * torch.randn(T, H, generator=g, dtype=torch.float64), R.log_sigmoid(torch.randn(T, H, generator=g, dtype=torch.float64))
  y, end = R.matrix_memory(q, k, v, li, lf)
  for t in range(T):
    for h in range(H):
      w = [float(li[j, h] + lf[j + 1:t + 1, h].sum()) for j in range(t + 1)]
      top = max([float(lf[:t + 1, h].sum())] + w)          # (the maximum begins at zero)
      dots = [math.exp(x - top) * float(q[t, h] @ k[j, h]) for j, x in enumerate(w)]
      den = max(abs(sum(dots)), math.exp(-top)) + 1e-6
      torch.testing.assert_close(y[t, h], sum(d * v[j, h] for j, d in enumerate(dots)) / den)
  a, mid = R.matrix_memory(q[:3], k[:3], v[:3], li[:3], lf[:3])
  b, last = R.matrix_memory(q[3:], k[3:], v[3:], li[3:], lf[3:], mid)
  torch.testing.assert_close(torch.cat([a, b]), y)
  for x, z in zip(last, end):
    torch.testing.assert_close(x, z)


def test_oracle_gates():
  z = torch.linspace(-40, 40, 81, dtype=torch.float64)
  torch.testing.assert_close(R.log_sigmoid(z), torch.nn.functional.logsigmoid(z))
  torch.testing.assert_close(R.soft_cap(z, 3.0), 3.0 * torch.tanh(z / 3.0))


def test_oracle_is_causal():
  d = C.CONFIGS["mixed"]
  w = C.random_weights(d, 3)
  toks = C.tokens(d, 16, 4)
  a = R.forward(d, w, toks, torch.float64)
  other = list(toks)
  other[9] = (other[9] + 1) % d["vocab"]
  b = R.forward(d, w, other, torch.float64)
  assert torch.allclose(a[:9], b[:9], atol=1e-6) and not torch.allclose(a[9:], b[9:], atol=1e-3)
  assert torch.allclose(a[:6], R.forward(d, w, toks[:6], torch.float64), atol=1e-8)
