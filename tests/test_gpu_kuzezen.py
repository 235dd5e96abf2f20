"""Kuzezen on the GPU against the plain implementation (oracle/kuzezen_ref.py): every mechanism alone, then whole
models -- prompts, token-by-token decoding, portions, unequal batches, reused slots, greedy generation -- in bf16
and in fp32, at sizes that reach every kernel."""
import json
import math
import os
import subprocess
import sys

import numpy as np
import pytest
import torch

from oracle import kuzezen_ref as R
from tests import kuzezen_cases as C
from tests.test_gpu_lapevik import source
from tests.test_gpu_nunezen import BF, DTYPES, F32, all_logits, err, i32, rel, rnd, unfrag
from tunix_amd import _lib as L
from tunix_amd import config, ops
from tunix_amd.generate import CacheConfig, Sampler
from tunix_amd.generate.replay import Replay
from tunix_amd.generate.utils import IdTokenizer
from tunix_amd.rl.rollout import HipRollout, RolloutConfig
from tunix_amd.stack_model import StackModel

pytestmark = pytest.mark.gpu
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))


def up(n, m):
  return (n + m - 1) // m * m


# ---- embedding, soft cap, head norms ----------------------------------------------------------------
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("D", [52, 128])
def test_embedding_is_scaled(gpu, dtype, D):
  table, ids = rnd(37, D).to(BF).to(dtype), torch.tensor([[3, 36, 0, 9], [5, 5, 1, 2]], dtype=torch.int32)
  x = torch.empty(4, D, device=gpu)
  ops.embed_rows(table.to(gpu), ids.to(gpu), i32([2], gpu), 2, 2, 37, D, x, scale=2.75)
  assert torch.equal(x.cpu(), table[ids[:, 2:].long()].view(4, D).float() * 2.75)


def test_soft_cap(gpu):
  z = torch.cat([rnd(5000, scale=30.0), torch.tensor([0.0, 1e-6, 1e4, -1e4, 3e38])])
  t = z.to(gpu)
  ops.soft_cap(t, 7.5)
  torch.testing.assert_close(t.cpu(), 7.5 * torch.tanh(z / 7.5), rtol=2e-6, atol=1e-9)


@pytest.mark.parametrize("M,V", [(1, 320), (20, 304), (130, 1024)])
def test_soft_capped_head(gpu, M, V):
  """Logits and statistics of the statistics head: through its many-row kernel, through its own (fp32 logits)."""
  D, cap = 128, 6.0
  x, w = rnd(M, D, seed=1).to(BF), rnd(V, D, seed=2).to(BF)
  want = R.soft_cap(x.double() @ w.double().T, cap)
  we = ops.dense_expand(w.to(gpu))
  xg, wg, tg = x.to(gpu), w.to(gpu), torch.arange(M, dtype=torch.int32, device=gpu)
  for fp32 in (0, 1):
    out, lse, best, tl = (torch.empty(n, dtype=t, device=gpu) for n, t in (((M, V), F32), (M, F32), (M, torch.int32), (M, F32)))
    part = torch.empty(M * ops.lmhead_nblocks(V) * 4, device=gpu)
    d = L.LmHeadDesc()
    d.M, d.D, d.V, d.x, d.w_bf16, d.w_expanded, d.temperature, d.softcap, d.logits_fp32 = M, D, V, xg.data_ptr(), wg.data_ptr(), we.data_ptr(), 1.0, cap, fp32
    d.part, d.logits_out, d.lse, d.best_id, d.targets, d.target_logp = part.data_ptr(), out.data_ptr(), lse.data_ptr(), best.data_ptr(), tg.data_ptr(), tl.data_ptr()
    ops.lmhead(d)
    tol = 1e-5 if fp32 else 2e-2
    assert float((out.cpu() - want).abs().max()) < tol
    assert float((lse.cpu() - torch.logsumexp(want, -1)).abs().max()) < tol
    rows = torch.arange(M)
    assert float((want.max(-1).values - want[rows, best.cpu().long()]).max()) < 2 * tol
    assert float((tl.cpu() - torch.log_softmax(want, -1)[rows, rows]).abs().max()) < 2 * tol


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("W,groups,split", [(70, 5, 1), (256, 2, 1), (4096, 32, 2), (72, 9, 3), (2048, 1, 1), (9000, 3, 1)])
def test_norms_of_heads_and_gate(gpu, dtype, W, groups, split):
  M, eps = 5, 0.3
  o, w, g = rnd(M, W, seed=1), rnd(W, seed=2), rnd(M, W + 16, seed=3).to(dtype).float()
  src, keep = source(g, dtype, gpu, split)
  og, wg = o.to(gpu), w.to(gpu)
  want = R.rms(o.view(M, groups, -1), eps).view(M, W) * w * torch.sigmoid(g[:, 16:])
  for fr in ([False, True] if dtype == BF else [False]):
    out = torch.zeros(128, up(W, 128), dtype=dtype, device=gpu)
    d = L.GatedNormDesc()
    d.M, d.W, d.dtype, d.eps, d.groups = M, W, ops.DTYPES[dtype], eps, groups
    d.o, d.o_ld, d.g, d.g_off, d.w = og.data_ptr(), W, src, 16, wg.data_ptr()
    d.out, d.out_ld, d.out_frag = out.data_ptr(), out.shape[1], int(fr)
    ops.gated_norm(d)
    assert rel((unfrag(out, M) if fr else out[:M])[:, :W], want) < (2e-6 if dtype == F32 else 4e-3)


# ---- residual + norm + input convolutions --------------------------------------------------------------
class Step:
  """The step over a batch of sequences whose columns come in portions."""

  def __init__(self, gpu, dtype, D, taps, starts, S, n_in=3, conv=True, add=True, seed=0):
    self.gpu, self.dtype, self.D, self.taps, self.S, self.starts, self.B, self.n_in = gpu, dtype, D, taps, S, list(starts), len(starts), n_in
    B, self.eps, self.mult, self.scales = self.B, 0.05, 0.6, [0.5, 0.5, 1.0]
    self.x = rnd(B, S, D, seed=seed + 1)
    self.y = [rnd(B, S, D, seed=seed + 2 + p, scale=2.0).to(BF).float() for p in range(n_in)]
    self.wp = [rnd(D, seed=seed + 8 + p) if p != 2 else None for p in range(n_in)]
    self.wn, self.add = rnd(D, seed=seed + 5), rnd(D, seed=seed + 6) if add else None
    self.conv = [rnd(D, taps, seed=seed + 20 + i) for i in range(2)] if conv else None
    self.slots = max(taps - 1, 1)
    self.ring = torch.full((B, self.slots, D), 9.0, device=gpu)     # another sequence's rows

  def run(self, col, T, split=1, fr=False):
    gpu, B, D, M = self.gpu, self.B, self.D, self.B * T
    dev = lambda t: t.to(gpu).contiguous()
    cut = lambda t: t[:, col:col + T].reshape(M, D)
    x, x2 = dev(cut(self.x)), torch.full((M, D), float("nan"), device=gpu)
    outs = [torch.zeros(up(M, 128), up(D, 128), dtype=self.dtype, device=gpu) for _ in range(2)]
    keep, d = [x, x2, outs], L.ParallelStepDesc()
    d.M, d.D, d.dtype, d.eps, d.mult, d.n_in, d.B, d.T = M, D, ops.DTYPES[self.dtype], self.eps, self.mult, self.n_in, B, T
    for p in range(self.n_in):
      s, k = source(cut(self.y[p]), self.dtype, gpu, split)
      d.y[p], d.y_scale[p] = s, self.scales[p]
      keep.append(k)
      if self.wp[p] is not None:
        keep.append(dev(self.wp[p]))
        d.w_post[p] = keep[-1].data_ptr()
    for n, t in (("w_next", self.wn), ("add", self.add)):
      if t is not None:
        keep.append(dev(t))
        setattr(d, n, keep[-1].data_ptr())
    st, cp = i32(self.starts, gpu), i32([col], gpu)
    moved = self.n_in > 0 or self.add is not None
    d.x, d.x_out = x.data_ptr(), (x2 if T > 1 else x).data_ptr() if moved else None
    d.out1, d.out_ld, d.out_frag = outs[0].data_ptr(), outs[0].shape[1], int(fr)
    n_tail = min(T, self.slots)
    tail = torch.zeros(B * n_tail, D, device=gpu)
    if self.conv is not None:
      keep += [dev(c.T) for c in self.conv]
      d.conv1, d.conv2, d.out2, d.taps, d.slots = keep[-2].data_ptr(), keep[-1].data_ptr(), outs[1].data_ptr(), self.taps, self.slots
      d.ring, d.tail, d.starts, d.col_ptr = self.ring.data_ptr(), tail.data_ptr(), st.data_ptr(), cp.data_ptr()
    ops.parallel_step(d)
    if self.conv is not None and T > 1 and self.taps > 1:
      ops.ring_write(ops.rows_src(y=tail, ld=D), 0, B, n_tail, cp, self.ring, t0=T - n_tail)
    torch.cuda.synchronize()
    get = lambda o: (unfrag(o, M) if fr else o[:M])[:, :D].float().cpu().view(B, T, D)
    return (x2 if moved and T > 1 else x).cpu().view(B, T, D), get(outs[0]), get(outs[1])

  def check(self, got, col):
    x, o1, o2 = got
    T, tol = x.shape[1], 2e-6 if self.dtype == F32 else 4e-3
    for b, s in enumerate(self.starts):
      new = self.x[b].clone()
      for p in range(self.n_in):
        new = new + self.mult * self.scales[p] * (self.y[p][b] if self.wp[p] is None else R.rms(self.y[p][b], self.eps) * self.wp[p])
      if self.add is not None:
        new = new + self.add
      assert rel(x[b], new[col:col + T]) < 2e-6
      lo = max(s, col)
      if lo >= col + T:
        continue
      h = R.rms(new[s:], self.eps) * self.wn
      for got_o, i in ((o1, 0), (o2, 1)):
        if self.conv is None and i:
          continue
        want = h if self.conv is None else h + R.causal_conv(h, self.conv[i])
        assert rel(got_o[b, lo - col:], want[lo - s:col + T - s]) < tol, (b, i, col, T)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("D,taps", [(96, 3), (100, 5), (128, 1), (2048, 4), (2304, 2), (60, 4), (4104, 3), (128, 7)])
def test_parallel_step_in_portions(gpu, dtype, D, taps):
  """A prompt at once, then in portions from two tokens up and single tokens, over rows of which one begins inside a
  portion, one with it and one late; finished rows and partial planes, fragment order."""
  a = Step(gpu, dtype, D, taps, [0, 5, 31, 2], 40, seed=D)
  a.check(a.run(0, 40), 0)
  a.ring.fill_(-7.0)
  col = 0
  for T in (2, 3, 1, 2, 17, 1, 1, 1, 5, 1, 6):
    split = 3 if dtype == BF and T in (1, 3) else 1
    a.check(a.run(col, T, split=split, fr=dtype == BF and T != 17), col)
    col += T
  assert col == 40


@pytest.mark.parametrize("dtype", DTYPES)
def test_parallel_step_forms(gpu, dtype):
  """Nothing incoming, no vector, one or two incoming rows, no convolution; many rows (several tokens per work-group)."""
  for n_in, add, conv in ((0, False, True), (0, True, True), (2, False, True), (1, True, False), (3, True, False), (0, False, False)):
    for D in (104, 52):
      a = Step(gpu, dtype, D, 3, [0, 4], 12, n_in=n_in, add=add, conv=conv, seed=n_in)
      for col, T in ((0, 7), (7, 1), (8, 4)):
        a.check(a.run(col, T), col)
  a = Step(gpu, dtype, 64, 4, [0, 700, 1399], 1400, seed=3)
  a.check(a.run(0, 1400), 0)


# ---- convolution + cache write -------------------------------------------------------------------------
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,G,dk,dv,taps", [(6, 2, 32, 48, 3), (4, 4, 64, 24, 2), (3, 3, 21, 13, 5), (10, 5, 12, 45, 1), (4, 1, 200, 136, 4), (2, 2, 8, 8, 1), (2, 1, 16, 264, 6)])
def test_convolution_temperature_value_norm(gpu, dtype, H, G, dk, dv, taps):
  """q, keys and values of a prompt, of portions from two tokens up and of single tokens; a portion's first tokens read
  the ring, a sequence's first ones zeros; a temperature that steps at every third position."""
  S, starts, coef, every, eps = 60, [0, 7, 33, 20], 0.4, 3.0, 0.02
  B = len(starts)
  offs = [0, up(H * dk, 16), up(H * dk, 16) + up(G * dk, 16)]
  Cn, code = offs[2] + up(G * dv, 16), ops.DTYPES[dtype]
  u = torch.zeros(B, S, 16 + Cn)
  w = torch.zeros(taps, Cn)
  for o, n in zip(offs, (H * dk, G * dk, G * dv)):
    u[:, :, 16 + o:16 + o + n] = rnd(B, S, n, seed=o).to(BF).float()
    w[:, o:o + n] = rnd(taps, n, seed=o + 1)
  dkp, dvp = ops.sink_attn_pad(dk, True, dtype), ops.sink_attn_pad(dv, True, dtype)
  wg, st = w.to(gpu), i32(starts, gpu)
  want = []
  for b, s in enumerate(starts):
    c = [R.causal_conv(u[b, s:, 16 + o:16 + o + n], w[:, o:o + n].T) for o, n in zip(offs, (H * dk, G * dk, G * dv))]
    temp = R.query_temperature(torch.arange(S - s), coef, every).float()[:, None, None]
    want.append((c[0].view(-1, H, dk) * temp, c[1].view(-1, G, dk), R.rms(c[2].view(-1, G, dv), eps)))
  for portions in ((60,), (2, 3, 1, 2, 1, 1, 17, 1, 32)):
    ring = torch.full((B, taps, Cn), 5.0, dtype=dtype, device=gpu)
    k, v = (torch.full((B, G, S, n), 3.0, dtype=dtype, device=gpu) for n in (dkp, dvp))
    col = 0
    for T in portions:
      src, keep = source(u[:, col:col + T].reshape(B * T, -1), dtype, gpu, 2 if dtype == BF and T in (1, 2) else 1)
      q, cp = torch.full((B * T, H, dkp), float("nan"), dtype=dtype, device=gpu), i32([col], gpu)
      d = L.ConvKvDesc()
      d.B, d.T, d.S, d.H, d.G, d.dk, d.dv, d.dkp, d.dvp, d.taps, d.slots, d.dtype = B, T, S, H, G, dk, dv, dkp, dvp, taps, taps, code
      d.temp_coef, d.temp_every, d.eps, d.value_norm, d.y, d.off, d.C = coef, every, eps, 1, src, 16, Cn
      d.q_off, d.k_off, d.v_off, d.w, d.ring = *offs, wg.data_ptr(), ring.data_ptr()
      d.starts, d.col_ptr, d.q_out, d.kcache, d.vcache = st.data_ptr(), cp.data_ptr(), q.data_ptr(), k.data_ptr(), v.data_ptr()
      ops.conv_kvwrite(d)
      if T > 1:
        ops.ring_write(src, 16, B, T, cp, ring)
      q = q.view(B, T, H, dkp).float().cpu()
      for b, s in enumerate(starts):
        lo = max(s, col)
        if lo < col + T:
          assert rel(q[b, lo - col:, :, :dk], want[b][0][lo - s:col + T - s]) < (2e-6 if dtype == F32 else 5e-3), (b, col)
          assert not q[b, lo - col:, :, dk:].any()
      col += T
    for b, s in enumerate(starts):
      for cache, n, i in ((k, dk, 1), (v, dv, 2)):
        got = cache[b].transpose(0, 1).float().cpu()[s:]
        assert rel(got[..., :n], want[b][i]) < (2e-6 if dtype == F32 else 5e-3) and not got[..., n:].any()


# ---- attention with mixed heads ---------------------------------------------------------------------------
class Mixed:
  def __init__(self, gpu, dtype, H, G, dk, dv, S, starts, seed=0, sharp=2.0, talk=None, scale=None):
    self.gpu, self.dtype, self.H, self.G, self.dk, self.dv, self.S, self.starts, self.B = gpu, dtype, H, G, dk, dv, S, list(starts), len(starts)
    self.dkp, self.dvp = ops.sink_attn_pad(dk, True, dtype), ops.sink_attn_pad(dv, True, dtype)
    r = lambda n, d, s: rnd(self.B, S, n, d, seed=seed + s).to(BF).float()
    self.q, self.k, self.v = r(H, dk, 1) * sharp, r(G, dk, 2), r(G, dv, 3)
    self.q = self.q.to(BF).float()
    self.g = rnd(self.B, S, 16 + H * dv, seed=seed + 4).to(BF).float()
    self.talk = (torch.eye(H) + 0.6 * H ** -0.5 * rnd(H, H, seed=seed + 5)).to(BF).float() if talk is None else talk
    self.scale = dk ** -0.5 if scale is None else scale
    self.lay_out()

  def lay_out(self):
    """q, k and v as the kernels read them: heads padded with zeros, one slab per kv head."""
    pad = lambda t, n: torch.nn.functional.pad(t, (0, n - t.shape[-1])).to(self.dtype)
    slab = lambda t, n: pad(t, n).transpose(1, 2).contiguous().to(self.gpu)
    self.qp, self.kc, self.vc = pad(self.q, self.dkp), slab(self.k, self.dkp), slab(self.v, self.dvp)

  def run(self, col, T, chunk=64, split=1, gated=True, fr=False):
    gpu, B, H = self.gpu, self.B, self.H
    assert self.qp.shape == (B, self.S, H, self.dkp) and col + T <= self.S
    assert self.kc.shape == (B, self.G, self.S, self.dkp) and self.vc.shape == (B, self.G, self.S, self.dvp)
    q = self.qp[:, col:col + T].contiguous().to(gpu)
    out = torch.zeros(up(B * T, 128), up(H * self.dv, 128), dtype=self.dtype, device=gpu)
    st, cp, talk = i32(self.starts, gpu), i32([col], gpu), self.talk.to(gpu)
    ws = torch.empty(max(1, ops.mixed_attn_ws_bytes(B, T, self.S, H, self.dvp, chunk) // 4), device=gpu)
    d = L.MixedAttnDesc()
    d.B, d.T, d.S, d.H, d.G, d.dk, d.dv, d.dkp, d.dvp = B, T, self.S, H, self.G, self.dk, self.dv, self.dkp, self.dvp
    d.scale, d.dtype, d.q, d.kcache, d.vcache, d.talk = self.scale, ops.DTYPES[self.dtype], q.data_ptr(), self.kc.data_ptr(), self.vc.data_ptr(), talk.data_ptr()
    d.starts, d.col_ptr, d.kv_chunk, d.ws = st.data_ptr(), cp.data_ptr(), chunk, ws.data_ptr()
    keep = None
    if gated:
      src, keep = source(self.g[:, col:col + T].reshape(B * T, -1), self.dtype, gpu, split)
      d.gate, d.g_off = src, 16
    d.out, d.out_ld, d.out_frag = out.data_ptr(), out.shape[1], int(fr)
    ops.mixed_attn(d)
    torch.cuda.synchronize()
    return (unfrag(out, B * T) if fr else out[:B * T])[:, :H * self.dv].float().cpu().view(B, T, H, self.dv)

  def want(self, b):
    if not hasattr(self, "_want"):
      self._want = {}
    if b not in self._want:
      s = self.starts[b]
      self._want[b] = R.mixed_attention(self.q[b, s:], self.k[b, s:], self.v[b, s:], self.scale, self.talk)
    return self._want[b]

  def check(self, got, col, gated=True):
    T = got.shape[1]
    for b, s in enumerate(self.starts):
      lo = max(s, col)
      if lo >= col + T:
        continue
      w = self.want(b)[lo - s:col + T - s]
      if gated:
        w = w * torch.sigmoid(self.g[b, lo:col + T, 16:]).view(w.shape)
      e = float((got[b, lo - col:] - w).abs().max() / w.abs().max())
      assert e < (2e-5 if self.dtype == F32 else 2e-2), (b, col, T, e)


MIXED = [(6, 2, 32, 48), (4, 4, 64, 24), (8, 1, 24, 64), (3, 3, 21, 13), (10, 5, 12, 45), (16, 2, 136, 200), (20, 5, 64, 96), (32, 8, 128, 128), (16, 4, 96, 128),
         (40, 8, 16, 8), (5, 1, 256, 256), (12, 6, 160, 40), (2, 1, 300, 16), (64, 4, 32, 32), (1, 1, 16, 16), (14, 7, 128, 256)]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,G,dk,dv", MIXED)
def test_mixed_attention_prompt_portions_and_steps(gpu, dtype, H, G, dk, dv):
  """Every group of head sizes and counts; rows with different starts; portions from two tokens up at places that are no
  tile's edge; single tokens with key chunks of every length; finished gate rows and partial planes, fragment order."""
  S = 150
  a = Mixed(gpu, dtype, H, G, dk, dv, S, [0, 37, 149], seed=H)
  a.check(a.run(0, S), 0)
  a.check(a.run(0, S, gated=False), 0, gated=False)
  bf = dtype == BF
  for col, T in ((0, 2), (2, 3), (5, 64), (69, 16), (85, 33), (148, 2)):
    a.check(a.run(col, T, split=2 if bf and T < 4 else 1, fr=bf and T < 40), col)
  for i, t in enumerate((0, 1, 37, 63, 64, 65, 127, 128, 149)):
    a.check(a.run(t, 1, chunk=(64, 128, 192, 320)[i % 4], split=2 if bf and i % 2 else 1, fr=bf and i % 3 == 0), t)


@pytest.mark.parametrize("how", ["prompt", "portion", "decoded"])
@pytest.mark.parametrize("far", [0, 15, 16, 31, 32, 63, 64, 127, 128, 255, 256, 319, 320, 398, 399])
def test_one_key_stands_out(gpu, how, far):
  """One key far above all others -- at the edges of tiles and chunks and at both ends of what is visible -- takes the whole
  weight of the heads that ask for it; the key behind the position, higher still, is not seen.  The mixture hands the weight
  on: a head whose own scores are flat gets it from the one that asked, on its own values."""
  S, H, G, n = 460, 6, 3, 32
  talk = torch.zeros(H, H)
  talk[0, 0], talk[1, 0], talk[2, 0], talk[4, 0] = 1.0, -1.0, 2.0, 0.5
  talk[3, 3], talk[5, 0], talk[5, 3] = 1.0, 1.0, -1.0
  a = Mixed(gpu, BF, H, G, n, n, S, [0], seed=far, talk=talk, scale=1.0)
  a.q[:] = 0.0
  a.q[:, :, 0, 0] = 60.0                          # head 0 asks, the others are flat
  a.k[:] = 0.0
  a.k[0, far, 0, 0], a.k[0, 400, 0, 0] = 1.0, 2.0
  a.lay_out()
  got = {"prompt": lambda: a.run(0, S, gated=False)[0, 399], "portion": lambda: a.run(393, 7, gated=False)[0, 6],
         "decoded": lambda: a.run(399, 1, chunk=320, gated=False)[0, 0]}[how]()
  v, mean = a.v[0, far], a.v[0, :400].mean(0)
  want = torch.stack([v[0], -v[0], 2 * v[1], mean[1], 0.5 * v[2], v[2] - mean[2]])
  assert float((got - want).abs().max()) < 2e-2
  if how == "decoded":
    assert float((a.run(399, 1, chunk=64, gated=False)[0, 0] - want).abs().max()) < 2e-2


def test_the_first_tokens(gpu):
  """A sequence's first position attends to itself alone, the second to two: wherever it begins in the batch."""
  for starts in ([0], [31], [32], [33], [95]):
    a = Mixed(gpu, BF, 8, 4, 64, 64, 100, starts, seed=3)
    s = starts[0]
    a.check(a.run(0, 100, gated=False), 0, gated=False)
    first = a.run(s, 1, gated=False)[0, 0]
    want = a.talk.sum(-1)[:, None] * a.v[0, s].repeat_interleave(2, 0)
    assert rel(first, want) < 5e-3
    a.check(a.run(s, 2, gated=False), s, gated=False)


# ---- matrix memory ---------------------------------------------------------------------------------------
class Memory:
  def __init__(self, gpu, dtype, H, dk, dv, S, starts, seed=0, cap=6.0, spread=2.0):
    self.gpu, self.dtype, self.H, self.dk, self.dv, self.S, self.starts, self.B, self.cap = gpu, dtype, H, dk, dv, S, list(starts), len(starts), cap
    r = lambda d, s: rnd(self.B, S, H, d, seed=seed + s).to(BF).float()
    self.q, self.k, self.v = r(dk, 1), r(dk, 2), r(dv, 3)
    self.gi, self.gf = spread * rnd(self.B, S, H, seed=seed + 4), spread * rnd(self.B, S, H, seed=seed + 5)
    self.bi, self.bf = rnd(H, seed=seed + 6), 2.0 + 2.0 * rnd(H, seed=seed + 7)
    self.reset(7.0)

  def reset(self, x):
    """What another sequence has left: a new one must not see it."""
    B, H = self.B, self.H
    self.state, self.sum, self.top = (torch.full(s, x, device=self.gpu) for s in ((B, H, self.dk, self.dv), (B, H, self.dk), (B, H)))

  def run(self, col, T, split=1):
    gpu, B, H, M = self.gpu, self.B, self.H, self.B * T
    ok, ov = up(H * self.dk, 16), 2 * up(H * self.dk, 16)
    y = torch.zeros(B, T, 16 + ov + H * self.dv)
    for t, o, n in ((self.q, 0, H * self.dk), (self.k, ok, H * self.dk), (self.v, ov, H * self.dv)):
      y[:, :, 16 + o:16 + o + n] = t[:, col:col + T].reshape(B, T, n)
    src, keep = source(y.view(M, -1), self.dtype, gpu, split)
    g = torch.zeros(B, T, 16 + H)
    g[:, :, :H], g[:, :, 16:] = self.gi[:, col:col + T], self.gf[:, col:col + T]
    gates, keep2 = source(g.view(M, -1), F32, gpu, split)
    o = torch.full((M, H * self.dv), float("nan"), device=gpu)
    st, cp, bi, bf = i32(self.starts, gpu), i32([col], gpu), self.bi.to(gpu), self.bf.to(gpu)
    ws = torch.empty(max(1, ops.memory_ws_bytes(B, T, H, self.dk, self.dv) // 4), device=gpu)
    d = L.MemoryDesc()
    d.B, d.T, d.H, d.dk, d.dv, d.dtype, d.q_scale, d.cap = B, T, H, self.dk, self.dv, ops.DTYPES[self.dtype], self.dk ** -0.5, self.cap
    d.y, d.q_off, d.k_off, d.v_off, d.gates, d.i_off, d.f_off = src, 16, 16 + ok, 16 + ov, gates, 0, 16
    d.bias_i, d.bias_f, d.starts, d.col_ptr = bi.data_ptr(), bf.data_ptr(), st.data_ptr(), cp.data_ptr()
    d.state, d.sum, d.top, d.o, d.o_ld, d.ws = self.state.data_ptr(), self.sum.data_ptr(), self.top.data_ptr(), o.data_ptr(), o.shape[1], ws.data_ptr()
    ops.memory(d)
    torch.cuda.synchronize()
    return o.cpu().view(B, T, H, self.dv)

  def want(self, b):
    if not hasattr(self, "_want"):
      self._want = {}
    if b not in self._want:
      s = self.starts[b]
      li = R.soft_cap(self.gi[b, s:] + self.bi, self.cap).double()
      lf = R.log_sigmoid(R.soft_cap(self.gf[b, s:] + self.bf, self.cap)).double()
      self._want[b] = R.matrix_memory(self.q[b, s:].double() * self.dk ** -0.5, self.k[b, s:].double(), self.v[b, s:].double(), li, lf)
    return self._want[b]

  def check(self, got, col, tol=None):
    T = got.shape[1]
    tol = tol or (3e-5 if self.dtype == F32 else 2e-3)
    for b, s in enumerate(self.starts):
      lo = max(s, col)
      if lo >= col + T:
        continue
      o, (S, N, m) = self.want(b)
      # (a row is divided by a sum that may nearly vanish: rows against their own size)
      w, x = o[lo - s:col + T - s].float(), got[b, lo - col:]
      e = ((x - w).norm(dim=-1) / w.norm(dim=-1).clamp_min(1e-3)).flatten().sort().values
      assert float(e[int(0.9 * (len(e) - 1))]) < tol and float(e[-1]) < 100 * tol, (b, col, T, float(e[-1]))
      if col + T == self.S:
        assert rel(self.state[b], S) < tol and rel(self.sum[b], N) < tol and float((self.top[b].cpu() - m).abs().max()) < 1e-4


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,dk,dv", [(3, 16, 40), (2, 64, 128), (5, 40, 16), (2, 11, 9), (3, 20, 30), (2, 160, 136), (1, 128, 264), (9, 8, 8), (2, 256, 64), (1, 48, 7)])
def test_memory_prompt_portions_and_steps(gpu, dtype, H, dk, dv):
  """One pass (cut into spans that run in parallel), portions from two tokens up, token by token, over rows with different
  starts; finished rows and partial planes."""
  S = 330
  a = Memory(gpu, dtype, H, dk, dv, S, [0, 70, 129, 329], seed=H)
  a.check(a.run(0, S), 0)
  a.reset(-3.0)
  col = 0
  for T in (64, 2, 3, 63, 2, 130):
    a.check(a.run(col, T, split=2 if dtype == BF and T < 64 else 1), col)
    col += T
  for t in range(col, S):
    a.check(a.run(t, 1, split=2 if dtype == BF and t % 2 else 1), t)
  b = Memory(gpu, dtype, H, dk, dv, 20, [0, 5], seed=9)
  for t in range(20):
    b.check(b.run(t, 1), t)


@pytest.mark.parametrize("how", ["prompt", "portions", "steps"])
@pytest.mark.parametrize("at", [0, 1, 63, 64, 127, 128, 300])
def test_memory_keeps_and_loses(gpu, how, at):
  """One token far back with an open input gate, nothing else admitted: a head that forgets nothing hands its value back
  hundreds of tokens later, one with a slow gate too (the sum of keys forgets at the same pace), one with a fast gate falls
  below its floor and goes silent; before the token there is nothing."""
  S, H, n, cap = 420, 3, 32, 40.0
  a = Memory(gpu, BF, H, n, n, S, [0], seed=at, cap=cap)
  a.bi[:], a.gf[:] = 0.0, 0.0
  a.gi[:] = -200.0                                  # the capped gate: e^-40
  a.gi[0, at] = 3.0
  a.bf[:] = torch.tensor([200.0, 4.6, -3.0])        # forget nothing; one percent; nearly everything
  a.k[:], a.q[:] = 1.0, 1.0
  got = {"prompt": lambda: a.run(0, S), "portions": lambda: torch.cat([a.run(c, T) for c, T in ((0, 2), (2, 198), (200, 64), (264, 156))], 1),
         "steps": lambda: torch.cat([a.run(t, 1) for t in range(S)], 1)}[how]()[0]
  v = a.v[0, at]
  assert rel(got[at], v) < 5e-3 and float(got[:at].abs().max() if at else 0.0) < 1e-6
  assert rel(got[S - 1, 0], v[0]) < 5e-3
  log_f = math.log(1 / (1 + math.exp(-cap * math.tanh(4.6 / cap))))
  m = 3 + (S - 1 - at) * log_f
  want = v[1] if m > 0 else v[1] * min(1.0, n ** 0.5 * math.exp(m) / 1.0)
  assert rel(got[S - 1, 1], want) < 2e-2
  assert float(got[S - 1, 2].abs().max()) < 1e-5
  a.check(got[None], 0, tol=1e-2)


def test_memory_with_extreme_gates(gpu):
  """Gates at both caps in turn: no weight overflows, whatever the order of the maximum and the decays."""
  for dtype in DTYPES:
    a = Memory(gpu, dtype, 4, 16, 32, 200, [0, 11], seed=2, cap=15.0, spread=40.0)
    got = a.run(0, 200)
    assert torch.isfinite(got).all()
    a.check(got, 0)
    a.reset(1.0)
    a.check(torch.cat([a.run(t, 1) for t in range(200)], 1), 0)


# ---- whole models -----------------------------------------------------------------------------------------
def model_of(name, seed, dtype, gpu):
  d = C.CONFIGS[name]
  w = C.random_weights(d, seed)
  return d, w, StackModel(config.kuzezen_from_dict(d), w, gpu, dtype)


TOL = {BF: 0.12, F32: 2e-4}


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", sorted(C.CONFIGS))
def test_prompts_decoding_and_unequal_batches(gpu, name, dtype):
  """Streams of different lengths against the plain implementation: each alone as one prompt, each mostly decoded
  (one from its first token on), and all as one batch."""
  d, w, model = model_of(name, 5, dtype, gpu)
  streams = [C.tokens(d, n, 10 + n) for n in (140, 41, 33)]
  want = [R.forward(d, w, s).numpy() for s in streams]
  for i, s in enumerate(streams):
    e = [err(all_logits(model, [s], cut)[0], want[i]) for cut in (0, len(s) - 1 if i == 2 else 30)]
    assert max(e) < TOL[dtype], (i, e)
  e = [err(got, want[i]) for i, got in enumerate(all_logits(model, streams, 32))]
  assert max(e) < TOL[dtype], e


def test_residual_after_every_layer_run(gpu):
  for name in sorted(C.CONFIGS):
    d, w, model = model_of(name, 6, F32, gpu)
    toks, want, got = C.tokens(d, 23, 3), [], []
    R.forward(d, w, toks, layers_out=want)
    runner = model.new_runner(1, 23, 23, -1)
    runner.residual_sink = lambda x: got.append(x.cpu().clone())
    runner.forward_hidden(i32([toks], gpu), None, runner.zero, model.new_cache(1, 23))
    assert len(got) == len(want) == len(model.cfg.layer_runs)
    for a, b in zip(got, want):
      assert rel(a, b) < 3e-5


@pytest.mark.parametrize("name,dtype", [("mixed", BF), ("mixed", F32), ("odd", F32), ("wide", BF), ("heads", F32)])
def test_portions_of_a_prompt(gpu, name, dtype):
  """The same prompt in portions of 2, 3, 7, 64 and 40 tokens, rows starting at different columns."""
  d, w, model = model_of(name, 7, dtype, gpu)
  streams = [C.tokens(d, n, 20 + n) for n in (116, 90)]
  P = 116
  buf = torch.full((2, P), -1, dtype=torch.int32)
  for b, s in enumerate(streams):
    buf[b, P - len(s):] = torch.tensor(s)
  buf, starts = buf.to(gpu), i32([P - len(s) for s in streams], gpu)
  cache, hidden, col = model.new_cache(2, P), [], 0
  for T in (2, 3, 7, 64, 40):
    r = model.new_runner(2, T, P, -1)
    hidden.append(r.forward_hidden(buf, None, i32([col], gpu), cache, starts=starts)[:2 * T].view(2, T, -1).clone())
    col += T
  assert col == P
  x = torch.cat(hidden, dim=1)
  for b, s in enumerate(streams):
    rows = x[b, P - len(s):].contiguous()
    lg = torch.empty(len(s), d["vocab"], device=gpu)
    r.part = torch.empty(len(s) * r.nvb * 4, device=gpu)
    r.run_head(rows, len(s), logits_out=lg)
    assert err(lg.cpu().numpy(), R.forward(d, w, s).numpy()) < TOL[dtype]


@pytest.mark.parametrize("dtype", DTYPES)
def test_reused_slots(gpu, dtype):
  """A cache that other sequences have filled gives the same logits as a new one, bit for bit."""
  d, w, model = model_of("mixed", 8, dtype, gpu)
  toks = i32([C.tokens(d, 70, 31), [0] * 20 + C.tokens(d, 50, 32)], gpu)
  other = i32([C.tokens(d, 90, 33), C.tokens(d, 90, 34)], gpu)
  starts, out = i32([0, 20], gpu), []
  for used in (False, True):
    cache = model.new_cache(2, 96)
    if used:
      model.new_runner(2, 90, 96, -1).forward_hidden(other, None, i32([0], gpu), cache)
    r = model.new_runner(2, 60, 96, -1)
    h = [r.forward_hidden(toks, None, r.zero, cache, starts=starts).view(2, 60, -1).clone()]
    h[0][1, :20] = 0.0                                # (in front of the second row's first token)
    r1 = model.new_runner(2, 1, 96, -1)
    for t in range(60, 70):
      h.append(r1.forward_hidden(toks, None, i32([t], gpu), cache, starts=starts).view(2, 1, -1).clone())
    out.append(torch.cat(h, 1))
  assert torch.equal(out[0], out[1])


def test_long_decoding_across_cache_growth(gpu):
  """Two tokens of prompt, then hundreds of steps: the cache grows, states and rings are carried all the way."""
  for dtype in DTYPES:
    d, w, model = model_of("mixed", 9, dtype, gpu)
    s = C.tokens(d, 280, 40)
    assert err(all_logits(model, [s], 278)[0], R.forward(d, w, s).numpy()) < TOL[dtype]


def test_a_batch_whose_rows_end_one_after_another(gpu):
  """Slots that are given back go on beside the others without being read."""
  d, w, model = model_of("mixed", 15, F32, gpu)
  streams = {str(i): C.tokens(d, n, 60 + n) for i, n in enumerate((30, 26, 21))}
  rp, got = Replay(model), {r: [] for r in streams}
  at = {r: len(s) - 10 + 3 * int(r) for r, s in streams.items()}
  rp.step({"entries": [{"id": r, "tokens": s[:at[r]], "want": []} for r, s in streams.items()], "end": []})
  while rp.batches:
    live = [r for r in streams if at[r] < len(streams[r])]
    lg = rp.step({"entries": [{"id": r, "tokens": [streams[r][at[r]]], "want": [0]} for r in live],
                  "end": [r for r in live if at[r] + 1 == len(streams[r])]})
    for r, row in zip(live, lg):
      got[r].append(row)
      at[r] += 1
  for r, s in streams.items():
    assert err(np.stack(got[r]), R.forward(d, w, s).numpy()[len(s) - len(got[r]):]) < TOL[F32]


@pytest.mark.parametrize("name,dtype", [("mixed", BF), ("mixed", F32), ("odd", F32), ("wide", BF)])
def test_greedy_generation(gpu, name, dtype):
  """The public sampler (prompts of different lengths, graph replay): what it picks is the plain implementation's best
  up to rounding; replayed steps give what eager ones give."""
  d, w, model = model_of(name, 10, dtype, gpu)
  prompts = [np.array(C.tokens(d, n, 50 + n), dtype=np.int32) for n in (40, 3, 17, 1)]
  sampler = Sampler(model, IdTokenizer(d["vocab"], pad_id=0, eos_id=1), CacheConfig(64 + 40))
  out = sampler(prompts, 40, max_prompt_length=64, return_logprobs=True, eos_tokens=[-1])
  eager = Sampler(model, sampler.tokenizer, CacheConfig(64 + 40), use_graph=False)(prompts, 40, max_prompt_length=64, eos_tokens=[-1])
  for p, t, lp, te in zip(prompts, out.tokens, out.logprobs, eager.tokens):
    assert list(t) == list(te)
    lg = R.forward(d, w, list(p) + list(t)).double()[len(p) - 1:-1]
    spread, rows, ids = float(lg.std()), torch.arange(40), torch.tensor(t.astype(np.int64))
    tol = 1e-3 if dtype == F32 else 0.3
    assert float((lg.max(-1).values - lg[rows, ids]).max()) < tol * spread
    assert float((torch.tensor(lp).double() - torch.log_softmax(lg, -1)[rows, ids]).abs().max()) < tol * spread


@pytest.mark.parametrize("name,dtype", [("mixed", BF), ("odd", BF), ("mixed", F32)])
def test_sampling_modes(gpu, name, dtype):
  """top-k 1 is greedy; a seed repeats itself; draws, nucleus and top-k run on the capped logits; logits come back."""
  d, w, model = model_of(name, 11, dtype, gpu)
  prompts = [C.tokens(d, n, 60 + n) for n in (9, 20)]
  s = Sampler(model, IdTokenizer(d["vocab"], pad_id=-1, eos_id=1), CacheConfig(48))
  call = lambda **kw: [list(t) for t in s(prompts, 12, max_prompt_length=32, eos_tokens=[-1], **kw).tokens]
  greedy = call()
  assert call(temperature=1.0, top_p=1.0, top_k=1, seed=3) == greedy
  for kw in (dict(top_p=1.0), dict(top_p=0.8), dict(top_p=0.9, top_k=20), dict(top_p=1.0, top_k=d["vocab"])):
    a = call(temperature=2.5, seed=4, **kw)
    assert a == call(temperature=2.5, seed=4, **kw) and a != call(temperature=2.5, seed=5, **kw)
  out = s(prompts, 12, max_prompt_length=32, eos_tokens=[-1], return_logits=True)
  for p, t, lg in zip(prompts, out.tokens, out.logits):
    assert np.abs(lg).max() <= d["logit_softcap"] * 1.01
    assert err(lg, R.forward(d, w, list(p) + list(t)).numpy()[len(p) - 1:-1]) < TOL[dtype]


def test_rollout_log_probabilities_and_weight_updates(gpu):
  d, w, model = model_of("mixed", 12, F32, gpu)
  roll = HipRollout(model, IdTokenizer(d["vocab"], pad_id=0, eos_id=1), 64)
  prompts = [[5, 9, 33, 7], [8, 3]]
  res = roll.generate(prompts, RolloutConfig(max_tokens_to_generate=10, temperature=0.0, top_p=None, max_prompt_length=8,
                                             eos_tokens=[-1], return_logprobs=True))
  comp = np.stack(res.tokens)
  pt = np.array([[0] * (8 - len(p)) + p for p in prompts])
  lp = roll.get_per_token_logps(pt, comp).cpu().numpy()
  for i, p in enumerate(prompts):
    want = torch.log_softmax(R.forward(d, w, p + list(comp[i])).double(), -1)[len(p) - 1:-1]
    want = want[torch.arange(10), torch.tensor(comp[i].astype(np.int64))].numpy()
    assert np.abs(lp[i] - want).max() < 2e-3 and np.abs(np.array(res.logprobs[i]) - lp[i]).max() < 2e-3
  w2 = C.random_weights(d, 13)
  before = all_logits(model, [prompts[0]], 2)[0]
  bad = dict(w2)
  bad["l0.mix.left.k"] = bad["l0.mix.left.k"][:, :-1]
  with pytest.raises(ValueError, match="same shape"):
    roll.update_params(bad)
  with pytest.raises(ValueError, match="same structure"):
    roll.update_params({"l0.mix.right.q": w2["l0.mix.right.q"]})        # a member of a fused projection without the others
  assert np.array_equal(all_logits(model, [prompts[0]], 2)[0], before)
  for part in ("head", "l0.mix.left.talk", "l2.canon2", "l2.mix.left.v.conv", "loop.step", "embed"):      # alone, one after another
    w[part] = w2[part]
    roll.update_params({part: w2[part]})
    assert err(all_logits(model, [prompts[0]], 2)[0], R.forward(d, w, prompts[0]).numpy()) < TOL[F32], part
  roll.update_params(w2)
  assert err(all_logits(model, [prompts[0]], 2)[0], R.forward(d, w2, prompts[0]).numpy()) < TOL[F32]


@pytest.mark.parametrize("B", [1, 40, 130])
def test_batch_sizes_of_a_decode_step(gpu, B):
  """Every row tile of the few-row kernels: a batch of equal sequences gives every row the same logits."""
  d, w, model = model_of("mixed", 14, BF, gpu)
  s = C.tokens(d, 12, 70)
  got = all_logits(model, [s] * B, 4)
  want = R.forward(d, w, s).numpy()
  for g in got[:: max(1, B // 5)]:
    assert err(g, want) < TOL[BF]


def test_a_long_prompt_takes_the_many_row_kernels(gpu):
  """More rows than the few-row kernels take.  (Among so many rows of random weights one may have a memory whose n . q all
  but vanishes, which magnifies rounding in fp32 as in bf16: most rows, and every row loosely.)"""
  d, w, model = model_of("mixed", 16, BF, gpu)
  streams = [C.tokens(d, n, 90 + n) for n in (330, 300)]
  for g, s in zip(all_logits(model, streams, 2), streams):
    want = R.forward(d, w, s).numpy()
    e = g - want
    rows = np.sqrt(((e - e.mean(-1, keepdims=True)) ** 2).mean(-1)) / want.std()
    assert np.quantile(rows, 0.9) < 0.5 * TOL[BF] and rows.max() < 2.5 * TOL[BF]


def test_command_line(gpu, tmp_path):
  """bin/trace_run and `python -m tunix_amd generate` on a model folder, as child processes."""
  d, w = C.write_model(tmp_path, "odd", seed=17)
  a, b = C.tokens(d, 12, 80), C.tokens(d, 7, 81)
  steps = [{"step": 0, "entries": [{"id": "a", "tokens": a[:11], "want": [10, 0]}, {"id": "b", "tokens": b[:6], "want": []}], "end": []},
           {"step": 1, "entries": [{"id": "a", "tokens": a[11:], "want": [0]}, {"id": "b", "tokens": b[6:], "want": [0]}], "end": ["b", "a"]}]
  out = tmp_path / "out"
  out.mkdir()
  p = subprocess.run([os.path.join(ROOT, "bin", "trace_run"), "--model", str(tmp_path), "--dtype", "float32", "--out", str(out),
                      "--max-tokens", "64"], input="\n".join(json.dumps(s) for s in steps), capture_output=True, text=True, timeout=100)
  assert p.returncode == 0, p.stderr[-2000:]
  la, lb = R.forward(d, w, a).numpy(), R.forward(d, w, b).numpy()
  read = lambda n: np.fromfile(out / f"{n}.f32", "<f4").reshape(-1, d["vocab"])
  assert err(read(0), la[[10, 0]]) < 1e-4 and err(read(1), np.stack([la[11], lb[6]])) < 1e-4
  p = subprocess.run([sys.executable, "-m", "tunix_amd", "generate", "--model", str(tmp_path), "--dtype", "float32", "--max-tokens", "4",
                      "--prompt", " ".join(map(str, a))], capture_output=True, text=True, timeout=100, cwd=ROOT)
  assert p.returncode == 0, p.stderr[-2000:]
  full = list(a)
  for t in json.loads(p.stdout)["tokens"]:
    lg = R.forward(d, w, full)[-1]
    assert float(lg.max() - lg[t]) < 1e-3
    full.append(t)
  assert len(full) == len(a) + 4


def test_descriptor_errors(gpu):
  """Shapes the kernels do not take are refused before any launch."""
  z = torch.zeros(64, 128, dtype=BF, device=gpu)
  p = L.ParallelStepDesc()
  p.M, p.D, p.B, p.T, p.x, p.w_next, p.out1, p.out_ld = 2, 64, 1, 2, z.data_ptr(), z.data_ptr(), z.data_ptr(), 128
  p.conv1, p.taps, p.slots, p.starts, p.col_ptr, p.ring = z.data_ptr(), 3, 1, z.data_ptr(), z.data_ptr(), z.data_ptr()
  with pytest.raises(ValueError, match="need a ring"):
    ops.parallel_step(p)
  c = L.ConvKvDesc()
  c.B, c.T, c.S, c.H, c.G, c.dk, c.dv, c.dkp, c.dvp, c.taps, c.slots = 1, 1, 8, 2, 2, 16, 16, 16, 16, 3, 2
  with pytest.raises(ValueError, match="shorter than the taps"):
    ops.conv_kvwrite(c)
  a = L.MixedAttnDesc()
  a.B, a.T, a.S, a.H, a.G = 1, 1, 8, 3, 2
  with pytest.raises(ValueError, match="bad shape"):
    ops.mixed_attn(a)
  m = L.MemoryDesc()
  m.B, m.T, m.H, m.dk, m.dv = 1, 1, 2, 0, 8
  with pytest.raises(ValueError, match="bad shape"):
    ops.memory(m)
  with pytest.raises(ValueError, match="soft_cap"):
    ops.soft_cap(torch.zeros(4, device=gpu), 0.0)
