"""Kezolix on the GPU against the plain implementation (oracle/kezolix_ref.py): every mechanism alone, then whole
models -- prompts, token-by-token decoding, portions, unequal batches, reused slots, greedy generation -- in bf16
and in fp32, at sizes that reach every kernel."""
import json
import os
import subprocess
import sys

import numpy as np
import pytest
import torch

from oracle import kezolix_ref as R
from tests import kezolix_cases as C
from tests.test_gpu_lapevik import source
from tests.test_gpu_nunezen import BF, DTYPES, F32, all_logits, err, frag, i32, rel, rnd, run_linear, unfrag
from tunix_amd import _lib as L
from tunix_amd import config, ops
from tunix_amd.generate import CacheConfig, Sampler
from tunix_amd.generate.replay import Replay
from tunix_amd.generate.utils import IdTokenizer
from tunix_amd.rl.rollout import HipRollout, RolloutConfig
from tunix_amd.stack_model import DenseLinear, LinearBank, StackModel

pytestmark = pytest.mark.gpu
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))


def up(n, m):
  return (n + m - 1) // m * m


# ---- embedding ------------------------------------------------------------------------------------
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("D", [52, 128])
def test_learned_positions(gpu, dtype, D):
  """Positions count from every row's first column; columns in front of it, and behind the table, stay inside the table."""
  table, pos, ids = rnd(37, D).to(BF).to(dtype), rnd(5, D, seed=1).to(BF).to(dtype), torch.tensor([[3, 36, 0, 9, 1, 2], [5, 5, 1, 2, 7, 8]], dtype=torch.int32)
  x, starts = torch.empty(8, D, device=gpu), [0, 3]
  ops.embed_rows(table.to(gpu), ids.to(gpu), i32([2], gpu), 2, 4, 37, D, x, scale=2.0, pos=pos.to(gpu), starts=i32(starts, gpu))
  want = [2.0 * table[ids[b, 2 + t].long()].float() + pos[min(max(2 + t - s, 0), 4)].float() for b, s in enumerate(starts) for t in range(4)]
  torch.testing.assert_close(x.cpu(), torch.stack(want))


# ---- linears with a squared positive part -----------------------------------------------------------
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("M,K,N", [(1, 100, 48), (33, 128, 208), (65, 320, 96), (129, 1000, 272), (700, 256, 528), (1100, 128, 32), (2500, 136, 112)])
def test_square_relu_linear(gpu, dtype, M, K, N):
  w, x = rnd(N, K, seed=1, scale=K ** -0.5).to(BF).float(), rnd(M, K, seed=2).to(BF).float()
  f = DenseLinear(["w"], {"w": w}, dtype, gpu)
  z = x @ w.T
  want = z.clamp(min=0) ** 2
  xp = torch.zeros(M, f.Kp, dtype=dtype, device=gpu)
  xp[:, :K] = x.to(dtype)
  for fr in ([False, True] if dtype == BF and M <= 512 else [False]):
    out = torch.zeros(up(M, 128), up(N, 128), dtype=dtype, device=gpu)
    run_linear(f, frag(xp) if fr else xp, M, out, epilogue=L.TNX_EPI_RELU2, x_frag=fr, y_frag=fr)
    assert rel((unfrag(out, M) if fr else out[:M])[:, :N], want) < (2e-6 if dtype == F32 else 4e-3)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("M,top,E", [(3, 2, 5), (70, 3, 4), (600, 2, 3)])
def test_square_relu_experts(gpu, dtype, M, top, E):
  K, N = 136, 72
  names = [f"e{e}" for e in range(E)]
  w = {n: rnd(N, K, seed=i, scale=K ** -0.5).to(BF).float() for i, n in enumerate(names)}
  bank = LinearBank([DenseLinear([n], w, dtype, gpu) for n in names])
  x = rnd(M, K, seed=9).to(BF).float()
  ids = torch.stack([torch.randperm(E, generator=torch.Generator().manual_seed(m))[:top] for m in range(M)]).to(torch.int32)
  counts, offsets, order = (torch.empty(n, dtype=torch.int32, device=gpu) for n in (E, E + 1, M * top))
  ops.moe_sort_routes(ids.to(gpu), E, counts, offsets, order)
  xp = torch.zeros(M, bank.Kp, dtype=dtype, device=gpu)
  xp[:, :K] = x.to(dtype)
  out = torch.zeros(M * top, 128, dtype=dtype, device=gpu)
  d = L.DenseDesc()
  d.M, d.K, d.N, d.dtype, d.x, d.ldx, d.w, d.w_stride = M * top, bank.Kp, bank.N, ops.DTYPES[dtype], xp.data_ptr(), bank.Kp, bank.w.data_ptr(), bank.stride
  d.epilogue, d.y, d.ldy, d.split_k, d.n_experts, d.x_div = L.TNX_EPI_RELU2, out.data_ptr(), 128, 1, E, top
  d.offsets, d.sorted_route = offsets.data_ptr(), order.data_ptr()
  ops.dense_linear(d)
  want = torch.stack([(x[m] @ w[names[int(ids[m, k])]].T).clamp(min=0) ** 2 for m in range(M) for k in range(top)])
  assert rel(out[:, :N], want) < (2e-6 if dtype == F32 else 4e-3)


@pytest.mark.parametrize("dtype", DTYPES)
def test_columns_of_a_projection(gpu, dtype):
  """Members that begin at runs of 256 columns may be run apart from the others."""
  w = {n: rnd(r, 200, seed=r, scale=0.1).to(BF).float() for n, r in (("a", 40), ("b", 300), ("c", 264))}
  f, x = DenseLinear(["a", "b", "c"], w, dtype, gpu, align=256), rnd(600, 200, seed=4).to(BF).float()
  assert f.offsets == [0, 256, 768] and f.N == 1280
  xp = torch.zeros(600, f.Kp, dtype=dtype, device=gpu)
  xp[:, :200] = x.to(dtype)
  for n, c0, c1 in (("a", 0, 256), ("b", 256, 768), ("c", 768, 1280)):
    out = torch.zeros(600, c1 - c0, dtype=dtype, device=gpu)
    d = L.DenseDesc()
    d.M, d.K, d.N, d.dtype, d.x, d.ldx, d.split_k = 600, f.Kp, c1 - c0, ops.DTYPES[dtype], xp.data_ptr(), f.Kp, 1
    d.w, d.y, d.ldy = f.w.data_ptr() + c0 * f.Kp * f.w.element_size(), out.data_ptr(), c1 - c0
    ops.dense_linear(d)
    assert rel(out[:, :w[n].shape[0]], x @ w[n].T) < (2e-6 if dtype == F32 else 4e-3) and not out[:, w[n].shape[0]:].any()


# ---- residual step --------------------------------------------------------------------------------------
def layer_step(gpu, dtype, D, M, center=True, mult=0.6, n=0, store=True, routes=0, extra=False, mode=1, split=1, fr=False, w_next=True, apart=False, offset=0.0):
  """Runs one step on random rows and compares everything that it writes."""
  eps, tol = 0.03, 2e-6 if dtype == F32 else 4e-3
  g = lambda *s, seed: rnd(*s, seed=seed) + 0.7                    # (rows whose mean is not zero)
  x, y, e = g(M, D, seed=1), g(M * max(routes, 1), D, seed=2).to(BF).float(), g(M, D, seed=3).to(BF).float()
  rw, ew = rnd(M, max(routes, 1), seed=4), rnd(M, seed=5)
  wp, wn, hw, hist = rnd(D, seed=6), rnd(D, seed=7), rnd(n + 1, seed=8), rnd(n + 2, M, D, seed=9)
  dev = lambda t: t.to(gpu).contiguous()
  src, keep = source(y, dtype, gpu, 1 if routes else split)
  esrc, keep2 = source(e, dtype, gpu, split)
  xg, xo, hg, out = dev(x), torch.full((M, D), float("nan"), device=gpu), dev(hist), torch.zeros(up(M, 128), up(D, 128), dtype=dtype, device=gpu)
  wpg, wng, hwg, rwg, ewg = dev(wp), dev(wn), dev(hw), dev(rw), dev(ew)
  d = L.ResidualNormDesc()
  d.M, d.D, d.dtype, d.eps, d.mode, d.center, d.mult, d.w_offset = M, D, ops.DTYPES[dtype], eps, mode, int(center), mult, offset
  d.x, d.out, d.out_ld, d.out_frag = xg.data_ptr(), out.data_ptr(), out.shape[1], int(fr)
  if apart:
    d.x_out = xo.data_ptr()
  if mode == 1:
    d.y, d.w_post = src, wpg.data_ptr()
    if routes:
      d.route_w, d.route_k = rwg.data_ptr(), routes
    if extra:
      d.extra, d.extra_w = esrc, ewg.data_ptr()
  if w_next:
    d.w_next = wng.data_ptr()
  if n:
    d.hist, d.hist_plane, d.hist_n, d.hist_store, d.hist_w = hg.data_ptr(), M * D, n, int(store), hwg.data_ptr()
  ops.residual_norm(d)
  norm = (lambda v, w: R.layer_norm(v, w, eps)) if center else (lambda v, w: R.rms_norm(v, eps, w))
  new = x
  if mode == 1:
    z = (y.view(M, routes, D) * rw[:, :, None]).sum(1) if routes else y
    new = x + mult * norm(z + ew[:, None] * e if extra else z, offset + wp)
  if n:
    if store:
      assert rel(hg[n], new) < 3e-6
      hist[n] = new
    assert torch.equal(hg.cpu()[:n], hist[:n]) and torch.equal(hg.cpu()[n + 1], hist[n + 1]) and (store or torch.equal(hg.cpu()[n], hist[n]))
    new = R.depth_average(list(hist[:n]) + [new], hw)
  if apart and (mode or n):
    assert rel(xo, new) < 3e-6 and torch.equal(xg.cpu(), x)
  else:
    assert rel(xg, new) < 3e-6
  want = norm(new, offset + wn) if w_next else new
  assert rel((unfrag(out, M) if fr else out[:M])[:, :D], want) < tol


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("D", [8, 52, 128, 1000, 2048, 2056, 4096, 5000, 8192, 8200, 12288, 2051])
def test_layer_step_widths(gpu, dtype, D):
  bf = dtype == BF
  layer_step(gpu, dtype, D, 5, n=3, extra=True, split=2 if bf else 1)
  layer_step(gpu, dtype, D, 3, n=1, routes=2, extra=True, fr=bf, apart=True)
  layer_step(gpu, dtype, D, 2, center=False, n=6, store=False)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("D", [96, 100])
def test_layer_step_forms(gpu, dtype, D):
  """Every part with and without the others: layer norms and root-mean-square ones, factors, nothing incoming, the first
  layer and later ones, no next norm."""
  bf = dtype == BF
  for center in (True, False):
    for n in (0, 1, 9):
      for routes, extra in ((0, False), (0, True), (3, False), (5, True)):
        layer_step(gpu, dtype, D, 7, center=center, n=n, routes=routes, extra=extra, split=3 if bf and not routes else 1, fr=bf and n == 1)
    layer_step(gpu, dtype, D, 4, center=center, n=2, mult=1.0, w_next=False, offset=1.0)
    layer_step(gpu, dtype, D, 4, center=center, mult=1.7, mode=0, apart=True)
    layer_step(gpu, dtype, D, 4, center=center, mult=0.5, mode=0)
  layer_step(gpu, dtype, D, 1500, n=2, store=False)


def test_layer_norm_of_a_far_mean(gpu):
  """A row whose mean is thousands of times its spread: the deviations are formed from the mean, not from squares."""
  D, M = 1024, 4
  x = 3000.0 + rnd(M, D, seed=1)
  out, w, xg = torch.zeros(128, D, dtype=F32, device=gpu), torch.ones(D, device=gpu), x.to(gpu)
  d = L.ResidualNormDesc()
  d.M, d.D, d.dtype, d.eps, d.center, d.mode = M, D, L.TNX_F32, 1e-6, 1, 0
  d.x, d.w_next, d.out, d.out_ld = xg.data_ptr(), w.data_ptr(), out.data_ptr(), D
  ops.residual_norm(d)
  assert rel(out[:M], R.layer_norm(x.double(), torch.ones(D), 1e-6)) < 2e-4


# ---- norms over projections + cache write ----------------------------------------------------------------
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,G,dk,dv", [(6, 2, 32, 48), (4, 1, 64, 24), (3, 3, 21, 13), (10, 5, 12, 45), (16, 2, 136, 200), (32, 8, 128, 128), (2, 1, 300, 16), (64, 8, 128, 128), (40, 40, 256, 256)])
def test_row_norms_and_cache_write(gpu, dtype, H, G, dk, dv):
  B, T, S, col, eps = 3, 2, 9, 4, 0.05
  dkp, dvp = ops.sink_attn_pad(dk, False, dtype), ops.sink_attn_pad(dv, True, dtype)
  offs = [0, up(H * dk, 16), up(H * dk, 16) + up(G * dk, 16)]
  y = torch.zeros(B * T, offs[2] + up(G * dv, 16))
  q, k, v = (rnd(B * T, n, seed=n).to(BF).float() for n in (H * dk, G * dk, G * dv))
  for o, t in zip(offs, (q, k, v)):
    y[:, o:o + t.shape[1]] = t
  wq, wk = rnd(H * dk, seed=1), rnd(G * dk, seed=2)
  for split, own in ((1, True), (2, True), (1, False), (3, False)):
    if dtype == F32 and split > 1:
      continue
    src, keep = source(y, dtype, gpu, split)
    qo = torch.full((B * T, H, dkp), float("nan"), dtype=dtype, device=gpu)
    kc, vc = (torch.full((B, G, S, n), 3.0, dtype=dtype, device=gpu) for n in (dkp, dvp))
    wqg, wkg, cp = wq.to(gpu), wk.to(gpu), i32([col], gpu)
    d = L.RowNormKvDesc()
    d.B, d.T, d.S, d.H, d.G, d.dk, d.dv, d.dkp, d.dvp, d.dtype, d.eps = B, T, S, H, G, dk, dv, dkp, dvp, ops.DTYPES[dtype], eps
    d.w_q, d.y, d.k_off, d.v_off, d.col_ptr, d.q_out = wqg.data_ptr(), src, offs[1], offs[2], cp.data_ptr(), qo.data_ptr()
    if own:
      d.w_k, d.kcache, d.vcache = wkg.data_ptr(), kc.data_ptr(), vc.data_ptr()
    ops.rownorm_kvwrite(d)
    tol = 2e-6 if dtype == F32 else 4e-3
    assert rel(qo[..., :dk], R.rms_norm(q, eps, wq).view(B * T, H, dk)) < tol and not qo[..., dk:].any()
    written = slice(col, col + T)
    if own:
      for cache, n, t in ((kc, dk, R.rms_norm(k, eps, wk)), (vc, dv, v)):
        got = cache[:, :, written].transpose(1, 2).reshape(B * T, G, -1)
        assert rel(got[..., :n], t.view(B * T, G, n)) < tol and not got[..., n:].any()
        cache[:, :, written] = 3.0
    assert bool((kc == 3.0).all()) and bool((vc == 3.0).all())


# ---- attention with slopes and chunks ---------------------------------------------------------------------
class Biased:
  def __init__(self, gpu, dtype, H, G, dk, dv, S, starts, chunk, seed=0, sharp=2.0, scale=None, slopes=True):
    self.gpu, self.dtype, self.H, self.G, self.dk, self.dv, self.S, self.starts, self.B, self.chunk = gpu, dtype, H, G, dk, dv, S, list(starts), len(starts), chunk
    self.dkp, self.dvp = ops.sink_attn_pad(dk, False, dtype), ops.sink_attn_pad(dv, True, dtype)
    r = lambda n, d, s: rnd(self.B, S, n, d, seed=seed + s).to(BF).float()
    self.q, self.k, self.v = (r(H, dk, 1) * sharp).to(BF).float(), r(G, dk, 2), r(G, dv, 3)
    self.scale = dk ** -0.5 if scale is None else scale
    self.slopes = torch.tensor(config.distance_slopes(H)) if slopes else None
    self.lay_out()

  def lay_out(self):
    pad = lambda t, n: torch.nn.functional.pad(t, (0, n - t.shape[-1])).to(self.dtype)
    slab = lambda t, n: pad(t, n).transpose(1, 2).contiguous().to(self.gpu)
    self.qp, self.kc, self.vc = pad(self.q, self.dkp), slab(self.k, self.dkp), slab(self.v, self.dvp)

  def run(self, col, T, split=0, fr=False):
    gpu, B, H = self.gpu, self.B, self.H
    assert col + T <= self.S and self.kc.shape == (B, self.G, self.S, self.dkp)
    q = self.qp[:, col:col + T].contiguous().to(gpu)
    out = torch.zeros(up(B * T, 128), up(H * self.dv, 128), dtype=self.dtype, device=gpu)
    st, cp = i32(self.starts, gpu), i32([col], gpu)
    sl = None if self.slopes is None else self.slopes.to(gpu)
    ws = torch.empty(max(1, ops.sink_attn_ws_bytes(B, T, self.S, H, self.dvp, split) // 4), device=gpu)
    d = L.SinkAttnDesc()
    d.B, d.T, d.S, d.H, d.G, d.dk, d.dv, d.dkp, d.dvp = B, T, self.S, H, self.G, self.dk, self.dv, self.dkp, self.dvp
    d.scale, d.dtype, d.q, d.kcache, d.vcache = self.scale, ops.DTYPES[self.dtype], q.data_ptr(), self.kc.data_ptr(), self.vc.data_ptr()
    d.slopes, d.chunk = None if sl is None else sl.data_ptr(), self.chunk
    d.starts, d.col_ptr, d.kv_chunk, d.ws, d.out, d.out_ld, d.out_frag = st.data_ptr(), cp.data_ptr(), split, ws.data_ptr(), out.data_ptr(), out.shape[1], int(fr)
    ops.sink_attn(d)
    torch.cuda.synchronize()
    return (unfrag(out, B * T) if fr else out[:B * T])[:, :H * self.dv].float().cpu().view(B, T, H, self.dv)

  def want(self, b):
    if not hasattr(self, "_want"):
      self._want = {}
    if b not in self._want:
      s = self.starts[b]
      # (without slopes: keys and queries one dimension longer, whose product is what the slopes take off)
      q, k = self.q[b, s:], self.k[b, s:]
      if self.slopes is None:
        n = q.shape[0]
        at, ones = torch.arange(n).float(), torch.ones(n)
        sl = torch.tensor(R.slopes(self.H))
        q = torch.cat([q, (at[:, None] * sl / self.scale)[..., None], (-sl / self.scale).expand(n, -1)[..., None]], -1)
        k = torch.cat([k, ones[:, None, None].expand(n, self.G, 1), at[:, None, None].expand(n, self.G, 1)], -1)
      self._want[b] = R.biased_attention(q, k, self.v[b, s:], self.scale, self.chunk or 10 ** 9)
    return self._want[b]

  def check(self, got, col):
    T = got.shape[1]
    for b, s in enumerate(self.starts):
      lo = max(s, col)
      if lo >= col + T:
        continue
      w = self.want(b)[lo - s:col + T - s]
      e = float((got[b, lo - col:] - w).abs().max() / w.abs().max())
      assert e < (3e-5 if self.dtype == F32 else 2e-2), (b, col, T, e)


HEADS = [(6, 2, 32, 48), (4, 1, 64, 24), (3, 3, 21, 13), (10, 5, 12, 45), (16, 2, 136, 200), (20, 5, 64, 96), (32, 8, 128, 128), (5, 1, 256, 256), (2, 1, 300, 16), (1, 1, 16, 16)]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("i", range(len(HEADS)))
def test_biased_attention_prompt_portions_and_steps(gpu, dtype, i):
  """Every group of head sizes; chunks of every length beside a tile's, one of them a single position; rows with different
  starts; portions from two tokens up; single tokens whose keys are split."""
  S, bf = 150, dtype == BF
  for chunk in [(20, 1), (64, 7), (33, 500), (0, 31), (32, 127), (40, 150), (65, 16), (100, 3), (50, 2), (10, 0)][i]:
    a = Biased(gpu, dtype, *HEADS[i], S, [0, 37, 149], chunk, seed=i)
    a.check(a.run(0, S), 0)
    for col, T in ((0, 2), (2, 3), (5, 64), (69, 16), (85, 33), (148, 2)):
      a.check(a.run(col, T, fr=bf and T < 40), col)
    for j, t in enumerate((0, 1, 36, 37, 38, 63, 64, 65, 99, 100, 127, 128, 149)):
      a.check(a.run(t, 1, split=(32, 64, 0, 96)[j % 4] if bf else 0, fr=bf and j % 3 == 0), t)


@pytest.mark.parametrize("dtype", DTYPES)
def test_slopes_alone_and_chunks_alone(gpu, dtype):
  for chunk, slopes in ((0, True), (48, False)):
    a = Biased(gpu, dtype, 8, 2, 64, 64, 200, [0, 90], chunk, seed=5, slopes=slopes, scale=0.5 if slopes else -0.2)
    a.check(a.run(0, 200), 0)
    a.check(a.run(120, 5), 120)
    for t in (95, 96, 137, 138, 199):
      a.check(a.run(t, 1, split=32 if dtype == BF else 0), t)


@pytest.mark.parametrize("how", ["prompt", "portion", "decoded", "split"])
@pytest.mark.parametrize("start", [0, 13])
@pytest.mark.parametrize("chunk,at", [(120, 359), (120, 240), (120, 300), (64, 127), (64, 128), (63, 251), (63, 252), (31, 371), (400, 399), (397, 396), (397, 397), (5, 204), (1, 77)])
def test_a_key_at_a_chunks_edge(gpu, how, start, chunk, at):
  """The first position of the chunk holds a key far above the others, and the last one in front of it one still higher, as
  does the position behind: only the first is seen, from the chunk's last position as from its first one."""
  S, n = 440, 32
  a = Biased(gpu, BF, 4, 2, n, n, S, [start], chunk, seed=at, scale=1.0)
  first, q = start + at // chunk * chunk, start + at
  a.q[:] = 0.0
  a.q[..., 0] = 60.0
  a.k[:] = 0.0
  a.k[0, first, :, 0] = 6.0                          # (above what the steepest slope takes off over a chunk)
  if first > 0:
    a.k[0, first - 1, :, 0] = 12.0
  a.k[0, q + 1, :, 0] = 12.0
  a.lay_out()
  got = {"prompt": lambda: a.run(0, S)[0, q], "portion": lambda: a.run(max(q - 6, 0), 8)[0, q - max(q - 6, 0)], "decoded": lambda: a.run(q, 1)[0, 0],
         "split": lambda: a.run(q, 1, split=32)[0, 0]}[how]()
  assert rel(got, a.v[0, first].repeat_interleave(2, 0)) < 5e-3


def test_the_slope_is_taken_off(gpu):
  """Equal scores, then one far key exactly as much higher as the slope takes off: weights follow from the distances alone."""
  S, H = 100, 8
  for how in ("prompt", "decoded"):
    a = Biased(gpu, F32, H, 8, 16, 16, S, [0], 0, seed=1, scale=1.0)
    a.q[:], a.k[:] = 0.0, 0.0
    a.q[..., 0] = 1.0
    for h in range(H):
      a.k[0, 20, h, 0] = R.slopes(H)[h] * (90 - 20)    # as if it were the query's own position
    a.lay_out()
    got = a.run(0, S)[0, 90] if how == "prompt" else a.run(90, 1)[0, 0]
    for h in range(H):
      w = torch.exp(-R.slopes(H)[h] * (90.0 - torch.arange(91)))
      w[20] = 1.0
      assert rel(got[h], (w[:, None] * a.v[0, :91, h]).sum(0) / w.sum()) < 2e-5


# ---- recurrence with forget gates ---------------------------------------------------------------------------
class Gated:
  def __init__(self, gpu, dtype, H, dk, dv, S, starts, seed=0, spread=2.0, bias=1.5, lower=None):
    self.gpu, self.dtype, self.H, self.dk, self.dv, self.S, self.starts, self.B = gpu, dtype, H, dk, dv, S, list(starts), len(starts)
    r = lambda d, s: rnd(self.B, S, H, d, seed=seed + s).to(BF).float()
    self.q, self.v, self.z = r(dk, 1), r(dv, 2), spread * rnd(self.B, S, H, dk, seed=seed + 3)
    self.bias = bias + 2.0 * rnd(H, dk, seed=seed + 4)
    self.lower = (0.3 + 0.4 * rnd(H, dk, seed=seed + 5)).clamp(0.0, 1.0) if lower is None else torch.full((H, dk), lower)
    self.reset(7.0)

  def reset(self, x):
    """What another sequence has left: a new one must not see it."""
    self.state = torch.full((self.B, self.H, self.dk, self.dv), x, device=self.gpu)

  def run(self, col, T, split=1, y_f32=False, norm=None, eps=0.0, fr=False):
    gpu, B, H, M, qk = self.gpu, self.B, self.H, self.B * T, self.H * self.dk
    ov = 16 + up(qk, 16)
    y = torch.zeros(B, T, ov + up(H * self.dv, 16))
    y[:, :, 16:16 + qk], y[:, :, ov:ov + H * self.dv] = self.q[:, col:col + T].reshape(B, T, -1), self.v[:, col:col + T].reshape(B, T, -1)
    src, keep = source(y.view(M, -1), F32 if y_f32 else self.dtype, gpu, split)
    f, keep2 = source(torch.nn.functional.pad(self.z[:, col:col + T].reshape(M, qk), (32, 0)), F32, gpu, split)
    st, cp, bi, lo = i32(self.starts, gpu), i32([col], gpu), self.bias.to(gpu), self.lower.to(gpu)
    ws = torch.empty(max(1, ops.gated_state_ws_bytes(B, T, H, self.dk, self.dv) // 4), device=gpu)
    d = L.GatedStateDesc()
    d.B, d.T, d.H, d.dk, d.dv, d.dtype, d.y_f32 = B, T, H, self.dk, self.dv, ops.DTYPES[self.dtype], int(y_f32)
    d.y, d.q_off, d.v_off, d.f, d.f_off, d.bias, d.lower = src, 16, ov, f, 32, bi.data_ptr(), lo.data_ptr()
    d.starts, d.col_ptr, d.state, d.ws = st.data_ptr(), cp.data_ptr(), self.state.data_ptr(), ws.data_ptr()
    if norm is not None:
      wg, out = norm.to(gpu), torch.zeros(up(M, 128), up(H * self.dv, 128), dtype=self.dtype, device=gpu)
      d.norm_w, d.eps, d.out, d.out_ld, d.out_frag = wg.data_ptr(), eps, out.data_ptr(), out.shape[1], int(fr)
    else:
      out = torch.full((M, up(H * self.dv, 4)), float("nan"), device=gpu)
      d.o, d.o_ld = out.data_ptr(), out.shape[1]
    ops.gated_state(d)
    torch.cuda.synchronize()
    return (unfrag(out, M) if fr else out[:M])[:, :H * self.dv].float().cpu().view(B, T, H, self.dv)

  def want(self, b):
    if not hasattr(self, "_want"):
      self._want = {}
    if b not in self._want:
      s = self.starts[b]
      f = R.forget_gate(self.z[b, s:].double() + self.bias, self.lower.double())
      self._want[b] = R.gated_recurrence(R.silu(self.q[b, s:].double()), f, self.v[b, s:].double())
    return self._want[b]

  def check(self, got, col, tol=None):
    T = got.shape[1]
    tol = tol or (1e-5 if self.dtype == F32 else 4e-3)
    for b, s in enumerate(self.starts):
      lo = max(s, col)
      if lo >= col + T:
        continue
      o, S = self.want(b)
      assert rel(got[b, lo - col:], o[lo - s:col + T - s]) < tol, (b, col, T, rel(got[b, lo - col:], o[lo - s:col + T - s]))
      if col + T == self.S:
        assert rel(self.state[b], S) < (1e-5 if self.dtype == F32 else 1e-3), (b, col, T, rel(self.state[b], S))


GATED = [(3, 32, 48), (2, 64, 40), (2, 128, 128), (5, 16, 16), (2, 11, 9), (1, 20, 30), (2, 200, 136), (1, 256, 264), (9, 8, 8), (4, 96, 24), (1, 40, 1032)]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,dk,dv", GATED)
def test_recurrence_prompt_portions_and_steps(gpu, dtype, H, dk, dv):
  """One pass (cut into spans that run in parallel), portions from two tokens up, token by token, over rows with different
  starts; finished rows, fp32 rows and partial planes."""
  S, bf = 330, dtype == BF
  a = Gated(gpu, dtype, H, dk, dv, S, [0, 70, 129, 329], seed=H)
  a.check(a.run(0, S), 0)
  a.reset(-3.0)
  col = 0
  for T in (32, 2, 3, 31, 64, 2, 130):
    a.check(a.run(col, T, split=2 if bf and T < 64 else 1, y_f32=bf and T in (2, 64)), col)
    col += T
  for t in range(col, S):
    a.check(a.run(t, 1, split=2 if bf and t % 2 else 1, y_f32=bf and t % 4 == 0), t)
  b = Gated(gpu, dtype, H, dk, dv, 20, [0, 5], seed=9)
  for t in range(20):
    b.check(b.run(t, 1), t)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,dk,dv", [(3, 32, 48), (2, 128, 128), (5, 24, 4), (2, 64, 1000)])
def test_norms_behind_a_step(gpu, dtype, H, dk, dv):
  a, w, eps = Gated(gpu, dtype, H, dk, dv, 6, [0, 3], seed=2), rnd(dv, seed=8), 0.02
  assert ops.gated_state_step_ok(dk, dv)
  for t in range(6):
    fr = dtype == BF and t % 2 == 1
    got = a.run(t, 1, norm=w, eps=eps, fr=fr, split=2 if dtype == BF and t > 3 else 1)
    for b, s in enumerate(a.starts):
      if t >= s:
        assert rel(got[b, 0], R.rms_norm(a.want(b)[0][t - s], eps, w)) < (1e-5 if dtype == F32 else 6e-3)
  assert all(rel(a.state[b], a.want(b)[1]) < 1e-3 for b in range(2))


@pytest.mark.parametrize("how", ["prompt", "portions", "steps"])
@pytest.mark.parametrize("at", [0, 1, 15, 16, 31, 32, 33, 127, 128, 300])
def test_recurrence_keeps_and_loses(gpu, how, at):
  """One token writes, the others' gates are shut (the lower bound is one, or the sigmoid is): channels that keep hand the
  value back hundreds of tokens later, one with a bound below one keeps what the bound leaves, one loses it all."""
  S, H, dk, dv = 420, 2, 16, 32
  a = Gated(gpu, BF, H, dk, dv, S, [0], seed=at, lower=0.0)
  a.bias[:] = 0.0
  a.z[:] = 60.0                                     # nothing is written, nothing is lost
  a.z[0, at, :, :4] = -60.0                         # four channels take the token in full
  a.lower[:, 1] = 0.995                             # ... one of them a two-hundredth of it
  a.z[0, at + 1:, :, 2] = -60.0                     # one loses it at once
  a.v[0, at + 1:, :] = 0.0
  a.z[0, at + 1:, :, 1] = -60.0                     # one decays at its lower bound
  a.q[:] = 1.0
  got = {"prompt": lambda: a.run(0, S), "portions": lambda: torch.cat([a.run(c, T) for c, T in ((0, 2), (2, 198), (200, 64), (264, 156))], 1),
         "steps": lambda: torch.cat([a.run(t, 1) for t in range(S)], 1)}[how]()[0]
  v, silu1 = a.v[0, at], float(R.silu(torch.tensor(1.0)))
  assert float(got[:at].abs().max() if at else 0.0) < 1e-6
  far = S - 1 - at
  assert rel(got[at], silu1 * v * (3 + 0.005)) < 5e-3
  assert rel(got[S - 1], silu1 * v * (2 + 0.005 * 0.995 ** far)) < 5e-3
  a.check(got[None], 0)


@pytest.mark.parametrize("dtype", DTYPES)
def test_extreme_gates(gpu, dtype):
  """Gates at nought and one in turn, within a block and across: nothing overflows, and what a shut gate has dropped does not
  come back."""
  for H, dk, dv in ((3, 32, 16), (2, 128, 64), (2, 256, 32)):
    a = Gated(gpu, dtype, H, dk, dv, 200, [0, 11], seed=2, spread=60.0, lower=0.0)
    got = a.run(0, 200)
    assert torch.isfinite(got).all()
    a.check(got, 0)
    a.reset(float("nan") if dtype == F32 else 1.0)
    a.check(torch.cat([a.run(t, 1) for t in range(200)], 1), 0)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("W,groups", [(70, 5), (256, 2), (4096, 32), (72, 9), (2048, 1), (9000, 3)])
def test_norms_of_heads_with_shared_weights(gpu, dtype, W, groups):
  M, eps = 5, 0.3
  o, w = rnd(M, W, seed=1), rnd(W // groups, seed=2)
  og, wg, want = o.to(gpu), w.to(gpu), R.rms_norm(o.view(M, groups, -1), eps, w).view(M, W)
  for fr in ([False, True] if dtype == BF else [False]):
    out = torch.zeros(128, up(W, 128), dtype=dtype, device=gpu)
    d = L.GatedNormDesc()
    d.M, d.W, d.dtype, d.eps, d.groups, d.shared_w = M, W, ops.DTYPES[dtype], eps, groups, 1
    d.o, d.o_ld, d.w, d.out, d.out_ld, d.out_frag = og.data_ptr(), W, wg.data_ptr(), out.data_ptr(), out.shape[1], int(fr)
    ops.gated_norm(d)
    assert rel((unfrag(out, M) if fr else out[:M])[:, :W], want) < (2e-6 if dtype == F32 else 4e-3)


# ---- PolyNorm, choice of experts ------------------------------------------------------------------------------
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("F,split", [(40, 1), (33, 1), (200, 3), (2048, 2), (4096, 1), (5000, 2), (8192, 1), (14336, 2), (20000, 1), (33000, 1), (2051, 2)])
def test_poly_norm(gpu, dtype, F, split):
  M, eps = 4, 0.05
  z, coef = (1.5 * rnd(M, F, seed=1)).to(BF).float(), torch.tensor([0.7, -1.1, 0.4, 0.3])
  want = R.poly_norm(z, coef, eps)
  cg = coef.to(gpu)
  for fr in ([False, True] if dtype == BF else [False]):
    src, keep = source(z, dtype, gpu, split if dtype == BF else 1)
    out = torch.zeros(128, up(F, 128), dtype=dtype, device=gpu)
    ops.poly_norm(src, dtype, M, F, cg, eps, out, fr)
    got = unfrag(out, M) if fr else out[:M]
    assert rel(got[:, :F], want) < (2e-6 if dtype == F32 else 4e-3) and not got[:, F:].any()


@pytest.mark.parametrize("E,k", [(1, 1), (5, 2), (12, 3), (64, 8), (66, 66), (256, 6), (300, 7), (1000, 1)])
def test_choice_by_corrected_scores(gpu, E, k):
  M, scale = 37, 2.5
  z, c = 2.0 * rnd(M, E, seed=1), 0.2 * rnd(E, seed=2)
  z[3] = z[4]
  z[5, :] = 0.0                                     # (equal scores: the correction decides, then the lower id)
  c[E // 2:] = c[E // 2]
  both = torch.cat([z, torch.zeros(M, up(E, 16) - E), rnd(M, 1, seed=3)], 1)
  ids, w = R.route(z.double(), c.double(), k, scale)
  cg = c.to(gpu)
  for split in (1, 3):
    src, keep = source(both, F32, gpu, split)
    tw, ti, gw = torch.empty(M, k, device=gpu), torch.empty(M, k, dtype=torch.int32, device=gpu), torch.empty(M, device=gpu)
    ops.route_scores(src, M, E, k, cg, scale, tw, ti, up(E, 16), gw)
    assert torch.equal(ti.cpu().long()[5], ids[5]) and float((ti.cpu() == ids).float().mean()) > 0.999
    ok = (ti.cpu() == ids).all(1)
    assert rel(tw.cpu()[ok], w[ok]) < 2e-6
    torch.testing.assert_close(gw.cpu(), torch.sigmoid(both[:, -1]), rtol=2e-6, atol=1e-7)
    # beside experts that every row uses: the same, and longer rows
    for n in (1, 3):
      tw2, ti2 = torch.empty(M, k + n, device=gpu), torch.empty(M, k + n, dtype=torch.int32, device=gpu)
      ops.route_scores(src, M, E, k, cg, scale, tw2, ti2, up(E, 16), ld=k + n)
      assert torch.equal(ti2[:, :k], ti) and torch.equal(tw2[:, :k], tw)
      assert torch.equal(ti2[:, k:].cpu(), torch.arange(E, E + n, dtype=torch.int32).expand(M, n)) and torch.equal(tw2[:, k:], gw[:, None].expand(M, n))
  plain = torch.empty(M, k, device=gpu)
  ops.route_scores(src, M, E, k, None, 1.0, plain, ti)
  assert torch.equal(ti.cpu().long().sort(1).values[:1], R.route(z.double(), torch.zeros(E), k, 1.0)[0].sort(1).values[:1])
  assert rel(plain.sum(1), torch.ones(M)) < 1e-6


def test_scores_that_vanish_and_rows_of_nan(gpu):
  """Chosen experts whose scores are all but nought are divided by 1e-20 too; k distinct experts whatever the logits hold."""
  z = torch.full((2, 16), -300.0)
  z[0, 3] = 0.0
  z[1, 5] = float("nan")
  c = torch.zeros(16)
  c[3], c[7], c[9] = -5.0, 1.0, 0.5
  src, keep = source(z, F32, gpu, 1)
  tw, ti, cg = torch.empty(2, 2, device=gpu), torch.empty(2, 2, dtype=torch.int32, device=gpu), c.to(gpu)
  ops.route_scores(src, 2, 16, 2, cg, 1.0, tw, ti)
  assert ti.cpu().tolist() == [[7, 9], [7, 9]] and tw[0].cpu().tolist() == [0.0, 0.0] and bool(torch.isnan(tw[1]).all())


# ---- whole models -----------------------------------------------------------------------------------------
def model_of(name, seed, dtype, gpu):
  d = C.CONFIGS[name]
  w = C.random_weights(d, seed)
  return d, w, StackModel(config.kezolix_from_dict(d), w, gpu, dtype)


TOL = {BF: 0.12, F32: 2e-4}
# bf16 rounding may choose another expert where scores all but tie: whole models in bf16 use every expert
CASES = [(n, F32) for n in sorted(C.CONFIGS)] + [("all", BF), ("wide", BF), ("one", BF)]


@pytest.mark.parametrize("name,dtype", CASES)
def test_prompts_decoding_and_unequal_batches(gpu, name, dtype):
  """Streams of different lengths against the plain implementation: each alone as one prompt, each mostly decoded
  (one from its first token on), and all as one batch."""
  d, w, model = model_of(name, 5, dtype, gpu)
  streams = [C.tokens(d, n, 10 + n) for n in ((140, 41, 33) if name != "one" else (60, 41, 33))]
  want = [R.forward(d, w, s).numpy() for s in streams]
  for i, s in enumerate(streams):
    e = [err(all_logits(model, [s], cut)[0], want[i]) for cut in (0, len(s) - 1 if i == 2 else 30)]
    assert max(e) < TOL[dtype], (i, e)
  e = [err(got, want[i]) for i, got in enumerate(all_logits(model, streams, 32))]
  assert max(e) < TOL[dtype], e


def test_routed_models_in_bf16(gpu):
  """Where rounding may turn a close choice: nearly every position as close as elsewhere."""
  for name in ("mixed", "odd"):
    d, w, model = model_of(name, 4, BF, gpu)
    s = C.tokens(d, 120, 15)
    for cut in (0, 40):
      e = all_logits(model, [s], cut)[0] - R.forward(d, w, s).numpy()
      rows = np.sqrt(((e - e.mean(-1, keepdims=True)) ** 2).mean(-1)) / R.forward(d, w, s).numpy().std()
      assert np.quantile(rows, 0.8) < TOL[BF], (name, cut, np.quantile(rows, [0.5, 0.8, 1.0]))


def test_residual_after_every_layer(gpu):
  for name in sorted(C.CONFIGS):
    d, w, model = model_of(name, 6, F32, gpu)
    toks, want, got = C.tokens(d, 23, 3), [], []
    R.forward(d, w, toks, layers_out=want)
    runner = model.new_runner(1, 23, 23, -1)
    runner.residual_sink = lambda x: got.append(x.cpu().clone())
    runner.forward_hidden(i32([toks], gpu), None, runner.zero, model.new_cache(1, 23))
    assert len(got) == len(want) == len(d["layers"])
    for a, b in zip(got, want):
      assert rel(a, b) < 3e-5


@pytest.mark.parametrize("name,dtype", [("mixed", F32), ("all", BF), ("odd", F32), ("wide", BF)])
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


@pytest.mark.parametrize("name,dtype", [("mixed", F32), ("all", BF)])
def test_long_decoding_across_cache_growth(gpu, name, dtype):
  """Two tokens of prompt, then hundreds of steps over many chunks: the cache grows, borrowed entries with it."""
  d, w, model = model_of(name, 9, dtype, gpu)
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


def test_the_last_position_of_the_table(gpu):
  """A sequence may use every learned position, and no more: as a prompt, decoded, beside a longer row, through the sampler."""
  d, w, model = model_of("one", 3, F32, gpu)
  s = C.tokens(d, 64, 5)
  want = R.forward(d, w, s).numpy()
  assert err(all_logits(model, [s, s[:50]], 8)[0], want) < TOL[F32]
  rp = Replay(model)
  rp.step({"entries": [{"id": "a", "tokens": s, "want": []}, {"id": "b", "tokens": s[:40], "want": []}], "end": ["a"]})
  for t in range(40, 64):
    rp.step({"entries": [{"id": "b", "tokens": [s[t]], "want": []}], "end": []})
  for step in ({"entries": [{"id": "b", "tokens": [1], "want": []}], "end": []}, {"entries": [{"id": "c", "tokens": s + [1], "want": []}], "end": []}):
    with pytest.raises(ValueError, match="64 positions"):
      rp.step(step)
  sampler = Sampler(model, IdTokenizer(d["vocab"], pad_id=0, eos_id=1), CacheConfig(128))
  assert len(sampler([s[:60]], 5, max_prompt_length=64, eos_tokens=[-1]).tokens[0]) == 5
  with pytest.raises(ValueError, match="64 positions"):
    sampler([s[:60]], 6, max_prompt_length=64, eos_tokens=[-1])


@pytest.mark.parametrize("name,dtype", [("mixed", F32), ("all", BF), ("odd", F32), ("wide", BF)])
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


@pytest.mark.parametrize("name,dtype", [("all", BF), ("odd", F32)])
def test_sampling_modes(gpu, name, dtype):
  """top-k 1 is greedy; a seed repeats itself; draws, nucleus and top-k; logits come back."""
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
    assert err(lg, R.forward(d, w, list(p) + list(t)).numpy()[len(p) - 1:-1]) < TOL[dtype]


def test_rollout_log_probabilities_and_weight_updates(gpu):
  """The log-probability pass (a scratch cache, in which what is lent must stay) and new weights through the public calls."""
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
  with pytest.raises(ValueError, match="320 positions"):
    roll.get_per_token_logps(np.full((1, 300), 4), np.full((1, 21), 4))
  w2 = C.random_weights(d, 13)
  before = all_logits(model, [prompts[0]], 2)[0]
  bad = dict(w2)
  bad["l0.mix.f"] = bad["l0.mix.f"][:, :-1]
  with pytest.raises(ValueError, match="same shape"):
    roll.update_params(bad)
  with pytest.raises(ValueError, match="same structure"):
    roll.update_params({"l0.mix.q": w2["l0.mix.q"]})                    # a member of a fused projection without the others
  assert np.array_equal(all_logits(model, [prompts[0]], 2)[0], before)
  for part in ("head", "l0.mix.lower", "l2.dwa", "l4.mix.q.norm", "l4.mix.q", "l1.mlp.e3.up", "l1.mlp.shared.down", "l4.mlp.shared.up", "l1.mlp.correction", "l0.mlp.act", "pos", "embed"):
    w[part] = w2[part]                                                    # alone, one after another
    roll.update_params({part: w2[part]})
    assert err(all_logits(model, [prompts[0]], 2)[0], R.forward(d, w, prompts[0]).numpy()) < TOL[F32], part
  roll.update_params(w2)
  assert err(all_logits(model, [prompts[0]], 2)[0], R.forward(d, w2, prompts[0]).numpy()) < TOL[F32]


@pytest.mark.parametrize("B", [1, 40, 130])
def test_batch_sizes_of_a_decode_step(gpu, B):
  """Every row tile of the few-row kernels: a batch of equal sequences gives every row the same logits."""
  d, w, model = model_of("all", 14, BF, gpu)
  s = C.tokens(d, 12, 70)
  got = all_logits(model, [s] * B, 4)
  want = R.forward(d, w, s).numpy()
  for g in got[:: max(1, B // 5)]:
    assert err(g, want) < TOL[BF]


@pytest.mark.parametrize("name", ["all", "wide"])
def test_a_long_prompt_takes_the_many_row_kernels(gpu, name):
  """More rows than the few-row kernels take: gates apart from queries and values, and the many-row expert kernel."""
  d, w, model = model_of(name, 16, BF, gpu)
  streams = [C.tokens(d, n, 90 + n) for n in (310, 300)]
  for g, s in zip(all_logits(model, streams, 2), streams):
    assert err(g, R.forward(d, w, s).numpy()) < TOL[BF]


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
  z = torch.zeros(64, 128, dtype=F32, device=gpu)
  r = L.ResidualNormDesc()
  r.M, r.D, r.dtype, r.x, r.out, r.out_ld, r.center, r.groups = 2, 64, L.TNX_F32, z.data_ptr(), z.data_ptr(), 128, 1, 2
  with pytest.raises(ValueError, match="one part"):
    ops.residual_norm(r)
  r.groups, r.hist, r.hist_n, r.hist_plane, r.hist_w = 1, z.data_ptr(), 1, 64, z.data_ptr()
  with pytest.raises(ValueError, match="whole planes"):
    ops.residual_norm(r)
  k = L.RowNormKvDesc()
  k.B, k.T, k.S, k.H, k.G, k.dk, k.dv, k.dkp, k.dvp = 1, 1, 8, 3, 2, 16, 16, 16, 16
  with pytest.raises(ValueError, match="bad shape"):
    ops.rownorm_kvwrite(k)
  g = L.GatedStateDesc()
  g.B, g.T, g.H, g.dk, g.dv = 1, 1, 2, 0, 8
  with pytest.raises(ValueError, match="bad shape"):
    ops.gated_state(g)
  s = ops.rows_src(y=z, ld=128)
  with pytest.raises(ValueError, match="bad shape"):
    ops.poly_norm(s, F32, 2, 200, z, 1e-6, z, False)
  with pytest.raises(ValueError, match="outside the row"):
    ops.route_scores(s, 2, 8, 2, None, 1.0, z, z.to(torch.int32), 128, z)
  d = L.DenseDesc()
  d.M, d.K, d.N, d.dtype, d.x, d.ldx, d.w, d.epilogue, d.y, d.ldy, d.split_k, d.ws = 2, 128, 16, L.TNX_BF16, z.data_ptr(), 128, z.data_ptr(), L.TNX_EPI_RELU2, z.data_ptr(), 16, 2, z.data_ptr()
  with pytest.raises(ValueError, match="whole sums"):
    ops.dense_linear(d)
