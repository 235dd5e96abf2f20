"""Lapevik on the GPU against the plain implementation (oracle/lapevik_ref.py): every mechanism alone, then whole
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

from oracle import lapevik_ref as R
from tests import lapevik_cases as C
from tests.test_gpu_nunezen import BF, DTYPES, F32, all_logits, err, frag, i32, rel, rnd, unfrag
from tunix_amd import _lib as L
from tunix_amd import config, ops
from tunix_amd.generate import CacheConfig, Sampler
from tunix_amd.generate.replay import Replay
from tunix_amd.generate.utils import IdTokenizer
from tunix_amd.rl.rollout import HipRollout, RolloutConfig
from tunix_amd.stack_model import DenseLinear, LinearBank, StackModel

pytestmark = pytest.mark.gpu
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))


def source(y, dtype, gpu, split):
  """Rows y [M, N] as a linear leaves them: finished, or in `split` fp32 planes.  (source, what must stay alive)"""
  ld = (y.shape[1] + 15) // 16 * 16
  p = torch.zeros(y.shape[0], ld)
  p[:, :y.shape[1]] = y
  if split > 1:
    keep = torch.stack([p * 0.25, p * 0.75] + [p * 0.0] * (split - 2)).to(gpu).contiguous()
    return ops.rows_src(ws=keep, split_k=split, plane=y.shape[0] * ld, ld=ld), keep
  keep = p.to(dtype).to(gpu)
  return ops.rows_src(y=keep, ld=ld), keep


# ---- norms, shift ---------------------------------------------------------------------------------
class Residual:
  def __init__(self, gpu, dtype, D, groups, B, T, seed=0):
    self.gpu, self.dtype, self.D, self.groups, self.B, self.T, self.eps = gpu, dtype, D, groups, B, T, 0.02
    self.x, self.wp, self.wn = rnd(B * T, D, seed=seed + 1), rnd(D, seed=seed + 2), rnd(D, seed=seed + 3)

  def run(self, mode, src=None, w_next=False, shift=None, route=None, fr=False):
    """shift: (mix, before [B, D], starts, col).  Returns (x, out, before)."""
    gpu, M, D = self.gpu, self.B * self.T, self.D
    x, x2 = self.x.to(gpu), torch.full((M, D), float("nan"), device=gpu)
    out = torch.zeros((M + 127) // 128 * 128, (D + 127) // 128 * 128, dtype=self.dtype, device=gpu)
    wp, wn = self.wp.to(gpu), self.wn.to(gpu)
    d = L.ResidualNormDesc()
    d.M, d.D, d.dtype, d.eps, d.mode, d.groups = M, D, ops.DTYPES[self.dtype], self.eps, mode, self.groups
    if src is not None:
      d.y = src
    d.w_post, d.x, d.out, d.out_ld, d.out_frag = wp.data_ptr(), x.data_ptr(), out.data_ptr(), out.shape[1], int(fr)
    if w_next:
      d.w_next = wn.data_ptr()
    if route is not None:
      rw = route.to(gpu)
      d.route_w, d.route_k = rw.data_ptr(), rw.shape[1]
    before = None
    if shift is not None:
      mix, before, starts, col = shift
      mix, before, st, cp = mix.to(gpu), before.to(gpu), i32(starts, gpu), i32([col], gpu)
      d.shift, d.before, d.starts, d.col_ptr, d.B, d.T = mix.data_ptr(), before.data_ptr(), st.data_ptr(), cp.data_ptr(), self.B, self.T
      if self.T > 1:
        d.x_out = x2.data_ptr()
    ops.residual_norm(d)
    torch.cuda.synchronize()
    got = (unfrag(out, M) if fr else out[:M])[:, :D].float().cpu()
    return (x2 if shift is not None and self.T > 1 else x).cpu(), got, None if before is None else before.cpu()


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("D,groups", [(96, 2), (100, 5), (4096, 16), (2304, 1), (60, 60), (8192, 4)])
def test_norms_in_groups(gpu, dtype, D, groups):
  """x += norm(y), x = norm(x), x = y, each with a next norm and without."""
  r = Residual(gpu, dtype, D, groups, 1, 5)
  y = rnd(5, D, seed=7, scale=3.0).to(dtype).float()
  for mode in (1, 2, 3):
    for split in (1, 3):
      src, keep = source(y, dtype, gpu, split)
      for w_next in (False, True):
        x, out, _ = r.run(mode, src if mode != 3 else None, w_next, fr=dtype == BF and split == 3)
        want = y if mode == 2 else R.group_norm(r.x, r.wp, r.eps, groups) if mode == 3 else r.x + R.group_norm(y, r.wp, r.eps, groups)
        assert rel(x, want) < 1e-6
        assert rel(out, R.group_norm(want, r.wn, r.eps, groups) if w_next else want) < (1e-6 if dtype == F32 else 4e-3)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("D,groups,k", [(128, 2, 3), (100, 4, 1), (64, 1, 8)])
def test_routed_rows_are_summed_with_their_weights(gpu, dtype, D, groups, k):
  r = Residual(gpu, dtype, D, groups, 1, 6)
  y, w = rnd(6 * k, D, seed=5).to(dtype).float(), torch.rand(6, k, generator=torch.Generator().manual_seed(1))
  src, keep = source(y, dtype, gpu, 1)
  x, out, _ = r.run(1, src, route=w)
  want = r.x + R.group_norm((y.view(6, k, D) * w[:, :, None]).sum(1), r.wp, r.eps, groups)
  assert rel(x, want) < 1e-6 and rel(out, want) < (1e-6 if dtype == F32 else 4e-3)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("D,groups,T", [(96, 3, 21), (100, 5, 21), (128, 1, 2), (128, 2, 1), (52, 1, 1), (64, 2, 1400)])
def test_token_shift(gpu, dtype, D, groups, T):
  """Rows of which one begins inside the call, one goes on from an earlier one, one begins with it; the runs of
  a work-group meet inside a sequence."""
  B, col = 3, 10
  starts = [10 + min(7, T - 1), 4, 10]
  r = Residual(gpu, dtype, D, groups, B, T)
  y, mix, before = rnd(B * T, D, seed=5).to(dtype).float(), rnd(D, seed=8), rnd(B, D, seed=9)
  src, keep = source(y, dtype, gpu, 1)
  for mode in (1, 3):
    x, out, kept = r.run(mode, src if mode == 1 else None, shift=(mix, before, starts, col), fr=dtype == BF and T == 1)
    new = R.group_norm(r.x if mode == 3 else y, r.wp, r.eps, groups) + (r.x if mode == 1 else 0.0)
    assert rel(x, new) < 1e-6
    new, got = new.view(B, T, D), out.view(B, T, D)
    for b in range(B):
      lo = max(0, starts[b] - col)
      want = R.token_shift(new[b, lo:], mix, before[b] if starts[b] < col else None)
      assert rel(got[b, lo:], want) < (1e-6 if dtype == F32 else 4e-3), b
    if T == 1:
      assert rel(kept, new[:, 0]) < 1e-6


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("W,groups,split", [(70, 5, 1), (256, 2, 1), (4096, 8, 2), (72, 72, 3), (2048, 1, 1)])
def test_gate_in_front_of_the_norm(gpu, dtype, W, groups, split):
  M, eps = 5, 0.3
  o, w, g = rnd(M, W, seed=1), rnd(W, seed=2), rnd(M, W + 16, seed=3).to(dtype).float()
  src, keep = source(g, dtype, gpu, split)
  og, wg = o.to(gpu), w.to(gpu)
  want = R.group_norm(o * R.silu(g[:, 16:]), w, eps, groups)
  for fr in ([False, True] if dtype == BF else [False]):
    out = torch.zeros(128, (W + 127) // 128 * 128, dtype=dtype, device=gpu)
    d = L.GatedNormDesc()
    d.M, d.W, d.dtype, d.eps, d.gate_first, d.groups = M, W, ops.DTYPES[dtype], eps, 1, groups
    d.o, d.o_ld, d.g, d.g_off, d.w = og.data_ptr(), W, src, 16, wg.data_ptr()
    d.out, d.out_ld, d.out_frag = out.data_ptr(), out.shape[1], int(fr)
    ops.gated_norm(d)
    assert rel((unfrag(out, M) if fr else out[:M])[:, :W], want) < (2e-6 if dtype == F32 else 4e-3)


# ---- experts, batches of projections ----------------------------------------------------------------
def test_choice_of_experts(gpu):
  for E, k, split in ((9, 3, 1), (130, 70, 1), (64, 64, 3), (1, 1, 1), (300, 8, 2)):
    z = rnd(37, E, seed=E, scale=2.0)
    z[3] = 0.25                        # all equal: the first ones
    z[4, -1] = 90.0
    src, keep = source(z, F32, gpu, split)
    w, ids = torch.empty(37, k, device=gpu), torch.empty(37, k, dtype=torch.int32, device=gpu)
    ops.route_softmax(src, 37, E, k, w, ids)
    val, idx = torch.sort(z, dim=-1, descending=True, stable=True)
    assert torch.equal(ids.cpu().long(), idx[:, :k])
    torch.testing.assert_close(w.cpu(), torch.softmax(val[:, :k], -1), rtol=2e-5, atol=1e-6)
  z = rnd(2, 8)
  z[0, 3] = float("nan")
  src, keep = source(z, F32, gpu, 1)
  w, ids = torch.empty(2, 4, device=gpu), torch.empty(2, 4, dtype=torch.int32, device=gpu)
  ops.route_softmax(src, 2, 8, 4, w, ids)
  assert len(set(ids[0].tolist())) == 4 and not set(ids[0].tolist()) - set(range(8))
  assert torch.isnan(w[0]).all() and torch.isfinite(w[1]).all()


@pytest.mark.parametrize("M,k,E", [(1, 1, 1), (1, 3, 9), (32, 8, 64), (37, 5, 130), (128, 8, 512), (700, 6, 7), (4099, 8, 64), (20000, 4, 100), (50, 2, 600)])
def test_routes_sorted_by_expert(gpu, M, k, E):
  """Stable: an expert's routes in increasing order; experts without a route, and one with most of them."""
  g = torch.Generator().manual_seed(M)
  ids = torch.randint(0, E, (M, k), generator=g)
  ids[torch.rand(M, k, generator=g) < 0.4] = E // 2
  counts, offsets, order = (torch.full((n,), -7, dtype=torch.int32, device=gpu) for n in (E, E + 1, M * k))
  ops.moe_sort_routes(ids.int().to(gpu), E, counts, offsets, order)
  flat = ids.reshape(-1)
  want = torch.bincount(flat, minlength=E)
  assert torch.equal(counts.cpu().long(), want) and torch.equal(order.cpu().long(), torch.sort(flat, stable=True).indices)
  assert offsets[0] == 0 and torch.equal(offsets[1:].cpu().long(), torch.cumsum(want, 0))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("M,K,F,E,k", [(1, 64, 40, 3, 2), (5, 100, 33, 6, 6), (70, 128, 256, 8, 3), (300, 256, 96, 5, 2), (700, 128, 272, 3, 1)])
def test_experts(gpu, dtype, M, K, F, E, k):
  """gate | up and down of routed rows: few rows per expert (row-major and fragment order), the many-row kernel, fp32;
  one expert gets no row, one gets most."""
  g = torch.Generator().manual_seed(M)
  w = {f"{n}{e}": (torch.randn(*s, generator=g) * s[1] ** -0.5).to(BF) for e in range(E) for n, s in (("g", (F, K)), ("u", (F, K)), ("d", (K, F)))}
  x = torch.randn(M, K, generator=g).to(dtype)
  z = torch.randn(M, E, generator=g)
  z[:, 0] += 3.0
  if E > k:
    z[:, 1] = -50.0
  ids = torch.topk(z, k).indices.int()
  gu = LinearBank([DenseLinear([f"g{e}", f"u{e}"], w, dtype, gpu, paired=True) for e in range(E)])
  dn = LinearBank([DenseLinear([f"d{e}"], w, dtype, gpu) for e in range(E)])
  counts, offsets, order = (torch.empty(n, dtype=torch.int32, device=gpu) for n in (E, E + 1, M * k))
  ops.moe_sort_routes(ids.to(gpu), E, counts, offsets, order)

  def call(f, inp, fr, div, epi, out):
    d = L.DenseDesc()
    d.M, d.K, d.N, d.dtype, d.x, d.ldx, d.x_frag = M * k, f.Kp, f.N, ops.DTYPES[dtype], inp.data_ptr(), inp.shape[1], int(fr)
    d.w, d.w_stride, d.epilogue, d.y, d.ldy, d.split_k = f.w.data_ptr(), f.stride, epi, out.data_ptr(), out.shape[1], 1
    d.n_experts, d.x_div, d.offsets, d.sorted_route = E, div, offsets.data_ptr(), order.data_ptr()
    ops.dense_linear(d)

  xp = torch.zeros(M, gu.Kp, dtype=dtype, device=gpu)
  xp[:, :K] = x.to(gpu)
  flat = ids.reshape(-1).tolist()
  act_want = torch.stack([R.silu(x[r // k].double() @ w[f"g{e}"].double().T) * (x[r // k].double() @ w[f"u{e}"].double().T) for r, e in enumerate(flat)])
  for fr in ([False, True] if dtype == BF else [False]):
    act = torch.zeros(M * k, dn.Kp, dtype=dtype, device=gpu)
    if dtype == F32:
      y = torch.full((M * k, gu.N), float("nan"), device=gpu)
      call(gu, xp, False, k, L.TNX_EPI_STORE, y)
      ops.silu_mul(y, gu.offsets[1], M * k, F, act)
    else:
      call(gu, frag(xp) if fr else xp, fr, k, L.TNX_EPI_SILU_MUL, act)
    assert rel(act[:, :F], act_want) < (2e-6 if dtype == F32 else 4e-3) and not act[:, (F + 15) // 16 * 16:].any()
  out = torch.full((M * k, dn.N), float("nan"), dtype=dtype, device=gpu)
  call(dn, act, False, 1, L.TNX_EPI_STORE, out)
  want = torch.stack([act[r, :F].double().cpu() @ w[f"d{e}"].double().T for r, e in enumerate(flat)])
  assert rel(out[:, :K], want) < (2e-6 if dtype == F32 else 4e-3)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("M,H,n,rank", [(1, 3, 21, 50), (40, 5, 32, 80), (130, 2, 128, 512)])
def test_a_projection_per_head(gpu, dtype, M, H, n, rank):
  """Each head's columns through its own (transposed) rows of one weight."""
  w = {"k": (rnd(H * n, rank, seed=1) * n ** -0.5).to(BF)}
  f = LinearBank([DenseLinear([("k", h * n, (h + 1) * n)], w, dtype, gpu, transpose=True) for h in range(H)])
  x = rnd(M, H, n, seed=2).to(dtype)
  xp = torch.zeros(M, H, f.Kp, dtype=dtype, device=gpu)
  xp[:, :, :n] = x.to(gpu)
  y = torch.zeros(M, H, f.N + 8, dtype=dtype, device=gpu)
  d = L.DenseDesc()
  d.M, d.K, d.N, d.dtype, d.x, d.ldx, d.x_stride = M, f.Kp, f.N, ops.DTYPES[dtype], xp.data_ptr(), H * f.Kp, f.Kp
  d.w, d.w_stride, d.y, d.ldy, d.y_stride, d.split_k, d.batch = f.w.data_ptr(), f.stride, y.data_ptr(), H * (f.N + 8), f.N + 8, 1, H
  ops.dense_linear(d)
  want = torch.stack([x[:, h].double() @ w["k"][h * n:(h + 1) * n].double() for h in range(H)], 1)
  assert rel(y[:, :, :rank], want) < (2e-6 if dtype == F32 else 4e-3) and not y[:, :, f.N:].any()


# ---- convolution and recurrence -----------------------------------------------------------------------
class Ssd:
  """One layer's kernels over a batch; `cut` runs its columns in portions."""

  def __init__(self, gpu, dtype, H, P, N, G, taps, S, starts, seed=0, A=None, dt_bias=None):
    self.gpu, self.dtype, self.H, self.P, self.N, self.G, self.taps, self.S = gpu, dtype, H, P, N, G, taps, S
    self.starts, self.B, self.inner, self.C = list(starts), len(starts), H * P, H * P + 2 * G * N
    self.u = rnd(self.B, S, self.C, seed=seed + 1).to(BF).float()
    self.dt = rnd(self.B, S, H, seed=seed + 2).to(BF).float()
    self.w, self.bias = rnd(self.C, taps, seed=seed + 3) * taps ** -0.5, rnd(self.C, seed=seed + 4, scale=0.3)
    self.A = rnd(H, seed=seed + 5) - 1.0 if A is None else torch.tensor(A)
    self.dt_bias = rnd(H, seed=seed + 6) - 1.0 if dt_bias is None else torch.tensor(dt_bias)
    self.D = rnd(H, seed=seed + 7)
    # what another sequence has left: a new one must not see it
    self.state = torch.full((self.B, H, N, P), 7.0, device=gpu)
    self.ring = torch.full((self.B, taps, self.C), 5.0, dtype=dtype, device=gpu)
    self.conv_out = None

  def run(self, col, T, split=1, step=True):
    gpu, B, H = self.gpu, self.B, self.H
    up = lambda n: (n + 15) // 16 * 16
    dto = up(self.C)
    y = torch.zeros(B, T, dto + H)
    y[:, :, :self.C], y[:, :, dto:] = self.u[:, col:col + T], self.dt[:, col:col + T]
    src, keep = source(y.view(B * T, -1), self.dtype, gpu, split)
    st, cp, code = i32(self.starts, gpu), i32([col], gpu), ops.DTYPES[self.dtype]
    dev = [t.to(gpu).contiguous() for t in (self.w.T, self.bias, self.A, self.dt_bias, self.D)]
    o = torch.full((B * T, self.inner), float("nan"), device=gpu)
    d = L.SsdDesc()
    d.B, d.T, d.H, d.G, d.N, d.P, d.dtype, d.y, d.dt_off = B, T, H, self.G, self.N, self.P, code, src, dto
    if not (step and T == 1 and ops.ssd_step_ok(self.N, self.P)):
      out = torch.full((B * T, (self.C + 7) // 8 * 8), float("nan"), dtype=self.dtype, device=gpu)
      c = L.ShortConvDesc()
      c.B, c.T, c.C, c.taps, c.slots, c.dtype, c.y = B, T, self.C, self.taps, self.taps, code, src
      c.w, c.bias, c.ring, c.starts, c.col_ptr = dev[0].data_ptr(), dev[1].data_ptr(), self.ring.data_ptr(), st.data_ptr(), cp.data_ptr()
      c.out, c.out_ld = out.data_ptr(), out.shape[1]
      ops.short_conv(c)
      ops.ring_write(src, 0, B, T, cp, self.ring)
      d.u, d.u_ld = out.data_ptr(), out.shape[1]
      self.conv_out = out[:, :self.C].float().cpu().view(B, T, self.C)
    d.taps, d.slots, d.conv_w, d.conv_b, d.ring = self.taps, self.taps, dev[0].data_ptr(), dev[1].data_ptr(), self.ring.data_ptr()
    d.A_log, d.dt_bias, d.D = (t.data_ptr() for t in dev[2:])
    ws = torch.empty(max(1, ops.ssd_ws_bytes(B, T, H, self.G, self.N, self.P) // 4), device=gpu)
    d.starts, d.col_ptr, d.state, d.o, d.o_ld, d.ws = st.data_ptr(), cp.data_ptr(), self.state.data_ptr(), o.data_ptr(), self.inner, ws.data_ptr()
    ops.ssd(d)
    torch.cuda.synchronize()
    return o.cpu().view(B, T, H, self.P)

  def reference(self):
    """(convolved rows, outputs, states) of every row's sequence."""
    if not hasattr(self, "_ref"):
      self._ref = []
      for b, s in enumerate(self.starts):
        u = R.silu(R.short_conv(self.u[b, s:], self.w, self.bias))
        v = u.to(BF).float() if self.dtype == BF else u
        T, gn = v.shape[0], self.G * self.N
        args = (v[:, :self.inner].view(T, self.H, self.P).double(), v[:, self.inner:self.inner + gn].view(T, self.G, self.N).double(),
                v[:, self.inner + gn:].view(T, self.G, self.N).double(), R.softplus(self.dt[b, s:] + self.dt_bias).double(), self.A.double(), self.D.double())
        self._ref.append((u, R.ssd_recurrence(*args)))
    return self._ref

  def check(self, got, col, conv=False):
    T = got.shape[1]
    for b, s0 in enumerate(self.starts):
      s = max(s0, col)
      if s >= col + T:
        continue
      u, (o, S) = self.reference()[b]
      e = [rel(got[b, s - col:], o[s - s0:col + T - s0])]
      if conv:
        e.append(rel(self.conv_out[b, s - col:], u[s - s0:col + T - s0]))
      if col + T == self.S:
        e.append(rel(self.state[b], S))
      # (one token at a time x, B and C stay fp32 behind their activation, in a prompt they are rounded)
      assert max(e) < (2e-5 if self.dtype == F32 else 2.5e-2 if T == 1 else 5e-3), (b, col, T, e)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,P,N,G,taps", [(4, 32, 16, 2, 4), (2, 64, 128, 1, 4), (3, 20, 12, 3, 3), (4, 10, 7, 2, 5), (6, 24, 40, 2, 2), (1, 136, 160, 1, 1)])
def test_recurrence_prompt_portions_and_steps(gpu, dtype, H, P, N, G, taps):
  """One pass (cut into spans that run in parallel), portions from two tokens up, token by token, over rows with
  different starts; finished rows and partial planes; the step kernel and convolved single tokens."""
  S = 210
  a = Ssd(gpu, dtype, H, P, N, G, taps, S, [0, 70, 129, 209], seed=H)
  a.check(a.run(0, S), 0, conv=True)
  a.state.fill_(-3.0), a.ring.fill_(-9.0)
  col = 0
  for T in (64, 2, 3, 63, 2):
    a.check(a.run(col, T, split=2 if T == 3 else 1), col, conv=True)
    col += T
  for t in range(col, S):
    a.check(a.run(t, 1, split=2 if t % 2 else 1, step=t % 5 != 0), t)
  b = Ssd(gpu, dtype, H, P, N, G, taps, 20, [0, 5], seed=9)
  for t in range(20):
    b.check(b.run(t, 1), t)


def test_recurrence_remembers_and_forgets(gpu):
  """One input far back: without decay it returns whole after hundreds of tokens, with a fast one it is gone; the last
  token of a chunk and the first of the next are the same to it."""
  S, n = 420, 32
  for at in (0, 63, 64, 127, 128, 300):
    a = Ssd(gpu, BF, 3, 32, n, 1, 2, S, [0], A=[-30.0, 6.0, math.log(0.02)], dt_bias=[0.0, 0.0, 0.0])
    a.w[:], a.bias[:], a.D[:], a.dt[:] = 0.0, 0.0, 0.0, math.log(math.e - 1)       # softplus = 1
    a.w[:, 1] = 1.0
    a.u[:] = -20.0                                                                 # silu(-20) = 0 to bf16
    a.u[:, :, a.inner + n:] = 1.0                                                  # C
    a.u[0, at, :a.inner + n] = 2.0                                                 # x and B of one token
    got = a.run(0, S)[0]
    silu = lambda z: z / (1 + math.exp(-z))
    full = n * silu(1.0) * silu(2.0) ** 2
    for h, lam in enumerate((1.0, 0.0, math.exp(-0.02))):
      for t in (at, at + 1, S - 1):
        want = full * lam ** (t - at)
        assert abs(float(got[t, h, 5]) - want) < 1.5e-2 * full, (at, h, t, float(got[t, h, 5]), want)
      assert at == 0 or float(got[:at, h].abs().max()) < 1e-3


# ---- latent attention -----------------------------------------------------------------------------------
class Latent:
  """One layer's kernels behind its projections, over a batch."""

  def __init__(self, gpu, dtype, H, n, r, vd, q_rank, rank, S, starts, scale=None, base=1000.0, seed=0, sharp=1.0):
    self.gpu, self.dtype, self.S, self.starts, self.B = gpu, dtype, S, list(starts), len(starts)
    m = config.LatentMixer(H, n, r, vd, q_rank, rank, base, (n + r) ** -0.5 if scale is None else scale)
    self.m = m
    g = torch.Generator().manual_seed(seed)
    D = 64
    w = {"l0.mix." + k: (torch.randn(*s, generator=g) * (s[1] ** -0.5 if len(s) == 2 else 1.0)).to(BF) for k, s in m.weight_shapes(D).items()}
    w["l0.mix.uq"] = w["l0.mix.uq"] * sharp
    cfg = config.StackConfig("lapevik", 64, D, (config.LayerSpec(m, None),), 1e-5, norm_offset=0.0, pre_norm=False, embed_norm=True, token_shift=True)
    full = {k: torch.randn(*s, generator=g).to(BF) for k, s in cfg.weight_shapes().items()}
    full.update(w)
    self.w, self.model = {k: v.float() for k, v in full.items()}, StackModel(cfg, full, gpu, dtype)
    self.src_rows = torch.randn(self.B, S, m.q_rank + rank + r + H * vd, generator=g).to(BF).float()    # dq | dkv | g
    self.cache = self.model.new_cache(self.B, S)
    self.cache.entries[0]["mixer"].c.fill_(3.0)         # another sequence's rows

  def run(self, col, T, prompt=False, split=1, kv_chunk=None):
    """Gated heads of the portion [col, col + T): [B, T, H * vd]."""
    m, B = self.m, self.B
    ly, offs = self.model.layers[0], self.model.layers[0]["in"].offsets
    r = self.model.new_runner(B, T, self.S, -1)
    if kv_chunk is not None:
      r._latent_chunk = lambda _: kv_chunk
      r.attn_ws = torch.empty(max(1, ops.latent_attn_ws_bytes(B, T, self.S, m.heads, m.kv_rank, kv_chunk) // 4), device=self.gpu)
    y = torch.zeros(B, T, offs[2] + m.heads * m.vdim)
    part, cut = self.src_rows[:, col:col + T], (m.q_rank, m.kv_rank + m.rot_dim)
    y[:, :, :cut[0]], y[:, :, offs[1]:offs[1] + cut[1]], y[:, :, offs[2]:] = part[:, :, :cut[0]], part[:, :, cut[0]:sum(cut)], part[:, :, sum(cut):]
    src, keep = source(y.view(B * T, -1), self.dtype, self.gpu, split)
    at = (self.cache.entries[0]["mixer"], r.zero if prompt else i32([col], self.gpu), i32(self.starts, self.gpu), B, T)
    cq, ckv = r.latent_prep(ly, src, *at, expand=prompt)
    heads, y_head = r.latent_prompt(ly, cq, ckv, *at) if prompt else r.latent_rows(ly, cq, *at)
    out = r.gate_mul(ly, heads, m.vdim, y_head, src, B * T)
    torch.cuda.synchronize()
    out = unfrag(out, B * T) if r.frag else out[:B * T]
    return out[:, :m.heads * m.vdim].float().cpu().view(B, T, -1)

  def want(self, b):
    m, s, w = self.m, self.starts[b], self.w
    rows, T = self.src_rows[b, s:], self.S - s
    rd = lambda t: t.to(BF).float() if self.dtype == BF else t
    cq = rd(R.group_norm(rows[:, :m.q_rank], w["l0.mix.dq.norm"], 1e-5))
    c = rd(R.group_norm(rows[:, m.q_rank:m.q_rank + m.kv_rank], w["l0.mix.dkv.norm"], 1e-5))
    pos = torch.arange(T)
    kr = R.rotate_interleaved(rows[:, m.q_rank + m.kv_rank:m.q_rank + m.kv_rank + m.rot_dim], pos, m.rot_base)
    q = (cq @ w["l0.mix.uq"].T).view(T, m.heads, -1)
    q = torch.cat([q[..., :m.dim], R.rotate_interleaved(q[..., m.dim:], pos, m.rot_base)], -1)
    k = torch.cat([(c @ w["l0.mix.uk"].T).view(T, m.heads, m.dim), kr[:, None].expand(T, m.heads, m.rot_dim)], -1)
    o = R.causal_attention(q, k, (c @ w["l0.mix.uv"].T).view(T, m.heads, m.vdim), m.scale).reshape(T, -1)
    return o * torch.sigmoid(rows[:, m.q_rank + m.kv_rank + m.rot_dim:])

  def check(self, got, col):
    T = got.shape[1]
    for b in range(self.B):
      s = max(self.starts[b], col)
      if s < col + T:
        if not hasattr(self, "_want"):
          self._want = [self.want(i) for i in range(self.B)]
        w = self._want[b][s - self.starts[b]:col + T - self.starts[b]]
        assert torch.isfinite(got[b, s - col:]).all()
        e = float((got[b, s - col:] - w).abs().max() / w.abs().max())
        assert e < (3e-5 if self.dtype == F32 else 3e-2), (b, col, T, e)


LATENTS = [(5, 32, 16, 48, 64, 80), (3, 21, 6, 45, 37, 50), (3, 128, 64, 128, 160, 320), (2, 96, 32, 200, 64, 224), (2, 64, 64, 64, 32, 256),
           (1, 32, 0, 32, 32, 600), (40, 32, 64, 32, 48, 512), (2, 200, 100, 300, 16, 64)]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,n,r,vd,q_rank,rank", LATENTS)
def test_latent_attention_prompt_portions_and_steps(gpu, dtype, H, n, r, vd, q_rank, rank):
  """A prompt through expanded keys and values, then in portions and token by token through the cache rows; rows with
  different starts, finished rows and partial planes, a split key range and none."""
  S = 300
  a = Latent(gpu, dtype, H, n, r, vd, q_rank, rank, S, [0, 137, 299], seed=H, sharp=2.0)
  a.check(a.run(0, S, prompt=True), 0)
  a.cache.entries[0]["mixer"].c.fill_(-2.0)
  col = 0
  for T in (64, 2, 63, 3, 126):
    a.check(a.run(col, T, split=2 if T == 3 else 1), col)
    col += T
  for t in list(range(col, 262)) + list(range(296, S)):
    if t == 296:
      a.check(a.run(262, 34), 262)
    a.check(a.run(t, 1, split=3 if t % 3 == 0 else 1, kv_chunk=128 if t % 2 else 0), t)


@pytest.mark.parametrize("how", ["prompt", "rows", "decoded", "chunks"])
@pytest.mark.parametrize("far", [0, 63, 64, 127, 128, 255, 256, 298, 299])
def test_one_latent_stands_out(gpu, how, far):
  """A single position far above the others, at tile and chunk borders and at both ends of the visible range, takes
  the weight; the one behind the query, higher still and in the cache, is not seen."""
  S, m = 400, (2, 32, 16, 32, 32, 64)
  a = Latent(gpu, BF, *m, S, [0], seed=far, base=1e9)
  rank, n, r, vd, w = 64, 32, 16, 32, a.w
  for h in range(2):       # keys of a head: the first 32 of the latent; values: the last 32
    w["l0.mix.uk"][h * n:(h + 1) * n] = torch.eye(n, rank)
    w["l0.mix.uv"][h * vd:(h + 1) * vd] = torch.roll(torch.eye(vd, rank), 32, 1)
  w["l0.mix.dq.norm"][:], w["l0.mix.dkv.norm"][:] = 1.0, 1.0
  w["l0.mix.uq"] = torch.zeros_like(w["l0.mix.uq"])
  for h in range(2):       # queries: the first direction, 60 times
    w["l0.mix.uq"][h * (n + r), 0] = 60.0
  a.model.update_params({k: w[k] for k in ("l0.mix.uk", "l0.mix.uv", "l0.mix.uq", "l0.mix.dq.norm", "l0.mix.dkv.norm")})
  rows = a.src_rows
  rows[:, :, 0] = 2.0                            # the query's direction
  rows[:, :, 32] = 0.0                           # every key is flat in it ...
  rows[0, far, 32], rows[0, 300, 32] = 4.0, 9.0  # ... but two
  rows[:, :, 32 + rank + r:] = 30.0              # an open gate
  got = a.run(0, S, prompt=how == "prompt")[0, 299]
  if how == "decoded":
    got = a.run(299, 1, kv_chunk=0)[0, 0]
  elif how == "chunks":
    got = a.run(299, 1, kv_chunk=128)[0, 0]
  c = R.group_norm(rows[0, far, 32:32 + rank], torch.ones(rank), 1e-5)
  assert float((got.view(2, vd) - c[32:]).abs().max()) < 3e-2


# ---- whole models -----------------------------------------------------------------------------------------
def model_of(name, seed, dtype, gpu):
  d = C.CONFIGS[name]
  w = C.random_weights(d, seed)
  return d, w, StackModel(config.lapevik_from_dict(d), w, gpu, dtype)


# bf16 rounding through up to eight sublayers with sharp scores: a single row can be several times off the rest
TOL = {BF: 0.25, F32: 2e-4}


def close(d, got, want, dtype):
  """Every row; in bf16 and with routers that choose, most rows: one whose router decides between two close logits
  may take another expert than in exact arithmetic, and rows behind it read what it left."""
  e = got - want
  e = e - e.mean(-1, keepdims=True)
  rows = np.sort(np.sqrt((e ** 2).mean(-1)) / want.std())
  n = len(rows)
  if dtype == F32:
    return rows[-1] < TOL[F32]
  chooses = any(ly["mlp"] and ly["mlp"]["router"]["top"] < ly["mlp"]["router"]["experts"] for ly in d["layers"])
  return rows[n // 2] < 0.3 * TOL[BF] and rows[int(0.75 * (n - 1)) if chooses else -1] < TOL[BF]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", sorted(C.CONFIGS))
def test_prompts_decoding_and_unequal_batches(gpu, name, dtype):
  """Streams of different lengths against the plain implementation: each alone as one prompt, each mostly decoded
  (one from its first token on), and all as one batch."""
  d, w, model = model_of(name, 5, dtype, gpu)
  streams = [C.tokens(d, n, 10 + n) for n in (140, 41, 33)]
  want = [R.forward(d, w, s).numpy() for s in streams]
  for i, s in enumerate(streams):
    for cut in (0, len(s) - 1 if i == 2 else 30):
      assert close(d, all_logits(model, [s], cut)[0], want[i], dtype), (i, cut)
  for i, got in enumerate(all_logits(model, streams, 32)):
    assert close(d, got, want[i], dtype), i


def test_residual_after_every_layer(gpu):
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


@pytest.mark.parametrize("name,dtype", [("all", BF), ("mixed", F32), ("odd", F32)])
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
    assert close(d, lg.cpu().numpy(), R.forward(d, w, s).numpy(), dtype)


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
    h = [r.forward_hidden(toks, None, r.zero, cache, starts=starts).view(2, 60, -1)[0].clone()]
    r1 = model.new_runner(2, 1, 96, -1)
    for t in range(60, 70):
      h.append(r1.forward_hidden(toks, None, i32([t], gpu), cache, starts=starts).clone())
    out.append(torch.cat(h))
  assert torch.equal(out[0], out[1])


def test_long_decoding_across_cache_growth(gpu):
  """Two tokens of prompt, then hundreds of steps: the cache grows, states and rings are carried all the way."""
  d, w, model = model_of("mixed", 9, F32, gpu)
  s = C.tokens(d, 280, 40)
  assert close(d, all_logits(model, [s], 278)[0], R.forward(d, w, s).numpy(), F32)


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
    assert close(d, np.stack(got[r]), R.forward(d, w, s).numpy()[len(s) - len(got[r]):], F32)


@pytest.mark.parametrize("name,dtype", [("all", BF), ("odd", F32), ("mixed", F32)])
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
    spread, rows = float(lg.std()), torch.arange(40)
    pick = lg[rows, torch.tensor(t.astype(np.int64))]
    gap = np.sort((lg.max(-1).values - pick).numpy())
    want = torch.log_softmax(lg, -1)[rows, torch.tensor(t.astype(np.int64))]
    off = np.sort((torch.tensor(lp).double() - want).abs().numpy())
    if dtype == F32:
      assert gap[-1] < 1e-3 * spread and off[-1] < 1e-3 * spread
    else:
      assert gap[-1] < 0.4 * spread and off[-1] < 0.5 * spread


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
  bad["l0.mix.uk"] = bad["l0.mix.uk"][:, :-1]
  with pytest.raises(ValueError, match="same shape"):
    roll.update_params(bad)
  with pytest.raises(ValueError, match="same structure"):
    roll.update_params({"l0.mlp.e1.gate": w2["l0.mlp.e1.gate"]})        # an expert's gate without its up
  assert np.array_equal(all_logits(model, [prompts[0]], 2)[0], before)
  roll.update_params(w2)
  assert close(d, all_logits(model, [prompts[0]], 2)[0], R.forward(d, w2, prompts[0]).numpy(), F32)


@pytest.mark.parametrize("B", [1, 40, 130])
def test_batch_sizes_of_a_decode_step(gpu, B):
  """Every row tile of the few-row kernels: a batch of equal sequences gives every row the same logits."""
  d, w, model = model_of("all", 14, BF, gpu)
  s = C.tokens(d, 12, 70)
  got = all_logits(model, [s] * B, 4)
  want = R.forward(d, w, s).numpy()
  for g in got[:: max(1, B // 5)]:
    assert close(d, g, want, BF)


def test_a_long_prompt_takes_the_many_row_kernels(gpu):
  """More rows than the few-row kernels take: the expert and dense kernels of prompts."""
  d, w, model = model_of("all", 16, BF, gpu)
  streams = [C.tokens(d, n, 90 + n) for n in (330, 300)]
  for g, s in zip(all_logits(model, streams, 2), streams):
    assert close(d, g, R.forward(d, w, s).numpy(), BF)


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
  s = L.SsdDesc()
  s.B, s.T, s.H, s.G, s.N, s.P = 1, 1, 3, 2, 8, 8
  with pytest.raises(ValueError, match="bad shape"):
    ops.ssd(s)
  a = L.LatentAttnDesc()
  a.B, a.T, a.S, a.H, a.rank, a.row = 1, 1, 8, 2, 64, 96
  with pytest.raises(ValueError, match="no kernel"):
    ops.latent_attn(a)
  q = L.LatentQDesc()
  q.B, q.T, q.H, q.n, q.r, q.un_pad, q.rot_pad = 1, 1, 2, 8, 4, 4, 4
  with pytest.raises(ValueError, match="short heads"):
    ops.latent_q(q)
  z = torch.zeros(64, 128, dtype=BF, device=gpu)
  d = L.DenseDesc()
  d.M, d.K, d.N, d.x, d.w, d.y, d.ldx, d.ldy, d.split_k = 1, 128, 16, z.data_ptr(), z.data_ptr(), z.data_ptr(), 128, 16, 1
  d.n_experts = 2
  with pytest.raises(ValueError, match="sorted routes"):
    ops.dense_linear(d)
  r = L.ResidualNormDesc()
  r.M, r.D, r.x, r.out, r.out_ld, r.groups = 1, 100, z.data_ptr(), z.data_ptr(), 128, 3
  with pytest.raises(ValueError, match="does not divide"):
    ops.residual_norm(r)
