"""Nunezen on the GPU against the plain implementation (oracle/nunezen_ref.py): every mechanism alone,
then whole models -- prompts, token-by-token decoding, portions, unequal batches, reused slots, greedy
generation -- in bf16 and in fp32, at sizes that reach every kernel."""
import json
import math
import os
import subprocess
import sys

import numpy as np
import pytest
import torch

from oracle import nunezen_ref as R
from tests import nunezen_cases as C
from tunix_amd import _lib as L
from tunix_amd import config, ops
from tunix_amd.generate import CacheConfig, Sampler
from tunix_amd.generate.replay import Replay
from tunix_amd.generate.utils import IdTokenizer
from tunix_amd.rl import common
from tunix_amd.rl.rollout import HipRollout, RolloutConfig
from tunix_amd.stack_model import DenseLinear, StackModel

pytestmark = pytest.mark.gpu
BF, F32 = torch.bfloat16, torch.float32
DTYPES = [BF, F32]
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))


def rnd(*shape, seed=0, scale=1.0):
  return torch.randn(*shape, generator=torch.Generator().manual_seed(seed + 1000 * len(shape) + sum(shape))) * scale


def i32(x, gpu):
  return torch.tensor(x, dtype=torch.int32, device=gpu)


def rel(a, b):
  return float((a.float().cpu() - b).norm() / b.norm().clamp_min(1e-9))


def frag(x):
  """[M, K] -> the fragment order, whole blocks of 128 rows (zeros behind)."""
  M, K = x.shape
  p = torch.zeros((M + 127) // 128 * 128, K, dtype=x.dtype, device=x.device)
  p[:M] = x
  return p.view(-1, 32, K // 16, 2, 8).permute(0, 2, 3, 1, 4).contiguous().view(p.shape)


def unfrag(y, M):
  rows, K = y.shape
  return y.view(rows // 32, K // 16, 2, 32, 8).permute(0, 3, 1, 2, 4).reshape(rows, K)[:M]


# ---- linears ------------------------------------------------------------------------------------
def run_linear(f, x, M, out, epilogue=L.TNX_EPI_STORE, x_frag=False, y_frag=False, split=1, ws=None, N=None):
  d = L.DenseDesc()
  d.M, d.K, d.N, d.dtype = M, f.Kp, f.N if N is None else N, ops.DTYPES[f.dtype]
  d.x, d.ldx, d.x_frag, d.w, d.epilogue = x.data_ptr(), x.shape[1], int(x_frag), f.w.data_ptr(), epilogue
  d.y, d.ldy, d.y_frag, d.split_k = out.data_ptr(), out.shape[-1], int(y_frag), split
  d.ws = ws.data_ptr() if ws is not None else None
  ops.dense_linear(d)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("M,K,N", [(1, 100, 48), (33, 128, 211), (65, 320, 96), (129, 1000, 272), (700, 256, 528)])
def test_dense_linear(gpu, dtype, M, K, N):
  """Few-row kernel (row-major and fragment-order rows, k splits), many-row kernel, fp32 kernel; a width
  that is no multiple of 16 through the fp32-result form."""
  w, x = rnd(N, K, seed=1).to(BF), rnd(M, K, seed=2).to(dtype)
  want = x.double() @ w.double().T
  f = DenseLinear(["w"], {"w": w}, dtype, gpu)
  xp = torch.zeros(M, f.Kp, dtype=dtype, device=gpu)
  xp[:, :K] = x.to(gpu)
  tol = 2e-6 if dtype == F32 else 4e-3
  y = torch.full((M, f.N), float("nan"), dtype=dtype, device=gpu)
  run_linear(f, xp, M, y)
  assert rel(y[:, :N], want) < tol
  y = torch.full((M, N), float("nan"), dtype=F32, device=gpu)
  run_linear(f, xp, M, y, L.TNX_EPI_F32, N=N)
  assert rel(y, want) < 2e-6
  if dtype == F32:
    return
  y = torch.full(((M + 127) // 128 * 128, (f.N + 15) // 16 * 16), float("nan"), dtype=BF, device=gpu)
  run_linear(f, frag(xp), M, y, x_frag=True, y_frag=True)
  assert rel(unfrag(y, M)[:, :N], want) < tol
  for split in (2, 3):
    ws = torch.full((split, M, f.N), float("nan"), device=gpu)
    run_linear(f, frag(xp), M, ws, L.TNX_EPI_F32, x_frag=True, split=split, ws=ws)
    assert rel(ws.sum(0)[:, :N], want) < 2e-6


@pytest.mark.parametrize("M,K,F", [(2, 64, 40), (100, 256, 96), (600, 128, 272)])
def test_gated_unit(gpu, M, K, F):
  wg, wu, x = rnd(F, K, seed=1, scale=K ** -0.5).to(BF), rnd(F, K, seed=2).to(BF), rnd(M, K, seed=3).to(BF)
  want = R.gelu_tanh(x.double() @ wg.double().T) * (x.double() @ wu.double().T)
  f = DenseLinear(["g", "u"], {"g": wg, "u": wu}, BF, gpu, paired=True)
  xp = torch.zeros(M, f.Kp, dtype=BF, device=gpu)
  xp[:, :K] = x.to(gpu)
  ld = (F + 127) // 128 * 128
  y = torch.zeros(M, ld, dtype=BF, device=gpu)
  run_linear(f, xp, M, y, L.TNX_EPI_GELU_MUL)
  assert rel(y[:, :F], want) < 4e-3 and not y[:, F:].any()
  y = torch.zeros((M + 127) // 128 * 128, ld, dtype=BF, device=gpu)
  run_linear(f, frag(xp), M, y, L.TNX_EPI_GELU_MUL, x_frag=True, y_frag=True)
  assert rel(unfrag(y, M)[:, :F], want) < 4e-3
  f32 = DenseLinear(["g", "u"], {"g": wg, "u": wu}, F32, gpu, paired=True)
  y = torch.empty(M, f32.N, device=gpu)
  run_linear(f32, xp.float(), M, y)
  out = torch.zeros(M, ld, device=gpu)
  ops.gelu_mul(y, f32.offsets[1], M, F, out)
  assert rel(out[:, :F], want) < 3e-6


# ---- embedding, norms ---------------------------------------------------------------------------
@pytest.mark.parametrize("dtype", DTYPES)
def test_embed_rows(gpu, dtype):
  V, D, B, T = 37, 52, 3, 4
  table = rnd(V, D).to(BF).to(dtype)
  ids = torch.randint(0, V, (B, 9), generator=torch.Generator().manual_seed(1), dtype=torch.int32)
  x = torch.empty(B * T, D, device=gpu)
  cat = torch.zeros(128, 128, dtype=dtype, device=gpu)
  for fr in ([False, True] if dtype == BF else [False]):
    cat.zero_()
    ops.embed_rows(table.to(gpu), ids.to(gpu), i32([3], gpu), B, T, V, D, x, cat=cat, cat_off=D, cat_frag=fr)
    want = table[ids[:, 3:7].long()].view(B * T, D)
    assert torch.equal(x.cpu(), want.float())
    got = unfrag(cat, B * T) if fr else cat[:B * T]
    assert torch.equal(got[:, D:2 * D].cpu(), want) and not got[:, :D].any() and not got[:, 2 * D:].any()


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("M,D", [(3, 100), (5, 128), (130, 4104)])
@pytest.mark.parametrize("split", [0, 1, 3])
def test_residual_norm(gpu, dtype, M, D, split):
  """x += post-norm(y), x = y and x alone, with a next norm and without; y finished or in partial planes."""
  eps, ld = 0.02, (D + 15) // 16 * 16
  x0, y, wp, wn = rnd(M, D, seed=1), rnd(M, D, seed=2, scale=3.0), rnd(D, seed=3), rnd(D, seed=4)
  if split:
    planes = rnd(split, M, ld, seed=5)
    y = planes[:, :, :D].sum(0)
    src = ops.rows_src(ws=planes.to(gpu), split_k=split, plane=M * ld, ld=ld)
    keep = planes.to(gpu)
    src.ws = keep.data_ptr()
  else:
    yp = torch.zeros(M, ld, dtype=dtype)
    yp[:, :D] = y.to(dtype)
    y, keep = yp[:, :D].float(), yp.to(gpu)
    src = ops.rows_src(y=keep, ld=ld)
  wpg, wng = wp.to(gpu), wn.to(gpu)
  for mode in (0, 1, 2):
    for w_next in (wng, None):
      for fr in ([False, True] if dtype == BF else [False]):
        x = x0.to(gpu)
        out = torch.zeros((M + 127) // 128 * 128, (D + 127) // 128 * 128, dtype=dtype, device=gpu)
        d = L.ResidualNormDesc()
        d.M, d.D, d.dtype, d.eps, d.w_offset, d.mode, d.y = M, D, ops.DTYPES[dtype], eps, 1.0, mode, src
        d.w_post, d.x = wpg.data_ptr(), x.data_ptr()
        d.w_next = None if w_next is None else w_next.data_ptr()
        d.out, d.out_ld, d.out_frag = out.data_ptr(), out.shape[1], int(fr)
        ops.residual_norm(d)
        want = x0 if mode == 0 else x0 + R.rms_norm(y, wp, eps) if mode == 1 else y
        assert rel(x, want) < 1e-6
        got = (unfrag(out, M) if fr else out[:M])[:, :D]
        assert rel(got, want if w_next is None else R.rms_norm(want, wn, eps)) < (1e-6 if dtype == F32 else 4e-3)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("W,split", [(70, 1), (256, 1), (4096, 2), (70, 3)])
def test_gated_norm(gpu, dtype, W, split):
  M, off, eps = 5, 16, 0.5
  ld = (off + W + 15) // 16 * 16
  o, w = rnd(M, W, seed=1), rnd(W, seed=2)
  if split > 1:
    keep = rnd(split, M, ld, seed=3).to(gpu)
    g = keep.cpu().sum(0)[:, off:off + W]
    src = ops.rows_src(ws=keep, split_k=split, plane=M * ld, ld=ld)
  else:
    keep = rnd(M, ld, seed=3).to(dtype).to(gpu)
    g = keep.cpu().float()[:, off:off + W]
    src = ops.rows_src(y=keep, ld=ld)
  og, wg = o.to(gpu), w.to(gpu)
  want = R.rms_norm(o, w, eps, around_zero=False) * torch.sigmoid(g)
  for fr in ([False, True] if dtype == BF else [False]):
    out = torch.zeros(128, (W + 127) // 128 * 128, dtype=dtype, device=gpu)
    d = L.GatedNormDesc()
    d.M, d.W, d.dtype, d.eps, d.w_offset = M, W, ops.DTYPES[dtype], eps, 0.0
    d.o, d.o_ld, d.g, d.g_off, d.w = og.data_ptr(), W, src, off, wg.data_ptr()
    d.out, d.out_ld, d.out_frag = out.data_ptr(), out.shape[1], int(fr)
    ops.gated_norm(d)
    assert rel((unfrag(out, M) if fr else out[:M])[:, :W], want) < (1e-6 if dtype == F32 else 4e-3)


# ---- rotation + attention -----------------------------------------------------------------------
class Attn:
  """One attention layer's kernels over a batch: the plain implementation's inputs and the device's cache."""

  def __init__(self, gpu, dtype, H, G, dk, dv, rot, S, starts, scale=None, base=1000.0, seed=0, sharp=1.0):
    self.gpu, self.dtype, self.H, self.G, self.dk, self.dv, self.rot, self.S = gpu, dtype, H, G, dk, dv, rot, S
    self.starts, self.B = list(starts), len(starts)
    self.scale, self.base = dk ** -0.5 if scale is None else scale, base
    self.q = (rnd(self.B, S, H, dk, seed=seed + 1) * sharp).to(BF).float()
    self.k = rnd(self.B, S, G, dk, seed=seed + 2).to(BF).float()
    self.v = rnd(self.B, S, G, dv, seed=seed + 3).to(BF).float()
    self.sink = rnd(H, seed=seed + 4, scale=2.0)
    self.dkp, self.dvp = ops.sink_attn_pad(dk, False, dtype), ops.sink_attn_pad(dv, True, dtype)
    self.kc = torch.zeros(self.B, G, S, self.dkp, dtype=dtype, device=gpu)
    self.vc = torch.zeros(self.B, G, S, self.dvp, dtype=dtype, device=gpu)
    self.freq = torch.tensor([base ** (-2.0 * i / max(rot, 1)) for i in range(rot // 2)] or [0.0], dtype=F32, device=gpu)

  def run(self, col, T, kv_chunk=0, split=1, out_frag=False, sink=True):
    """The portion [col, col + T) of every row; output [B, T, H, dv]."""
    H, G, dk, dv, B = self.H, self.G, self.dk, self.dv, self.B
    up = lambda n: (n + 15) // 16 * 16
    ko, vo = up(H * dk), up(H * dk) + up(G * dk)
    ld = vo + up(G * dv)
    y = torch.zeros(B, T, ld)
    sl = slice(col, col + T)
    y[:, :, :H * dk], y[:, :, ko:ko + G * dk] = self.q[:, sl].reshape(B, T, -1), self.k[:, sl].reshape(B, T, -1)
    y[:, :, vo:vo + G * dv] = self.v[:, sl].reshape(B, T, -1)
    y = y.view(B * T, ld)
    if split > 1:
      keep = torch.stack([y * (0.5 if z == 0 else 0.5 / (split - 1)) for z in range(split)]).to(self.gpu).contiguous()
      src = ops.rows_src(ws=keep, split_k=split, plane=B * T * ld, ld=ld)
    else:
      keep = y.to(self.dtype).to(self.gpu)
      src = ops.rows_src(y=keep, ld=ld)
    st, cp = i32(self.starts, self.gpu), i32([col], self.gpu)
    q = torch.zeros(B * T, H * self.dkp, dtype=self.dtype, device=self.gpu)
    rd = L.PartRopeDesc()
    rd.B, rd.T, rd.S, rd.H, rd.G, rd.dk, rd.dv, rd.dkp, rd.dvp = B, T, self.S, H, G, dk, dv, self.dkp, self.dvp
    rd.rot_dims, rd.dtype, rd.inv_freq, rd.y, rd.k_off, rd.v_off = self.rot, ops.DTYPES[self.dtype], self.freq.data_ptr(), src, ko, vo
    rd.starts, rd.col_ptr, rd.q_out, rd.kcache, rd.vcache = st.data_ptr(), cp.data_ptr(), q.data_ptr(), self.kc.data_ptr(), self.vc.data_ptr()
    ops.part_rope_kvwrite(rd)
    ld_o = (H * dv + 127) // 128 * 128
    out = torch.zeros((B * T + 127) // 128 * 128, ld_o, dtype=self.dtype, device=self.gpu)
    ws = torch.empty(max(1, ops.sink_attn_ws_bytes(B, T, self.S, H, self.dvp, kv_chunk) // 4), device=self.gpu)
    sk = self.sink.to(self.gpu)
    ad = L.SinkAttnDesc()
    ad.B, ad.T, ad.S, ad.H, ad.G, ad.dk, ad.dv, ad.dkp, ad.dvp = B, T, self.S, H, G, dk, dv, self.dkp, self.dvp
    ad.scale, ad.dtype, ad.q, ad.kcache, ad.vcache = self.scale, rd.dtype, q.data_ptr(), rd.kcache, rd.vcache
    ad.sinks = sk.data_ptr() if sink else None
    ad.starts, ad.col_ptr, ad.kv_chunk, ad.ws = rd.starts, rd.col_ptr, kv_chunk, ws.data_ptr()
    ad.out, ad.out_ld, ad.out_frag = out.data_ptr(), ld_o, int(out_frag)
    ops.sink_attn(ad)
    torch.cuda.synchronize()
    got = unfrag(out, B * T) if out_frag else out[:B * T]
    return got[:, :H * dv].float().cpu().view(B, T, H, dv)

  def want(self, b, sink=True):
    """Output of row b's sequence (from its start on), [S - start, H, dv]."""
    s = self.starts[b]
    pos = torch.arange(self.S - s)
    q, k = (R.rotate(t[b, s:], pos, self.rot, self.base) for t in (self.q, self.k))
    if self.dtype == BF:      # the cache and the rotated queries are kept in bf16
      q, k = q.to(BF).float(), k.to(BF).float()
    return R.causal_attention(q, k, self.v[b, s:], self.scale, self.sink if sink else torch.full((self.H,), -1e30))

  def check(self, got, col, tol=None):
    tol = (2e-5 if self.dtype == F32 else 1e-2) if tol is None else tol
    T = got.shape[1]
    for b in range(self.B):
      s = max(self.starts[b], col)
      if s < col + T:
        w = self.want(b)[s - self.starts[b]:col + T - self.starts[b]]
        d = (got[b, s - col:] - w).abs().max() / w.abs().max()
        assert float(d) < tol, (b, float(d))


SHAPES = [(6, 1, 64, 112, 48), (6, 2, 48, 24, 48), (5, 1, 136, 200, 2), (8, 8, 32, 64, 0), (3, 3, 256, 256, 256), (10, 5, 21, 45, 6),
          (16, 4, 128, 128, 64), (2, 1, 192, 128, 64), (40, 1, 64, 64, 32), (2, 1, 320, 300, 64)]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,G,dk,dv,rot", SHAPES)
def test_attention_prompt_portions_and_steps(gpu, dtype, H, G, dk, dv, rot):
  """A prompt in one pass, then in portions (two tokens and more), then token by token, over the same
  rows with different starts; finished rows and partial planes, with a split key range and without."""
  S = 150
  a = Attn(gpu, dtype, H, G, dk, dv, rot, S, [0, 37, 149], sharp=3.0, seed=H)
  whole = a.run(0, S)
  a.check(whole, 0)
  a.kc.zero_(), a.vc.zero_()
  col = 0
  for T in (64, 2, 63, 5, 2, 14):
    a.check(a.run(col, T, split=2 if T == 5 else 1, out_frag=dtype == BF and T == 2), col)
    col += T
  assert col == S
  a.kc.zero_(), a.vc.zero_()
  a.run(0, 60)
  for t in range(60, 100):
    a.check(a.run(t, 1, kv_chunk=32 if dtype == BF and t % 2 else 0, split=3 if t % 3 == 0 else 1,
                  out_frag=dtype == BF and t % 4 == 0), t)


@pytest.mark.parametrize("decoded", [False, True])
@pytest.mark.parametrize("far", [0, 31, 32, 63, 64, 255, 298, 299])
def test_one_key_stands_out(gpu, decoded, far):
  """A single key far above the others, at tile and chunk borders and at both ends of the visible range,
  takes the weight; the key one column behind the query, higher still and in the cache, is not seen."""
  S = 400
  a = Attn(gpu, BF, 4, 2, 64, 64, 0, S, [0], scale=1.0, seed=far)
  a.q *= 0.02
  a.k *= 0.02
  a.sink[:] = 0.0
  a.q[0, 299] = 1.0
  a.k[0, far] = 0.4          # score 25.6 against about 0
  a.k[0, 300] = 0.8          # just behind the query
  got = a.run(0, S)[0, 299]
  if decoded:
    got = a.run(299, 1, kv_chunk=64)[0, 0]
  want = a.v[0, far].repeat_interleave(2, 0)
  assert float((got - want).abs().max()) < 2e-2


@pytest.mark.parametrize("dtype", DTYPES)
def test_sink_counts_once_and_has_no_value(gpu, dtype):
  """First token: the output is v * e^s / (e^s + e^sink); without sinks it is v."""
  a = Attn(gpu, dtype, 4, 2, 32, 48, 16, 8, [0, 3], seed=3)
  for sink in (True, False):
    got = a.run(0, 8, sink=sink)
    for b, s in enumerate(a.starts):
      for h in range(4):
        sc = float(a.q[b, s, h] @ a.k[b, s, h // 2]) * a.scale
        w = 1.0 / (1.0 + math.exp(float(a.sink[h]) - sc)) if sink else 1.0
        assert float((got[b, 0 if s == 0 else s, h] - w * a.v[b, s, h // 2]).abs().max()) < (1e-5 if dtype == F32 else 3e-2)


def test_large_sink_and_large_scores_stay_finite(gpu):
  for sink, sharp in ((80.0, 1.0), (-80.0, 1.0), (0.0, 60.0)):
    a = Attn(gpu, BF, 2, 1, 64, 64, 0, 90, [0], seed=5, sharp=sharp)
    a.sink[:] = sink
    w = a.want(0)
    for got in (a.run(0, 90)[0], torch.stack([a.run(t, 1)[0, 0] for t in range(90)])):
      assert torch.isfinite(got).all() and float((got - w).abs().max()) < 3e-2


# ---- lightning ----------------------------------------------------------------------------------
class Light:
  def __init__(self, gpu, dtype, H, dk, dv, S, starts, decay, seed=0):
    self.gpu, self.dtype, self.H, self.dk, self.dv, self.S, self.starts, self.B = gpu, dtype, H, dk, dv, S, starts, len(starts)
    self.decay = list(decay)
    self.q, self.k, self.v = (rnd(self.B, S, H, n, seed=seed + j).to(BF).float() for j, n in ((1, dk), (2, dk), (3, dv)))
    # a slot another sequence has used: a fresh sequence must not see it
    self.state = torch.full((self.B, H, dk, dv), 7.0, device=gpu)

  def run(self, col, T, split=1):
    H, dk, dv, B = self.H, self.dk, self.dv, self.B
    up = lambda n: (n + 15) // 16 * 16
    ko, vo = up(H * dk), 2 * up(H * dk)
    ld = vo + up(H * dv)
    y = torch.zeros(B, T, ld)
    sl = slice(col, col + T)
    y[:, :, :H * dk], y[:, :, ko:ko + H * dk] = self.q[:, sl].reshape(B, T, -1), self.k[:, sl].reshape(B, T, -1)
    y[:, :, vo:vo + H * dv] = self.v[:, sl].reshape(B, T, -1)
    y = y.view(B * T, ld)
    if split > 1:
      keep = torch.stack([y * 0.25, y * 0.75] + [y * 0.0] * (split - 2)).to(self.gpu).contiguous()
      src = ops.rows_src(ws=keep, split_k=split, plane=B * T * ld, ld=ld)
    else:
      keep = y.to(self.dtype).to(self.gpu)
      src = ops.rows_src(y=keep, ld=ld)
    lam, st, cp = torch.tensor(self.decay, device=self.gpu), i32(self.starts, self.gpu), i32([col], self.gpu)
    o = torch.full((B * T, H * dv), float("nan"), device=self.gpu)
    ws = torch.empty(max(1, ops.lightning_ws_bytes(B, T, H, dk, dv) // 4), device=self.gpu)
    d = L.LightningDesc()
    d.B, d.T, d.H, d.dk, d.dv, d.dtype, d.decay, d.y = B, T, H, dk, dv, ops.DTYPES[self.dtype], lam.data_ptr(), src
    d.k_off, d.v_off, d.starts, d.col_ptr = ko, vo, st.data_ptr(), cp.data_ptr()
    d.state, d.o, d.o_ld, d.ws = self.state.data_ptr(), o.data_ptr(), H * dv, ws.data_ptr()
    ops.lightning(d)
    torch.cuda.synchronize()
    return o.cpu().view(B, T, H, dv)

  def want(self, b, n):
    s = self.starts[b]
    q, k, v = (R.silu(t[b, s:n]) for t in (self.q, self.k, self.v))
    if self.dtype == BF and self.rounds:
      q, k, v = (t.to(BF).float() for t in (q, k, v))
    return R.lightning_recurrence(q.double(), k.double(), v.double(), self.decay)

  rounds = True

  def check(self, got, col):
    T = got.shape[1]
    for b in range(self.B):
      s = max(self.starts[b], col)
      if s < col + T:
        o, S = self.want(b, col + T)
        w = o[s - self.starts[b]:]
        # (one token at a time q, k, v stay fp32 behind their activation, in a prompt they are rounded)
        tol = 2e-5 if self.dtype == F32 else 1.2e-2
        e = rel(got[b, s - col:], w), rel(self.state[b], S)
        assert max(e) < tol, (b, col, e)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,dk,dv", [(4, 16, 40), (2, 64, 128), (3, 20, 36), (1, 160, 136), (2, 128, 64), (2, 8, 264), (5, 12, 10)])
def test_lightning_prompt_portions_and_steps(gpu, dtype, H, dk, dv):
  decay = [0.5, 0.9, 1.0, 0.0, 0.995][:H]
  S = 330
  a = Light(gpu, dtype, H, dk, dv, S, [0, 70, 129, 329], decay, seed=H)
  a.check(a.run(0, S), 0)                 # one pass (cut into spans that run in parallel where few rows ask for it)
  a.state.fill_(-3.0)
  col = 0
  for T in (64, 2, 63, 2, 100, 65, 3):
    a.check(a.run(col, T), col)
    col += T
  for t in range(col, S):                 # then token by token, finished rows and partial planes
    a.check(a.run(t, 1, split=2 if t % 2 else 1), t)
  b = Light(gpu, dtype, H, dk, dv, 40, [0, 5], decay, seed=9)
  for t in range(40):                     # all of it token by token
    b.check(b.run(t, 1), t)


def test_lightning_remembers_and_forgets(gpu):
  """One key-value pair far back: with decay 1 it returns whole after hundreds of tokens, with decay 0 it
  is gone with the next token; the last token of a chunk and the first of the next are the same to it."""
  S = 520
  for at in (0, 63, 64, 127, 128, 300):
    a = Light(gpu, BF, 3, 32, 32, S, [0], [1.0, 0.0, 0.98])
    a.q[:], a.k[:], a.v[:] = -20.0, -20.0, 0.0        # silu(-20) = 0 to bf16
    a.k[0, at], a.v[0, at] = 2.0, a.v[0, at] + 1.0
    a.q[0, at], a.q[0, at + 1], a.q[0, S - 1] = 1.0, 1.0, 1.0
    got = a.run(0, S)[0]
    full = float(R.silu(torch.tensor(1.0)) * R.silu(torch.tensor(2.0)) * 32 * R.silu(torch.tensor(1.0)))
    for h, lam in enumerate(a.decay):
      for t in (at, at + 1, S - 1):
        want = full * lam ** (t - at)
        assert abs(float(got[t, h, 5]) - want) < 1e-2 * full, (at, h, t, float(got[t, h, 5]), want)


# ---- logits -------------------------------------------------------------------------------------
def test_logits_stats(gpu):
  M, V, temp = 6, 1003, 0.7
  lg = rnd(M, V, scale=3.0).to(gpu)
  lg[2, 17] = lg[2, 900] = 50.0
  tg, fb = i32([0, 5, 900, 1002, 7, 33], gpu), i32([3, 17], gpu)
  out = {k: torch.zeros(M, dtype=torch.int32 if k.endswith("id") else F32, device=gpu)
         for k in ("best_id", "best_logp", "target_logp", "lse", "entropy", "draw_id", "draw_logp")}
  d = L.LogitsDesc()
  d.M, d.V, d.logits, d.temperature = M, V, lg.data_ptr(), temp
  d.forbidden, d.n_forbidden, d.targets = fb.data_ptr(), 2, tg.data_ptr()
  step = i32([4], gpu)
  d.draw_key1, d.draw_rng_variant, d.draw_step_ptr = 11, 1, step.data_ptr()
  for k, t in out.items():
    setattr(d, k, t.data_ptr())
  ops.logits_stats(d)
  x = lg.cpu().double() / temp
  x[:, [3, 17]] = -math.inf
  lp = torch.log_softmax(x, -1)
  o = {k: t.cpu() for k, t in out.items()}
  assert torch.equal(o["best_id"].long(), x.argmax(-1))
  rows = torch.arange(M)
  for name, w in (("best_logp", lp.max(-1).values), ("target_logp", lp[rows, tg.cpu().long()]), ("lse", torch.logsumexp(x, -1)),
                  ("entropy", -(lp.exp() * lp.masked_fill(lp == -math.inf, 0.0)).sum(-1)), ("draw_logp", lp[rows, o["draw_id"].long()])):
    torch.testing.assert_close(o[name].double(), w, rtol=2e-5, atol=2e-5)
  assert len(set(o["draw_id"].tolist())) > 1 and not set(o["draw_id"].tolist()) & {3, 17}


# ---- whole models -------------------------------------------------------------------------------
def model_of(name, seed, dtype, gpu):
  d = C.CONFIGS[name]
  w = C.random_weights(d, seed)
  return d, w, StackModel(config.nunezen_from_dict(d), w, gpu, dtype)


def err(got, want):
  """Row error of logits relative to the logits' spread: the worst row, or three times the mean one."""
  e = got - want
  e = e - e.mean(-1, keepdims=True)
  rows = np.sqrt((e ** 2).mean(-1)) / want.std()
  return float(max(rows.max(), 3.0 * np.sqrt((rows ** 2).mean()) if len(rows) > 8 else 0.0))


# bf16 rounding through up to eight sublayers with sharp scores: a single row can be several times off the rest
TOL = {BF: 0.15, F32: 1e-4}


def all_logits(model, streams, cut):
  """Logits of every position of the given streams as one batch: the first len - cut tokens of each as its
  prompt, the rest one by one."""
  rp = Replay(model)
  first = rp.step({"entries": [{"id": str(i), "tokens": s[:len(s) - cut], "want": list(range(len(s) - cut))}
                               for i, s in enumerate(streams)], "end": []})
  parts, at = [], 0
  for s in streams:
    parts.append([first[at:at + len(s) - cut]])
    at += len(s) - cut
  for j in range(cut):
    lg = rp.step({"entries": [{"id": str(i), "tokens": [s[len(s) - cut + j]], "want": [0]} for i, s in enumerate(streams)],
                  "end": [str(i) for i in range(len(streams))] if j == cut - 1 else []})
    for i in range(len(streams)):
      parts[i].append(lg[i:i + 1])
  assert cut == 0 or not rp.batches
  return [np.concatenate(p) for p in parts]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", sorted(C.CONFIGS))
def test_prompts_decoding_and_unequal_batches(gpu, name, dtype):
  """Streams of different lengths (1 token too) against the plain implementation: each alone as one prompt,
  each mostly decoded, and all as one batch."""
  d, w, model = model_of(name, 5, dtype, gpu)
  streams = [C.tokens(d, n, 10 + n) for n in (150, 41, 33)]
  want = [R.forward(d, w, s).numpy() for s in streams]
  for i, s in enumerate(streams):
    e = [err(all_logits(model, [s], cut)[0], want[i]) for cut in (0, len(s) - 1 if i == 2 else 30)]
    assert max(e) < TOL[dtype], (i, e)
  e = [err(got, want[i]) for i, got in enumerate(all_logits(model, streams, 32))]
  assert max(e) < TOL[dtype], e


def test_residual_after_every_layer_run(gpu):
  """fp32: the residual stream behind every layer run, looped layers once per pass."""
  for name in sorted(C.CONFIGS):
    d, w, model = model_of(name, 6, F32, gpu)
    toks = C.tokens(d, 23, 3)
    want = []
    R.forward(d, w, toks, layers_out=want)
    got = []
    runner = model.new_runner(1, 23, 23, -1)
    runner.residual_sink = lambda x: got.append(x.cpu().clone())
    runner.forward_hidden(i32([toks], gpu), None, runner.zero, model.new_cache(1, 23))
    assert len(got) == len(want) == len(model.cfg.layer_runs)
    for a, b in zip(got, want):
      assert rel(a, b) < 2e-5


@pytest.mark.parametrize("dtype", DTYPES)
def test_portions_of_a_prompt(gpu, dtype):
  """The same prompt in portions of 2, 3, 7, 64 and 40 tokens, rows starting at different columns."""
  d, w, model = model_of("mixed", 7, dtype, gpu)
  streams = [C.tokens(d, n, 20 + n) for n in (116, 90)]
  P = 116
  buf = torch.full((2, P), -1, dtype=torch.int32)
  for b, s in enumerate(streams):
    buf[b, P - len(s):] = torch.tensor(s)
  buf, starts = buf.to(gpu), i32([P - len(s) for s in streams], gpu)
  cache = model.new_cache(2, P)
  hidden, col = [], 0
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
  starts = i32([0, 20], gpu)
  out = []
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
  """Two tokens of prompt, then hundreds of steps: the cache grows, states are carried all the way."""
  d, w, model = model_of("mixed", 9, F32, gpu)
  s = C.tokens(d, 300, 40)
  got = all_logits(model, [s], 298)[0]
  assert err(got, R.forward(d, w, s).numpy()) < 2e-4


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["mixed", "odd"])
def test_greedy_generation(gpu, name, dtype):
  """The public sampler (prompts of different lengths, graph replay): every token it picks is the plain
  implementation's best up to rounding, and its log-probabilities are that distribution's."""
  d, w, model = model_of(name, 10, dtype, gpu)
  prompts = [np.array(C.tokens(d, n, 50 + n), dtype=np.int32) for n in (40, 3, 17, 1)]
  sampler = Sampler(model, IdTokenizer(d["vocab"], pad_id=0, eos_id=1), CacheConfig(64 + 40))
  out = sampler(prompts, 40, max_prompt_length=64, return_logprobs=True, eos_tokens=[-1])
  eager = Sampler(model, sampler.tokenizer, CacheConfig(64 + 40), use_graph=False)(prompts, 40, max_prompt_length=64, eos_tokens=[-1])
  for p, t, lp, te in zip(prompts, out.tokens, out.logprobs, eager.tokens):
    assert list(t) == list(te)
    lg = R.forward(d, w, list(p) + list(t)).double()[len(p) - 1:-1]
    spread = float(lg.std())
    pick = lg[torch.arange(40), torch.tensor(t.astype(np.int64))]
    tol = 1e-3 if dtype == F32 else 0.25
    assert float((lg.max(-1).values - pick).max()) < tol * spread
    want = torch.log_softmax(lg, -1)[torch.arange(40), torch.tensor(t.astype(np.int64))]
    assert float((torch.tensor(lp).double() - want).abs().max()) < tol * spread


@pytest.mark.parametrize("name,dtype", [("mixed", BF), ("odd", BF), ("mixed", F32)])
def test_sampling_modes(gpu, name, dtype):
  """top-k 1 is greedy; a seed repeats itself; the whole-vocabulary draw, nucleus and top-k run; logits come back."""
  d, w, model = model_of(name, 11, dtype, gpu)
  prompts = [C.tokens(d, n, 60 + n) for n in (9, 20)]
  s = Sampler(model, IdTokenizer(d["vocab"], pad_id=-1, eos_id=1), CacheConfig(48))
  call = lambda **kw: [list(t) for t in s(prompts, 12, max_prompt_length=32, eos_tokens=[-1], **kw).tokens]
  greedy = call()
  assert call(temperature=1.0, top_p=1.0, top_k=1, seed=3) == greedy
  for kw in (dict(top_p=1.0), dict(top_p=0.8), dict(top_p=0.9, top_k=20), dict(top_p=1.0, top_k=d["vocab"])):
    a = call(temperature=2.5, seed=4, **kw)
    assert a == call(temperature=2.5, seed=4, **kw) and a != call(temperature=2.5, seed=5, **kw)
  banned = sorted({t for g in greedy for t in g})[:3]
  assert not {t for g in call(forbidden_tokens=banned) for t in g} & set(banned)
  out = s(prompts, 12, max_prompt_length=32, eos_tokens=[-1], return_logits=True)
  for p, t, lg in zip(prompts, out.tokens, out.logits):
    assert err(lg, R.forward(d, w, list(p) + list(t)).numpy()[len(p) - 1:-1]) < TOL[dtype]


def test_rollout_log_probabilities_and_weight_updates(gpu):
  d, w, model = model_of("mixed", 12, BF, gpu)
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
    assert np.abs(lp[i] - want).max() < 0.5 and np.abs(np.array(res.logprobs[i]) - lp[i]).max() < 0.5
  w2 = C.random_weights(d, 13)
  before = all_logits(model, [prompts[0]], 0)[0]
  bad = dict(w2)
  bad["l0.mix.k"] = bad["l0.mix.k"][:, :-1]
  with pytest.raises(ValueError, match="same shape"):
    roll.update_params(bad)
  with pytest.raises(ValueError, match="same structure"):
    roll.update_params({"l0.mix.q": w2["l0.mix.q"]})        # a member of a fused projection without the others
  assert np.array_equal(all_logits(model, [prompts[0]], 0)[0], before)
  roll.update_params(w2)
  assert err(all_logits(model, [prompts[0]], 0)[0], R.forward(d, w2, prompts[0]).numpy()) < TOL[BF]
  with pytest.raises(ValueError, match="packed"):
    common.compute_per_token_logps(model, pt, comp, pad_id=0, eos_id=1, segment_ids=np.ones((2, 18)),
                                   segment_positions=np.tile(np.arange(18), (2, 1)))


@pytest.mark.parametrize("B", [1, 40, 130])
def test_batch_sizes_of_a_decode_step(gpu, B):
  """Every row tile of the few-row linears: a batch of equal sequences gives every row the same logits."""
  d, w, model = model_of("mixed", 14, BF, gpu)
  s = C.tokens(d, 12, 70)
  got = all_logits(model, [s] * B, 4)
  want = R.forward(d, w, s).numpy()
  for g in got[:: max(1, B // 5)]:
    assert err(g, want) < TOL[BF]


def test_command_line(gpu, tmp_path):
  """bin/trace_run and `python -m tunix_amd generate` on a model folder, as child processes."""
  d, w = C.write_model(tmp_path, "odd", seed=15)
  a, b = C.tokens(d, 12, 80), C.tokens(d, 7, 81)
  steps = [{"step": 0, "entries": [{"id": "a", "tokens": a[:10], "want": [9, 0]}, {"id": "b", "tokens": b[:5], "want": []}], "end": []},
           {"step": 1, "entries": [{"id": "b", "tokens": b[5:6], "want": []}, {"id": "a", "tokens": a[10:11], "want": []}], "end": []},
           {"step": 2, "entries": [{"id": "a", "tokens": a[11:], "want": [0]}, {"id": "b", "tokens": b[6:], "want": [0]}], "end": ["b", "a"]},
           {"step": 3, "entries": [{"id": "c", "tokens": b, "want": [6]}], "end": ["c"]}]
  out = tmp_path / "out"
  out.mkdir()
  p = subprocess.run([os.path.join(ROOT, "bin", "trace_run"), "--model", str(tmp_path), "--dtype", "float32", "--out", str(out),
                      "--max-tokens", "64"], input="\n".join(json.dumps(s) for s in steps), capture_output=True, text=True, timeout=100)
  assert p.returncode == 0, p.stderr[-2000:]
  assert p.stdout.split() == "done 0 done 1 done 2 done 3".split()
  assert sorted(os.listdir(out)) == ["0.f32", "2.f32", "3.f32"]
  la, lb = R.forward(d, w, a).numpy(), R.forward(d, w, b).numpy()
  read = lambda n: np.fromfile(out / f"{n}.f32", "<f4").reshape(-1, d["vocab"])
  assert err(read(0), la[[9, 0]]) < 1e-4
  assert err(read(2), np.stack([la[11], lb[6]])) < 1e-4 and err(read(3), lb[6:7]) < 1e-4
  p = subprocess.run([sys.executable, "-m", "tunix_amd", "generate", "--model", str(tmp_path), "--dtype", "float32", "--max-tokens", "5",
                      "--prompt", " ".join(map(str, a))], capture_output=True, text=True, timeout=100, cwd=ROOT)
  assert p.returncode == 0, p.stderr[-2000:]
  line = json.loads(p.stdout)
  full = list(a)
  for t in line["tokens"]:
    lg = R.forward(d, w, full)[-1]
    assert float(lg.max() - lg[t]) < 1e-3
    full.append(t)
  assert len(line["tokens"]) == 5


def test_replay_rejects_what_it_cannot_run(gpu):
  d, _, model = model_of("attention", 16, BF, gpu)
  rp = Replay(model)
  step = lambda *es: rp.step({"entries": [{"id": i, "tokens": t, "want": w} for i, t, w in es], "end": []})
  with pytest.raises(ValueError, match="no token"):
    step(("a", [], []))
  with pytest.raises(ValueError, match="outside the vocabulary"):
    step(("a", [d["vocab"]], []))
  with pytest.raises(ValueError, match="wants a place"):
    step(("a", [1, 2], [2]))
  assert step(("a", [1, 2], []), ("b", [3], [])) is None
  with pytest.raises(ValueError, match="either starts"):
    step(("a", [4], []), ("c", [4], []))
  with pytest.raises(ValueError, match="go on together"):
    step(("a", [4], []))
  assert step(("a", [4], []), ("b", [4], [0])).shape == (1, d["vocab"])
  rp.step({"entries": [], "end": ["a", "b"]})
  assert not rp.batches


def test_descriptor_errors(gpu):
  """Shapes the kernels do not take are refused before any launch."""
  z = torch.zeros(16, 256, dtype=BF, device=gpu)
  d = L.DenseDesc()
  d.M, d.K, d.N, d.x, d.w, d.y, d.ldx, d.ldy, d.split_k = 1, 100, 16, z.data_ptr(), z.data_ptr(), z.data_ptr(), 256, 16, 1
  with pytest.raises(ValueError, match="multiple of 128"):
    ops.dense_linear(d)
  d.K, d.N = 128, 24
  with pytest.raises(ValueError, match="multiple of 16"):
    ops.dense_linear(d)
  a = L.SinkAttnDesc()
  a.B, a.T, a.S, a.H, a.G = 1, 1, 8, 3, 2
  with pytest.raises(ValueError, match="bad shape"):
    ops.sink_attn(a)
  r = L.PartRopeDesc()
  r.B, r.T, r.S, r.H, r.G, r.dk, r.dv, r.dkp, r.dvp, r.rot_dims = 1, 1, 8, 2, 2, 16, 16, 16, 16, 18
  with pytest.raises(ValueError, match="rot_dims"):
    ops.part_rope_kvwrite(r)

