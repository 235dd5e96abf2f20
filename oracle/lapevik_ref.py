"""Plain CPU implementation of the Lapevik decoder: one function per mechanism, one token loop or one
dense matrix per step, no cache, no batching.  It shares nothing with the product path; tests compare
the kernels and the model with it.

A configuration is the plain dictionary of a config.json; weights are a dictionary of tensors by
their file names, linear weights stored [out, in].
"""
from __future__ import annotations

import math

import torch

RECURRENT = ("mamba2", "mamba2_2")


def group_norm(x, w, eps, groups=1):
  """The last axis in `groups` equal runs, each divided by its own sqrt(mean(run^2) + eps); times w."""
  parts = x.reshape(*x.shape[:-1], groups, x.shape[-1] // groups)
  parts = parts / torch.sqrt((parts * parts).mean(-1, keepdim=True) + eps)
  return parts.reshape(x.shape) * w


def silu(z):
  return z / (1.0 + torch.exp(-z))


def softplus(z):
  return torch.where(z > 0, z, torch.zeros_like(z)) + torch.log1p(torch.exp(-z.abs()))


def token_shift(x, mix, before=None):
  """x [T, D]: every row moved towards the row in front of it by `mix`; in front of the first one lies
  `before` (zeros at the start of a sequence)."""
  first = torch.zeros_like(x[:1]) if before is None else before[None]
  prev = torch.cat([first, x[:-1]])
  return x + (prev - x) * mix


def short_conv(u, taps, bias, before=None):
  """u [T, C], taps [C, K]: out[t, c] = bias[c] + sum_j taps[c, K-1-j] u[t-j, c]; rows in front of the first
  one are `before` [K-1, C] (zeros at the start of a sequence)."""
  T, K = u.shape[0], taps.shape[1]
  if before is None:
    before = torch.zeros(K - 1, u.shape[1], dtype=u.dtype)
  full = torch.cat([before, u])
  out = bias.expand(T, -1).clone()
  for k in range(K):
    out = out + taps[:, k] * full[k:k + T]
  return out


def ssd_recurrence(x, B, C, dt, A_log, D, state=None):
  """x [T, H, P], B and C [T, G, N], dt [T, H] (after softplus): per head
  S <- exp(-exp(A_log) dt) S + dt B x^T, y = S^T C + D x.  Returns (y, the last S [H, N, P])."""
  T, H, P = x.shape
  G, N = B.shape[1:]
  S = torch.zeros(H, N, P, dtype=x.dtype) if state is None else state.clone()
  y = torch.empty_like(x)
  for t in range(T):
    for h in range(H):
      g = h // (H // G)
      S[h] = torch.exp(-torch.exp(A_log[h]) * dt[t, h]) * S[h] + dt[t, h] * torch.outer(B[t, g], x[t, h])
      y[t, h] = S[h].T @ C[t, g] + D[h] * x[t, h]
  return y, S


def rotate_interleaved(x, positions, base):
  """x [T, ..., n]: pairs (2i, 2i + 1) turned by position * base^(-2i / n)."""
  n = x.shape[-1]
  out = x.clone()
  shape = [-1] + [1] * (x.dim() - 2)
  for i in range(n // 2):
    a = positions.to(torch.float64) * float(base) ** (-2.0 * i / n)
    c, s = torch.cos(a).to(x.dtype).view(shape), torch.sin(a).to(x.dtype).view(shape)
    u, v = x[..., 2 * i], x[..., 2 * i + 1]
    out[..., 2 * i], out[..., 2 * i + 1] = u * c - v * s, v * c + u * s
  return out


def causal_attention(q, k, v, scale):
  """q, k [T, H, n], v [T, H, m] -> [T, H, m]: softmax over the keys up to the query."""
  T, H, _ = q.shape
  seen = torch.tril(torch.ones(T, T, dtype=torch.bool))
  out = torch.empty(T, H, v.shape[-1], dtype=q.dtype)
  for h in range(H):
    s = torch.where(seen, (q[:, h] @ k[:, h].T) * scale, torch.full((T, T), -math.inf, dtype=q.dtype))
    e = torch.exp(s - s.max(-1, keepdim=True).values)
    out[:, h] = (e / e.sum(-1, keepdim=True)) @ v[:, h]
  return out


def mamba2_mixer(h, w, p, m, eps):
  T = h.shape[0]
  H, P, N, G = m["heads"], m["vdim"], m["state"], m["groups"]
  inner = H * P
  y = h @ w[p + "in"].T
  z, u, dt = y[:, :inner], y[:, inner:2 * inner + 2 * G * N], y[:, 2 * inner + 2 * G * N:]
  u = silu(short_conv(u, w[p + "conv"], w[p + "conv.b"]))
  x, B, C = u[:, :inner].view(T, H, P), u[:, inner:inner + G * N].view(T, G, N), u[:, inner + G * N:].view(T, G, N)
  y, _ = ssd_recurrence(x, B, C, softplus(dt + w[p + "dt_bias"]), w[p + "A_log"], w[p + "D"])
  y = group_norm(y.reshape(T, inner) * silu(z), w[p + "norm"], eps, m["norm_groups"])
  return y @ w[p + "o"].T


def latent_attention_mixer(h, w, p, m, positions, eps):
  T = h.shape[0]
  H, n, r, vd, rank = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
  cq = group_norm(h @ w[p + "dq"].T, w[p + "dq.norm"], eps)
  q = (cq @ w[p + "uq"].T).view(T, H, n + r)
  kv = h @ w[p + "dkv"].T
  c = group_norm(kv[:, :rank], w[p + "dkv.norm"], eps)
  kr = rotate_interleaved(kv[:, rank:], positions, m["rot"]["base"])
  k = torch.cat([(c @ w[p + "uk"].T).view(T, H, n), kr[:, None].expand(T, H, r)], dim=-1)
  q = torch.cat([q[..., :n], rotate_interleaved(q[..., n:], positions, m["rot"]["base"])], dim=-1)
  o = causal_attention(q, k, (c @ w[p + "uv"].T).view(T, H, vd), m["scale"])
  return (o.reshape(T, H * vd) * torch.sigmoid(h @ w[p + "g"].T)) @ w[p + "o"].T


def route(h, router, top):
  """(experts [T, top], weights [T, top]): the largest logits and the softmax over them alone."""
  z = h @ router.T
  val, idx = torch.sort(z, dim=-1, descending=True, stable=True)
  val, idx = val[:, :top], idx[:, :top]
  e = torch.exp(val - val[:, :1])
  return idx, e / e.sum(-1, keepdim=True)


def experts_mlp(h, w, p, m):
  idx, wt = route(h, w[p + "router"], m["router"]["top"])
  out = torch.zeros_like(h)
  for t in range(h.shape[0]):
    for e, a in zip(idx[t].tolist(), wt[t]):
      u = silu(w[p + f"e{e}.gate"] @ h[t]) * (w[p + f"e{e}.up"] @ h[t])
      out[t] += a * (w[p + f"e{e}.down"] @ u)
  return out


def forward(cfg, weights, tokens, dtype=torch.float32, layers_out=None):
  """Logits [T, vocab] of one sequence; layers_out, a list, receives the residual after each layer."""
  w = {k: v.to(dtype) for k, v in weights.items()}
  eps, groups = cfg["norm"]["eps"], cfg["norm"]["groups"]
  tokens = torch.as_tensor(tokens, dtype=torch.int64)
  positions = torch.arange(tokens.numel())
  x = group_norm(w["embed"][tokens], w["embed.norm"], eps, groups)
  for i, ly in enumerate(cfg["layers"]):
    p = f"l{i}."
    h = token_shift(x, w[p + "shift"])
    if ly["type"] in RECURRENT:
      y = mamba2_mixer(h, w, p + "mix.", ly["mixer"], eps)
    else:
      y = latent_attention_mixer(h, w, p + "mix.", ly["mixer"], positions, eps)
    x = x + group_norm(y, w[p + "norm1"], eps, groups)
    if ly["mlp"] is not None:
      x = x + group_norm(experts_mlp(x, w, p + "mlp.", ly["mlp"]), w[p + "norm2"], eps, groups)
    if layers_out is not None:
      layers_out.append(x)
  return group_norm(x, w["final.norm"], eps, groups) @ w["embed"].T


def tensor_shapes(cfg):
  """File name -> shape of every tensor of a configuration."""
  D, V = cfg["width"], cfg["vocab"]
  out = {"embed": (V, D), "embed.norm": (D,), "final.norm": (D,)}
  for i, ly in enumerate(cfg["layers"]):
    p, m = f"l{i}.", ly["mixer"]
    x = p + "mix."
    H = m["heads"]
    out.update({p + "shift": (D,), p + "norm1": (D,)})
    if ly["type"] in RECURRENT:
      inner, bc = H * m["vdim"], 2 * m["groups"] * m["state"]
      out.update({x + "in": (2 * inner + bc + H, D), x + "conv": (inner + bc, m["conv"]), x + "conv.b": (inner + bc,),
                  x + "dt_bias": (H,), x + "A_log": (H,), x + "D": (H,), x + "norm": (inner,), x + "o": (D, inner)})
    else:
      n, r, vd, rank, qr = m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"], m["q_rank"]
      out.update({x + "dq": (qr, D), x + "dq.norm": (qr,), x + "uq": (H * (n + r), qr), x + "dkv": (rank + r, D),
                  x + "dkv.norm": (rank,), x + "uk": (H * n, rank), x + "uv": (H * vd, rank), x + "g": (H * vd, D),
                  x + "o": (D, H * vd)})
    if ly["mlp"] is not None:
      F, E = ly["mlp"]["expert"]["ff"], ly["mlp"]["router"]["experts"]
      out.update({p + "norm2": (D,), p + "mlp.router": (E, D)})
      for e in range(E):
        out.update({p + f"mlp.e{e}.gate": (F, D), p + f"mlp.e{e}.up": (F, D), p + f"mlp.e{e}.down": (D, F)})
  return out
