"""Plain CPU implementation of the Nunezen decoder: one function per mechanism, one token loop or
one dense matrix per step, no cache, no batching.  It shares nothing with the product path; tests
compare the kernels and the model with it.

A configuration is the plain dictionary of a config.json; weights are a dictionary of tensors by
their file names, linear weights stored [out, in].
"""
from __future__ import annotations

import math

import torch


def rms_norm(x, w, eps, around_zero=True):
  """x / sqrt(mean(x^2) + eps), times (1 + w) for a weight stored around zero, else times w."""
  y = x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)
  return y * (1.0 + w) if around_zero else y * w


def gelu_tanh(z):
  return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z * z * z)))


def silu(z):
  return z / (1.0 + torch.exp(-z))


def rotate(x, positions, dims, base):
  """x [T, heads, dim]: the first `dims` dimensions of every head are rotated in pairs
  (i, i + dims / 2) by the angle position * base^(-2i / dims); the rest passes through."""
  half = dims // 2
  out = x.clone()
  for i in range(half):
    f = float(base) ** (-2.0 * i / dims)
    a = positions.to(torch.float64) * f
    c, s = torch.cos(a).to(x.dtype)[:, None], torch.sin(a).to(x.dtype)[:, None]
    u, v = x[..., i], x[..., i + half]
    out[..., i] = u * c - v * s
    out[..., i + half] = v * c + u * s
  return out


def sink_softmax(scores, sink):
  """Softmax over the last axis whose denominator also holds exp(sink); -inf scores are unseen."""
  top = torch.maximum(scores.max(-1, keepdim=True).values, sink)
  e = torch.exp(scores - top)
  return e / (e.sum(-1, keepdim=True) + torch.exp(sink - top))


def causal_attention(q, k, v, scale, sink):
  """q [T, H, dim], k [T, G, dim], v [T, G, vdim], sink [H] -> [T, H, vdim]."""
  T, H, _ = q.shape
  G = k.shape[1]
  seen = torch.tril(torch.ones(T, T, dtype=torch.bool))
  out = torch.empty(T, H, v.shape[-1], dtype=q.dtype)
  for h in range(H):
    g = h // (H // G)
    s = (q[:, h] @ k[:, g].T) * scale
    s = torch.where(seen, s, torch.full_like(s, -math.inf))
    out[:, h] = sink_softmax(s, sink[h]) @ v[:, g]
  return out


def lightning_recurrence(q, k, v, decay, state=None):
  """q, k [T, H, dim], v [T, H, vdim], decay [H]: S <- decay S + k v^T, o = S^T q, token by token.
  Returns (o [T, H, vdim], the last S [H, dim, vdim])."""
  T, H, dim = q.shape
  S = torch.zeros(H, dim, v.shape[-1], dtype=q.dtype) if state is None else state.clone()
  lam = torch.as_tensor(decay, dtype=q.dtype)[:, None, None]
  out = torch.empty(T, H, v.shape[-1], dtype=q.dtype)
  for t in range(T):
    S = lam * S + k[t][:, :, None] * v[t][:, None, :]
    out[t] = torch.einsum("hd,hdv->hv", q[t], S)
  return out, S


def attention_mixer(h, w, p, m, positions):
  T = h.shape[0]
  q = (h @ w[p + "q"].T).view(T, m["heads"], m["dim"])
  k = (h @ w[p + "k"].T).view(T, m["kv_heads"], m["dim"])
  v = (h @ w[p + "v"].T).view(T, m["kv_heads"], m["vdim"])
  q = rotate(q, positions, m["rot"]["dims"], m["rot"]["base"])
  k = rotate(k, positions, m["rot"]["dims"], m["rot"]["base"])
  o = causal_attention(q, k, v, m["scale"], w[p + "sink"])
  return o.reshape(T, -1) @ w[p + "o"].T


def lightning_mixer(h, w, p, m, eps):
  T = h.shape[0]
  q = silu(h @ w[p + "q"].T).view(T, m["heads"], m["dim"])
  k = silu(h @ w[p + "k"].T).view(T, m["heads"], m["dim"])
  v = silu(h @ w[p + "v"].T).view(T, m["heads"], m["vdim"])
  o, _ = lightning_recurrence(q, k, v, m["decay"])
  o = rms_norm(o.reshape(T, -1), w[p + "norm"], eps, around_zero=False)
  return (o * torch.sigmoid(h @ w[p + "g"].T)) @ w[p + "o"].T


def glu_mlp(h, w, p):
  return (gelu_tanh(h @ w[p + "gate"].T) * (h @ w[p + "up"].T)) @ w[p + "down"].T


def layer_order(cfg):
  """[(layer index, whether a pass of the loop begins here)] in the order they run."""
  n, loop = len(cfg["layers"]), cfg.get("loop")
  if not loop:
    return [(i, False) for i in range(n)]
  order = [(i, False) for i in range(loop["start"])]
  for _ in range(loop["times"]):
    order += [(i, i == loop["start"]) for i in range(loop["start"], loop["stop"])]
  return order + [(i, False) for i in range(loop["stop"], n)]


def forward(cfg, weights, tokens, dtype=torch.float32, layers_out=None):
  """Logits [T, vocab] of one sequence; layers_out, a list, receives the residual after each layer run."""
  w = {k: v.to(dtype) for k, v in weights.items()}
  eps = cfg["norm"]["eps"]
  tokens = torch.as_tensor(tokens, dtype=torch.int64)
  positions = torch.arange(tokens.numel())
  x = x0 = w["embed"][tokens]
  for i, begins in layer_order(cfg):
    ly, p = cfg["layers"][i], f"l{i}."
    if begins:
      x = torch.cat([x, x0], dim=-1) @ w["loop.in"].T
    h = rms_norm(x, w[p + "norm1"], eps)
    if ly["type"] == "attention":
      y = attention_mixer(h, w, p + "mix.", ly["mixer"], positions)
    else:
      y = lightning_mixer(h, w, p + "mix.", ly["mixer"], eps)
    x = x + rms_norm(y, w[p + "norm1b"], eps)
    if ly["mlp"] is not None:
      y = glu_mlp(rms_norm(x, w[p + "norm2"], eps), w, p + "mlp.")
      x = x + rms_norm(y, w[p + "norm2b"], eps)
    if layers_out is not None:
      layers_out.append(x)
  return rms_norm(x, w["final.norm"], eps) @ w["embed"].T


def tensor_shapes(cfg):
  """File name -> shape of every tensor of a configuration."""
  D, V = cfg["width"], cfg["vocab"]
  out = {"embed": (V, D), "final.norm": (D,)}
  if cfg.get("loop"):
    out["loop.in"] = (D, 2 * D)
  for i, ly in enumerate(cfg["layers"]):
    p, m = f"l{i}.", ly["mixer"]
    H, dk, dv = m["heads"], m["dim"], m["vdim"]
    G = m["kv_heads"] if ly["type"] == "attention" else H
    out.update({p + "norm1": (D,), p + "norm1b": (D,), p + "mix.q": (H * dk, D), p + "mix.k": (G * dk, D),
                p + "mix.v": (G * dv, D), p + "mix.o": (D, H * dv)})
    if ly["type"] == "attention":
      out[p + "mix.sink"] = (H,)
    else:
      out.update({p + "mix.g": (H * dv, D), p + "mix.norm": (H * dv,)})
    if ly["mlp"] is not None:
      F = ly["mlp"]["ff"]
      out.update({p + "norm2": (D,), p + "norm2b": (D,), p + "mlp.gate": (F, D), p + "mlp.up": (F, D),
                  p + "mlp.down": (D, F)})
  return out
