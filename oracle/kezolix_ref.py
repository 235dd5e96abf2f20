"""Plain CPU implementation of the Kezolix decoder: one function per mechanism, one token loop or one
dense matrix per step, no cache, no batching.  It shares nothing with the product path; tests compare
the kernels and the model with it.

A configuration is the plain dictionary of a config.json; weights are a dictionary of tensors by
their file names, linear weights stored [out, in].
"""
from __future__ import annotations

import math

import torch


def layer_norm(x, w, eps):
  """The last axis centred and divided by sqrt(variance + eps); times w."""
  c = x - x.mean(-1, keepdim=True)
  return c / torch.sqrt((c * c).mean(-1, keepdim=True) + eps) * w


def rms_norm(x, eps, w=None):
  y = x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)
  return y if w is None else y * w


def sigmoid(z):
  e = torch.exp(-z.abs())
  return torch.where(z >= 0, 1.0 / (1.0 + e), e / (1.0 + e))


def silu(z):
  return z * sigmoid(z)


# ---- attention ----------------------------------------------------------------------------------
def slopes(H: int):
  return [2.0 ** (-8.0 * (h + 1) / H) for h in range(H)]


def visible(i: int, j: int, chunk: int) -> bool:
  """Whether position i reads position j: not a later one, and one of its own chunk."""
  return j <= i and i // chunk == j // chunk


def biased_attention(q, k, v, scale, chunk):
  """q [T, H, dk], k [T, G, dk], v [T, G, dv]: softmax over the visible keys of scale q k minus the
  distance times the head's slope -> [T, H, dv]."""
  T, H, G = q.shape[0], q.shape[1], k.shape[1]
  out = torch.zeros(T, H, v.shape[2], dtype=q.dtype)
  mask = torch.tensor([[visible(i, j, chunk) for j in range(T)] for i in range(T)])
  distance = (torch.arange(T)[:, None] - torch.arange(T)[None, :]).to(q.dtype)
  for h, slope in enumerate(slopes(H)):
    g = h // (H // G)
    s = (q[:, h] @ k[:, g].T) * scale - slope * distance
    s = torch.where(mask, s, torch.full_like(s, -math.inf))
    e = torch.exp(s - s.max(-1, keepdim=True).values)
    out[:, h] = (e / e.sum(-1, keepdim=True)) @ v[:, g]
  return out


def attention_mixer(h, m, w, p, eps, kept):
  """kept: the keys and values of every attention layer so far, by layer; returns (output, this layer's)."""
  T, H, G = h.shape[0], m["heads"], m["kv_heads"]
  q = rms_norm(h @ w[p + "q"].T, eps, w[p + "q.norm"]).reshape(T, H, m["dim"])
  if m.get("kv_from") is None:
    k = rms_norm(h @ w[p + "k"].T, eps, w[p + "k.norm"]).reshape(T, G, m["dim"])
    kv = k, (h @ w[p + "v"].T).reshape(T, G, m["vdim"])
  else:
    kv = kept[m["kv_from"]]
  o = biased_attention(q, *kv, m["scale"], m["mask"]["size"])
  return o.reshape(T, -1) @ w[p + "o"].T, kv


# ---- gated recurrence ---------------------------------------------------------------------------
def forget_gate(z, lower):
  return lower + (1.0 - lower) * sigmoid(z)


def gated_recurrence(q, f, v, state=None):
  """q, f [T, H, dk], v [T, H, dv]: S <- f S + (1 - f) v^T, o = S^T q -> (o [T, H, dv], S [H, dk, dv])."""
  T, H, dk = q.shape
  S = torch.zeros(H, dk, v.shape[2], dtype=q.dtype) if state is None else state.clone()
  out = []
  for t in range(T):
    S = f[t][:, :, None] * S + (1.0 - f[t])[:, :, None] * v[t][:, None, :]
    out.append((S * q[t][:, :, None]).sum(1))
  return torch.stack(out), S


def recurrent_mixer(h, m, w, p, eps):
  T, H, dk, dv = h.shape[0], m["heads"], m["dim"], m["vdim"]
  q = silu(h @ w[p + "q"].T).reshape(T, H, dk)
  f = forget_gate(h @ w[p + "f"].T + w[p + "f.b"], w[p + "lower"]).reshape(T, H, dk)
  v = (h @ w[p + "v"].T).reshape(T, H, dv)
  o, _ = gated_recurrence(q, f, v)
  return rms_norm(o, eps, w[p + "norm"]).reshape(T, H * dv) @ w[p + "o"].T


# ---- feed-forward -------------------------------------------------------------------------------
def poly_norm(z, coef, eps):
  a, b, c, e = coef
  return a * rms_norm(z, eps) + b * rms_norm(z * z, eps) + c * rms_norm(z * z * z, eps) + e


def dense_mlp(h, w, p, eps):
  return poly_norm(h @ w[p + "up"].T, w[p + "act"], eps) @ w[p + "down"].T


def square_relu_mlp(h, w, p):
  z = (h @ w[p + "up"].T).clamp(min=0.0)
  return (z * z) @ w[p + "down"].T


def route(z, correction, top, scale):
  """z [T, E] -> (chosen experts [T, top], their weights)."""
  e = torch.exp(z - z.max(-1, keepdim=True).values)
  s = e / e.sum(-1, keepdim=True)
  ids = torch.argsort(s + correction, dim=-1, descending=True, stable=True)[:, :top]
  chosen = torch.gather(s, 1, ids)
  return ids, chosen / (chosen.sum(-1, keepdim=True) + 1e-20) * scale


def experts_mlp(h, mlp, w, p):
  r = mlp["router"]
  ids, weights = route(h @ w[p + "router"].T, w[p + "correction"], r["top"], r["scale"])
  out = torch.zeros_like(h)
  for e in range(r["experts"]):
    hit = (ids == e)
    rows = hit.any(1)
    if rows.any():
      share = (weights * hit)[rows].sum(1, keepdim=True)
      out[rows] += share * square_relu_mlp(h[rows], w, f"{p}e{e}.")
  gate = sigmoid(h @ w[p + "shared.sg"].T)
  return out + gate * square_relu_mlp(h, w, p + "shared.")


def feed_forward(h, mlp, w, p, eps):
  return dense_mlp(h, w, p, eps) if mlp["kind"] == "dense" else experts_mlp(h, mlp, w, p)


# ---- the model ----------------------------------------------------------------------------------
def tensor_shapes(cfg):
  """File name -> shape of every tensor of a configuration."""
  D, V = cfg["width"], cfg["vocab"]
  out = {"embed": (V, D), "pos": (cfg["max_positions"], D), "final.norm": (D,), "head": (V, D)}
  for i, ly in enumerate(cfg["layers"]):
    p, m, mlp = f"l{i}.", ly["mixer"], ly.get("mlp")
    x, H, n, vd = p + "mix.", m["heads"], m["dim"], m["vdim"]
    out.update({p + "norm1": (D,), p + "norm1b": (D,), p + "dwa": (i + 2,), x + "o": (D, H * vd), x + "q": (H * n, D)})
    if ly["type"] == "attention":
      out[x + "q.norm"] = (H * n,)
      if m.get("kv_from") is None:
        G = m["kv_heads"]
        out.update({x + "k": (G * n, D), x + "k.norm": (G * n,), x + "v": (G * vd, D)})
    else:
      out.update({x + "f": (H * n, D), x + "f.b": (H * n,), x + "lower": (H * n,), x + "v": (H * vd, D), x + "norm": (vd,)})
    if mlp is None:
      continue
    out.update({p + "norm2": (D,), p + "norm2b": (D,)})
    y = p + "mlp."
    if mlp["kind"] == "dense":
      out.update({y + "up": (mlp["ff"], D), y + "down": (D, mlp["ff"]), y + "act": (4,)})
      continue
    E = mlp["router"]["experts"]
    out.update({y + "router": (E, D), y + "correction": (E,), y + "shared.sg": (1, D)})
    for name, ff in [(f"e{e}", mlp["expert"]["ff"]) for e in range(E)] + [("shared", mlp["shared"]["ff"])]:
      out.update({f"{y}{name}.up": (ff, D), f"{y}{name}.down": (D, ff)})
  return out


def depth_average(rows, coef):
  return sum(c * x for c, x in zip(coef, rows))


def forward(cfg, weights, tokens, dtype=torch.float32, layers_out=None):
  """Logits [T, vocab] of one sequence; `layers_out` (a list) takes the residual behind every layer."""
  w = {n: t.to(dtype) for n, t in weights.items()}
  eps, mult = cfg["norm"]["eps"], cfg["residual_mult"]
  tokens = torch.as_tensor(tokens)
  x = w["embed"][tokens] + w["pos"][:len(tokens)]
  rows, kept = [x], {}
  for i, ly in enumerate(cfg["layers"]):
    p, m = f"l{i}.", ly["mixer"]
    h = layer_norm(x, w[p + "norm1"], eps)
    if ly["type"] == "attention":
      y, kept[i] = attention_mixer(h, m, w, p + "mix.", eps, kept)
    else:
      y = recurrent_mixer(h, m, w, p + "mix.", eps)
    x = x + mult * layer_norm(y, w[p + "norm1b"], eps)
    if ly.get("mlp") is not None:
      y = feed_forward(layer_norm(x, w[p + "norm2"], eps), ly["mlp"], w, p + "mlp.", eps)
      x = x + mult * layer_norm(y, w[p + "norm2b"], eps)
    rows.append(x)
    x = depth_average(rows, w[p + "dwa"])
    if layers_out is not None:
      layers_out.append(x.clone())
  return layer_norm(x, w["final.norm"], eps) @ w["head"].T
