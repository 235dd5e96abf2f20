"""Plain CPU implementation of the Kuzezen decoder: one function per mechanism, one token loop or one
dense matrix per step, no cache, no batching.  It shares nothing with the product path; tests compare
the kernels and the model with it.

A configuration is the plain dictionary of a config.json; weights are a dictionary of tensors by
their file names, linear weights stored [out, in].
"""
from __future__ import annotations

import math

import torch


def rms(x, eps):
  """The last axis divided by sqrt(mean(x^2) + eps)."""
  return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def gelu_tanh(z):
  return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def sigmoid(z):
  return 1.0 / (1.0 + torch.exp(-z))


def log_sigmoid(z):
  return torch.minimum(z, torch.zeros_like(z)) - torch.log1p(torch.exp(-z.abs()))


def soft_cap(z, cap):
  return cap * torch.tanh(z / cap)


def causal_conv(u, taps, before=None):
  """u [T, C], taps [C, K]: out[t, c] = sum_j taps[c, K-1-j] u[t-j, c]; rows in front of the first one are
  `before` [K-1, C] (zeros at the start of a sequence)."""
  T, K = u.shape[0], taps.shape[1]
  if before is None:
    before = torch.zeros(K - 1, u.shape[1], dtype=u.dtype)
  full = torch.cat([before, u])
  out = torch.zeros_like(u)
  for k in range(K):
    out = out + taps[:, k] * full[k:k + T]
  return out


def query_temperature(positions, coef, every):
  """1 + coef ln(floor((p + 1) / every) + 1)."""
  return 1.0 + coef * torch.log(torch.floor((positions.to(torch.float64) + 1.0) / every) + 1.0)


def mixed_attention(q, k, v, scale, talk):
  """q [T, H, n], k [T, G, n], v [T, G, m] -> [T, H, m]: causal softmax per head, the heads' weights mixed by
  talk [H, H], each head's mixed weights applied to the values of its own group."""
  T, H, _ = q.shape
  R = H // k.shape[1]
  seen = torch.tril(torch.ones(T, T, dtype=torch.bool))
  weights = []
  for h in range(H):
    s = torch.where(seen, (q[:, h] @ k[:, h // R].T) * scale, torch.full((T, T), -math.inf, dtype=q.dtype))
    e = torch.exp(s - s.max(-1, keepdim=True).values)
    weights.append(e / e.sum(-1, keepdim=True))
  out = torch.empty(T, H, v.shape[-1], dtype=q.dtype)
  for h in range(H):
    out[:, h] = sum(talk[h, g] * weights[g] for g in range(H)) @ v[:, h // R]
  return out


def matrix_memory(q, k, v, log_i, log_f, state=None):
  """q, k [T, H, n], v [T, H, m], log gates [T, H].  Per head, with the running maximum M:
  M' = max(f + M, i), S' = e^(f + M - M') S + e^(i - M') k v^T, N' the same with k alone,
  o = S'^T q / (max(|N'.q|, e^(-M')) + 1e-6).  Returns (o, (S [H, n, m], N [H, n], M [H]))."""
  T, H, n = q.shape
  if state is None:
    S, N, M = torch.zeros(H, n, v.shape[-1], dtype=q.dtype), torch.zeros(H, n, dtype=q.dtype), torch.zeros(H, dtype=q.dtype)
  else:
    S, N, M = (x.clone() for x in state)
  out = torch.empty_like(v)
  for t in range(T):
    top = torch.maximum(log_f[t] + M, log_i[t])
    keep, add = torch.exp(log_f[t] + M - top), torch.exp(log_i[t] - top)
    S = keep[:, None, None] * S + add[:, None, None] * k[t][:, :, None] * v[t][:, None, :]
    N = keep[:, None] * N + add[:, None] * k[t]
    M = top
    num = (S * q[t][:, :, None]).sum(1)
    den = torch.maximum((N * q[t]).sum(-1).abs(), torch.exp(-M)) + 1e-6
    out[t] = num / den[:, None]
  return out, (S, N, M)


def attention_mixer(h, w, p, m, positions, eps):
  T, H, G, n, vd = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
  q, k, v = (causal_conv(h @ w[p + x].T, w[p + x + ".conv"]) for x in "qkv")
  q = q * query_temperature(positions, m["q_temp"]["coef"], m["q_temp"]["every"]).to(q.dtype)[:, None]
  o = mixed_attention(q.view(T, H, n), k.view(T, G, n), rms(v.view(T, G, vd), eps), m["scale"], w[p + "talk"])
  return (o.reshape(T, H * vd) * sigmoid(h @ w[p + "g"].T)) @ w[p + "o"].T


def memory_mixer(h, w, p, m, eps):
  T, H, n, vd, cap = h.shape[0], m["heads"], m["dim"], m["vdim"], m["gate_cap"]
  q, k, v = (h @ w[p + x].T for x in "qkv")
  log_i = soft_cap(h @ w[p + "i"].T + w[p + "i.b"], cap)
  log_f = log_sigmoid(soft_cap(h @ w[p + "f"].T + w[p + "f.b"], cap))
  o, _ = matrix_memory(q.view(T, H, n) * n ** -0.5, k.view(T, H, n), v.view(T, H, vd), log_i, log_f)
  o = rms(o, eps).reshape(T, H * vd) * w[p + "norm"] * sigmoid(h @ w[p + "g"].T)
  return o @ w[p + "o"].T


def parallel_mixer(h, w, p, m, positions, eps):
  a = rms(attention_mixer(h, w, p + "left.", m["left"], positions, eps), eps) * w[p + "left.out"]
  b = rms(memory_mixer(h, w, p + "right.", m["right"], eps), eps) * w[p + "right.out"]
  return 0.5 * (a + b)


def dense_mlp(h, w, p):
  return (gelu_tanh(h @ w[p + "gate"].T) * (h @ w[p + "up"].T)) @ w[p + "down"].T


def running_order(cfg):
  """(layer, number of the loop's pass that begins with it or None) in running order."""
  n, lp = len(cfg["layers"]), cfg.get("loop")
  if lp is None:
    return [(i, None) for i in range(n)]
  out = [(i, None) for i in range(lp["start"])]
  for t in range(lp["times"]):
    out += [(i, t if i == lp["start"] else None) for i in range(lp["start"], lp["stop"])]
  return out + [(i, None) for i in range(lp["stop"], n)]


def forward(cfg, weights, tokens, dtype=torch.float32, layers_out=None):
  """Logits [T, vocab] of one sequence; layers_out, a list, receives the residual after each layer run."""
  w = {k: v.to(dtype) for k, v in weights.items()}
  eps = cfg["norm"]["eps"]
  tokens = torch.as_tensor(tokens, dtype=torch.int64)
  positions = torch.arange(tokens.numel())
  x = w["embed"][tokens] * cfg["embedding"]["scale"]
  for i, begins in running_order(cfg):
    p, ly = f"l{i}.", cfg["layers"][i]
    if begins is not None:
      x = x + w["loop.step"][begins]
    h = rms(x, eps) * w[p + "norm1"]
    y = parallel_mixer(h + causal_conv(h, w[p + "canon1"]), w, p + "mix.", ly["mixer"], positions, eps)
    if ly["mlp"] is not None:
      y = y + dense_mlp(h + causal_conv(h, w[p + "canon2"]), w, p + "mlp.")
    x = x + cfg["residual_mult"] * y
    if layers_out is not None:
      layers_out.append(x)
  return soft_cap((rms(x, eps) * w["final.norm"]) @ w["head"].T, cfg["logit_softcap"])


def tensor_shapes(cfg):
  """File name -> shape of every tensor of a configuration."""
  D, V, taps = cfg["width"], cfg["vocab"], cfg["canon"]["taps"]
  out = {"embed": (V, D), "final.norm": (D,), "head": (V, D)}
  if cfg.get("loop") is not None:
    out["loop.step"] = (cfg["loop"]["times"], D)
  for i, ly in enumerate(cfg["layers"]):
    p, a, b = f"l{i}.", ly["mixer"]["left"], ly["mixer"]["right"]
    out.update({p + "norm1": (D,), p + "canon1": (D, taps)})
    x, H, G = p + "mix.left.", a["heads"], a["kv_heads"]
    for name, rows in (("q", H * a["dim"]), ("k", G * a["dim"]), ("v", G * a["vdim"])):
      out.update({x + name: (rows, D), x + name + ".conv": (rows, a["conv"])})
    out.update({x + "talk": (H, H), x + "g": (H * a["vdim"], D), x + "o": (D, H * a["vdim"]), x + "out": (D,)})
    x, H = p + "mix.right.", b["heads"]
    qk, v = H * b["dim"], H * b["vdim"]
    out.update({x + "q": (qk, D), x + "k": (qk, D), x + "v": (v, D), x + "g": (v, D), x + "o": (D, v), x + "norm": (v,),
                x + "i": (H, D), x + "i.b": (H,), x + "f": (H, D), x + "f.b": (H,), x + "out": (D,)})
    if ly["mlp"] is not None:
      F = ly["mlp"]["ff"]
      out.update({p + "canon2": (D, taps), p + "mlp.gate": (F, D), p + "mlp.up": (F, D), p + "mlp.down": (D, F)})
  return out
