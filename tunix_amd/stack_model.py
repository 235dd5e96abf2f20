"""Decoders given as a list of layers (`config.StackConfig`), with dense weights and an fp32 residual
stream: `StackModel` holds the weights on one GPU, `StackRunner` is the kernel sequence of one
forward pass over T tokens per row.  The sampler, the rollout engine and the log-probability pass
drive them as they drive `QLoRAModel` and `Runner`.

Two dtypes: bf16 (matrix operands bf16, fp32 accumulation; the residual, norms, angles, scores,
softmax and recurrent states fp32) and fp32 (everything).
"""
from __future__ import annotations

import math

import numpy as np
import torch

from . import _lib as L
from . import ops
from .cache import KVSpec, SequenceCache, StateSpec
from .config import AttentionMixer, LightningMixer, StackConfig
from .model import HeadRunner


def _up(n: int, m: int) -> int:
  return (n + m - 1) // m * m


# rows up to which a pass keeps its activations in fragment order for the few-row linear kernel
FRAG_ROWS = 512


class DenseLinear:
  """One dense projection, possibly several weights [N_i, K] that share an input.  Every member
  starts at a multiple of 16 output columns (`offsets`), K is zero-padded to a multiple of 128.
  paired: two members of one shape whose rows alternate in blocks of 16 (gate | up), so that the
  kernel's epilogue finds both in one wave (bf16)."""

  def __init__(self, names: list[str], weights: dict, dtype, device, paired: bool = False):
    self.names, self.dtype, self.device, self.paired = names, dtype, device, paired
    self.shapes = [tuple(weights[n].shape) for n in names]
    self.K = self.shapes[0][1]
    self.Kp = _up(self.K, 128)
    widths = [_up(s[0], 16) for s in self.shapes]
    self.offsets = [sum(widths[:i]) for i in range(len(widths))]
    self.N = sum(widths)
    self.w = None
    self.load(weights)

  def check(self, weights: dict):
    for n, s in zip(self.names, self.shapes):
      if n not in weights:
        raise ValueError(f"New state must have the same structure as the old state: {n} is missing")
      if tuple(weights[n].shape) != s:
        raise ValueError(f"New state must have the same shape as the old state: {n} {tuple(weights[n].shape)} vs {s}")

  def load(self, weights: dict):
    self.check(weights)
    w = torch.zeros(self.N, self.Kp, dtype=self.dtype, device=self.device)
    for n, off in zip(self.names, self.offsets):
      src = weights[n].to(self.device, self.dtype)
      w[off:off + src.shape[0], :self.K] = src
    if self.dtype == torch.bfloat16:
      if self.paired:
        w = w.view(2, self.N // 32, 16, self.Kp).transpose(0, 1).reshape(self.N, self.Kp).contiguous()
      w = ops.dense_expand(w)
    if self.w is None:
      self.w = w
    else:   # in place: captured graphs keep their pointers
      self.w.copy_(w)

  def nbytes(self) -> int:
    return sum(a * b for a, b in self.shapes) * (2 if self.dtype == torch.bfloat16 else 4)


class StackModel:
  """Weights of one layer-list decoder on one GPU."""

  def __init__(self, cfg: StackConfig, weights: dict, device="cuda", dtype=torch.bfloat16):
    L.lib()  # fail loudly when the HIP library is missing
    if dtype not in ops.DTYPES:
      raise ValueError(f"dtype {dtype} is not one of {list(ops.DTYPES)}")
    self.cfg, self.device, self.dtype = cfg, torch.device(device), dtype
    self.shapes = cfg.weight_shapes()
    self._check_names(weights, complete=True)
    dev, V, D = self.device, cfg.vocab_size, cfg.embed_dim
    self.Dp = _up(D, 128)
    vec = lambda name: weights[name].to(dev, torch.float32).contiguous()
    self.embed = torch.zeros(V, D, dtype=dtype, device=dev)
    self.final_norm = vec("final.norm")
    self.linears: dict[str, DenseLinear] = {}
    self.vectors: dict[str, torch.Tensor] = {"final.norm": self.final_norm}

    def linear(names, paired=False):
      f = DenseLinear(names, weights, dtype, dev, paired)
      for n in names:
        self.linears[n] = f
      return f

    def vector(name):
      self.vectors[name] = vec(name)
      return self.vectors[name]

    self.loop_in = linear(["loop.in"]) if cfg.loop is not None else None
    self.layers = []
    for i, spec in enumerate(cfg.layers):
      p, m = f"l{i}.", spec.mixer
      ly = {"spec": spec, "norm1": vector(p + "norm1"), "norm1b": vector(p + "norm1b")}
      if isinstance(m, AttentionMixer):
        ly["in"] = linear([p + "mix.q", p + "mix.k", p + "mix.v"])
        ly["sink"] = vector(p + "mix.sink") if m.sink else None
        freq = np.float64(m.rot_base) ** (-2.0 * np.arange(m.rot_dims // 2) / max(m.rot_dims, 1))
        ly["inv_freq"] = torch.from_numpy(freq.astype(np.float32)).to(dev)
      else:
        ly["in"] = linear([p + "mix.q", p + "mix.k", p + "mix.v", p + "mix.g"])
        ly["norm"] = vector(p + "mix.norm")
        ly["decay"] = torch.tensor(m.decay, dtype=torch.float32, device=dev)
      ly["out"] = linear([p + "mix.o"])
      if spec.mlp is not None:
        ly["norm2"], ly["norm2b"] = vector(p + "norm2"), vector(p + "norm2b")
        ly["gu"] = linear([p + "mlp.gate", p + "mlp.up"], paired=True)
        ly["down"] = linear([p + "mlp.down"])
      self.layers.append(ly)
    # the head is the embedding table: through the statistics head when its shape is one that
    # kernel takes, else as a plain linear into fp32 logits
    self.head = self.head_w = self.head_expanded = None
    self.block_head = dtype == torch.bfloat16 and D % 128 == 0 and V % 16 == 0
    self.head_linear = None
    self._load_embed(weights["embed"])
    torch.cuda.synchronize(dev)

  def _load_embed(self, table):
    self.embed.copy_(table.to(self.device, self.dtype))
    if self.block_head:
      if self.head_expanded is None:
        self.head_expanded = ops.dense_expand(self.embed)
      else:
        self.head_expanded.copy_(ops.dense_expand(self.embed))
    elif self.head_linear is None:
      self.head_linear = DenseLinear(["embed"], {"embed": self.embed}, self.dtype, self.device)
    else:
      self.head_linear.load({"embed": self.embed})

  def _check_names(self, weights: dict, complete: bool):
    extra = sorted(set(weights) - set(self.shapes))
    missing = sorted(set(self.shapes) - set(weights)) if complete else []
    if extra or missing:
      raise ValueError(f"New state must have the same structure as the old state. missing={missing} extra={extra}")
    for n, t in weights.items():
      if tuple(t.shape) != self.shapes[n]:
        raise ValueError(f"New state must have the same shape as the old state: {n} {tuple(t.shape)} vs {self.shapes[n]}")

  # ---- what the sampler asks of a model ------------------------------------------------------
  def cache_specs(self) -> list:
    specs = []
    for i, _ in self.cfg.layer_runs:
      m = self.cfg.layers[i].mixer
      if isinstance(m, AttentionMixer):
        specs.append(KVSpec(m.kv_heads, ops.sink_attn_pad(m.dim, False, self.dtype),
                            ops.sink_attn_pad(m.vdim, True, self.dtype), self.dtype))
      else:
        specs.append(StateSpec(m.heads, m.dim, m.vdim))
    return specs

  def new_cache(self, B: int, S: int, shared: bool = False) -> SequenceCache:
    return SequenceCache(self.cache_specs(), B, S, self.device, shared=shared)

  def new_runner(self, B: int, T: int, S: int, pad_id: int, **kw) -> "StackRunner":
    return StackRunner(self, B, T, S, pad_id, **kw)

  def update_lora(self, new_lora: dict):
    if new_lora:
      raise ValueError(f"New state must have the same structure as the old state. extra={sorted(new_lora)}")

  def update_params(self, new_state: dict):
    """Replaces parameters by name; the members of a fused projection come together.  A rejected
    state changes nothing."""
    self._check_names(new_state, complete=False)
    owners = {id(f): f for n, f in self.linears.items() if n in new_state}
    for f in owners.values():
      f.check(new_state)
    for f in owners.values():
      f.load(new_state)
    for n, t in new_state.items():
      if n in self.vectors:
        self.vectors[n].copy_(t.to(self.device, torch.float32))
    if "embed" in new_state:
      self._load_embed(new_state["embed"])
    torch.cuda.synchronize(self.device)

  def weight_bytes(self) -> dict:
    """Bytes one decode step reads: the linears (a looped layer's once per pass) and the head."""
    n = 0
    for i, begins in self.cfg.layer_runs:
      ly = self.layers[i]
      n += sum(ly[k].nbytes() for k in ("in", "out", "gu", "down") if k in ly)
      n += self.loop_in.nbytes() if begins else 0
    return {"dense": n, "head": self.embed.numel() * self.embed.element_size()}


class StackRunner(HeadRunner):
  """Workspaces + the kernel sequence for B*T token rows.  Token buffer, cache and step counter
  belong to the caller; kernels read the column from device memory, so a decode step can be
  captured into a HIP graph and replayed."""

  def __init__(self, model: StackModel, B: int, T: int, S: int, pad_id: int, kv_chunk=None,
               want_logits: bool = False, split_k_override: dict | None = None):
    cfg = model.cfg
    self.model, self.cfg, self.B, self.T, self.S = model, cfg, B, T, S
    self.pad_id = int(pad_id)
    self.dtype, dev = model.dtype, model.device
    M = B * T
    self.M = M
    self.code = ops.DTYPES[self.dtype]
    # few rows: activations in fragment order, for the few-row linear kernel
    self.frag = self.dtype == torch.bfloat16 and M <= FRAG_ROWS
    self._bufs: dict = {}
    D = cfg.embed_dim
    self.x = torch.empty(M, D, dtype=torch.float32, device=dev)
    # the final-normed rows (row-major, zero columns behind the model width)
    width = D if model.block_head else model.Dp
    self.xn = torch.zeros(M, width, dtype=self.dtype, device=dev)
    self.split_k_override = dict(split_k_override or {})
    n_y = n_ws = n_light = n_attn = 1
    for i, begins in cfg.layer_runs:
      ly = model.layers[i]
      m = ly["spec"].mixer
      for key in ("in", "out", "gu", "down"):
        if key in ly:
          f = ly[key]
          n_y = max(n_y, M * f.N)
          n_ws = max(n_ws, self._split(f) * M * f.N if self._split(f) > 1 else 1)
      if begins:
        n_ws = max(n_ws, self._split(model.loop_in) * M * model.loop_in.N)
      if isinstance(m, LightningMixer):   # (a call may bring fewer rows, and cut them into more spans)
        n_light = max([n_light] + [ops.lightning_ws_bytes(b, T, m.heads, m.dim, m.vdim) // 4 for b in range(1, B + 1)])
      else:
        n_attn = max(n_attn, ops.sink_attn_ws_bytes(B, T, S, m.heads, ops.sink_attn_pad(m.vdim, True, self.dtype),
                                                    self._kv_chunk(m, kv_chunk)) // 4)
    self.kv_chunk_arg = kv_chunk
    self.y = torch.empty(n_y, dtype=self.dtype, device=dev)
    self.ws = torch.empty(n_ws, dtype=torch.float32, device=dev)
    self.light_ws = torch.empty(n_light, dtype=torch.float32, device=dev)
    self.attn_ws = torch.empty(n_attn, dtype=torch.float32, device=dev)
    self.zero = torch.zeros(1, dtype=torch.int32, device=dev)
    self.no_starts = torch.zeros(B, dtype=torch.int32, device=dev)
    self.block_stats = model.block_head
    self._init_head(B, width, self.dtype, want_logits)
    self._head_logits = None
    if not model.block_head:
      self._head_logits = self.logits if self.logits is not None else torch.empty(
          B, cfg.vocab_size, dtype=torch.float32, device=dev)
    self.residual_sink = None   # called with the fp32 residual [M, D] behind every layer run

  # ---- building blocks -----------------------------------------------------------------------
  def _buf(self, name: str, cols: int, dtype=None) -> torch.Tensor:
    """Activation buffer [rows, cols], zero where nothing is ever written (the padding columns of a
    linear's input must be zero); whole blocks of 128 rows for the fragment order."""
    key = (name, cols)
    if key not in self._bufs:
      rows = _up(self.M, 128) if self.frag else self.M
      self._bufs[key] = torch.zeros(rows, cols, dtype=self.dtype if dtype is None else dtype, device=self.model.device)
    return self._bufs[key]

  def _kv_chunk(self, m: AttentionMixer, given) -> int:
    """Decode: split the key range only as far as needed to put about a thousand waves on the device."""
    if given is not None:
      return given
    waves = self.B * m.kv_heads * math.ceil(self.T * (m.heads // m.kv_heads) / 16)
    if self.dtype != torch.bfloat16 or self.T != 1 or waves >= 1024 or self.S <= 64:
      return 0
    n = min(math.ceil(1024 / waves), self.S // 32)
    chunk = max(32, _up(math.ceil(self.S / n), 32))
    return 0 if chunk >= self.S else chunk

  def _split(self, f: DenseLinear) -> int:
    """k split of a few-row linear whose reader sums fp32 planes."""
    key = f.names[0].split(".")[-1]
    if key in self.split_k_override:
      return self.split_k_override[key]
    if not self.frag or f.paired:
      return 1
    groups = math.ceil(f.N / 64) * math.ceil(self.M / 128)
    return int(max(1, min(8, (256 if self.M > 32 else 512) // groups, f.Kp // 512)))

  def linear(self, f: DenseLinear, x, M: int, fp32_out: bool = False) -> L.RowsSrc:
    """Runs one projection of x [M, f.Kp]; returns its output as the reading kernel wants it."""
    d = L.DenseDesc()
    d.M, d.K, d.N, d.dtype = M, f.Kp, f.N, self.code
    d.x, d.ldx, d.x_frag, d.w = x.data_ptr(), x.shape[1], 1 if self.frag else 0, f.w.data_ptr()
    d.ldy, d.split_k = f.N, self._split(f)
    src = L.RowsSrc()
    src.ld, src.plane, src.split_k = f.N, M * f.N, d.split_k
    if d.split_k > 1:
      d.epilogue, d.ws = L.TNX_EPI_F32, self.ws.data_ptr()
      src.ws = d.ws
    elif fp32_out and self.dtype != torch.float32:
      d.epilogue, d.y = L.TNX_EPI_F32, self.ws.data_ptr()
      src.ws = d.y
    else:
      d.epilogue, d.y = L.TNX_EPI_STORE, self.y.data_ptr()
      src.y = d.y
    ops.dense_linear(d)
    return src

  def residual_norm(self, pending, w_next, out, M: int, frag: bool):
    """x takes what is pending (None, ("add", rows, post-norm weight) or ("set", rows, None));
    out = norm(x) . w_next, or x itself when w_next is None."""
    cfg = self.cfg
    d = L.ResidualNormDesc()
    d.M, d.D, d.dtype, d.eps, d.w_offset = M, cfg.embed_dim, self.code, cfg.norm_eps, cfg.norm_offset
    if pending is not None:
      kind, d.y, w_post = pending
      d.mode = 1 if kind == "add" else 2
      d.w_post = None if w_post is None else w_post.data_ptr()
    d.x, d.w_next = self.x.data_ptr(), None if w_next is None else w_next.data_ptr()
    d.out, d.out_ld, d.out_frag = out.data_ptr(), out.shape[1], 1 if frag else 0
    ops.residual_norm(d)

  def rotate(self, ly, src, entry, col_ptr, starts, B, T):
    """Rotates q and k of an attention layer's projection and writes the cache; returns q."""
    m, f = ly["spec"].mixer, ly["in"]
    dkp, dvp = entry.k.shape[3], entry.v.shape[3]
    q = self._buf("q", m.heads * dkp)
    d = L.PartRopeDesc()
    d.B, d.T, d.S, d.H, d.G = B, T, entry.k.shape[2], m.heads, m.kv_heads
    d.dk, d.dv, d.dkp, d.dvp, d.rot_dims, d.dtype = m.dim, m.vdim, dkp, dvp, m.rot_dims, self.code
    d.inv_freq, d.y, d.k_off, d.v_off = ly["inv_freq"].data_ptr(), src, f.offsets[1], f.offsets[2]
    d.starts, d.col_ptr = starts.data_ptr(), col_ptr.data_ptr()
    d.q_out, d.kcache, d.vcache = q.data_ptr(), entry.k.data_ptr(), entry.v.data_ptr()
    ops.part_rope_kvwrite(d)
    return q

  def attend(self, ly, q, entry, col_ptr, starts, B, T) -> torch.Tensor:
    m = ly["spec"].mixer
    out = self._buf("attn", ly["out"].Kp)
    d = L.SinkAttnDesc()
    d.B, d.T, d.S, d.H, d.G = B, T, entry.k.shape[2], m.heads, m.kv_heads
    d.dk, d.dv, d.dkp, d.dvp, d.scale, d.dtype = m.dim, m.vdim, entry.k.shape[3], entry.v.shape[3], m.scale, self.code
    d.q, d.kcache, d.vcache = q.data_ptr(), entry.k.data_ptr(), entry.v.data_ptr()
    d.sinks = None if ly["sink"] is None else ly["sink"].data_ptr()
    d.starts, d.col_ptr = starts.data_ptr(), col_ptr.data_ptr()
    d.kv_chunk = self._kv_chunk(m, self.kv_chunk_arg) if T == 1 else 0
    d.ws, d.out, d.out_ld, d.out_frag = self.attn_ws.data_ptr(), out.data_ptr(), out.shape[1], 1 if self.frag else 0
    ops.sink_attn(d)
    return out

  def recur(self, ly, src, entry, col_ptr, starts, B, T) -> torch.Tensor:
    """The lightning recurrence of a projection's rows: fp32 [rows, heads * vdim]."""
    m, f = ly["spec"].mixer, ly["in"]
    o = self._buf("state_out", m.heads * m.vdim, torch.float32)
    d = L.LightningDesc()
    d.B, d.T, d.H, d.dk, d.dv, d.dtype = B, T, m.heads, m.dim, m.vdim, self.code
    d.decay, d.y, d.k_off, d.v_off = ly["decay"].data_ptr(), src, f.offsets[1], f.offsets[2]
    d.starts, d.col_ptr, d.state = starts.data_ptr(), col_ptr.data_ptr(), entry.s.data_ptr()
    d.o, d.o_ld, d.ws = o.data_ptr(), o.shape[1], self.light_ws.data_ptr()
    ops.lightning(d)
    return o

  def gate(self, ly, o, src, M: int) -> torch.Tensor:
    """norm(o) . weight * sigmoid(gate columns of the projection)."""
    out = self._buf("gated", ly["out"].Kp)
    d = L.GatedNormDesc()
    d.M, d.W, d.dtype, d.eps, d.w_offset = M, o.shape[1], self.code, self.cfg.norm_eps, 0.0
    d.o, d.o_ld, d.g, d.g_off, d.w = o.data_ptr(), o.shape[1], src, ly["in"].offsets[3], ly["norm"].data_ptr()
    d.out, d.out_ld, d.out_frag = out.data_ptr(), out.shape[1], 1 if self.frag else 0
    ops.gated_norm(d)
    return out

  def _mixer(self, ly, h, entry, col_ptr, starts, B, T) -> L.RowsSrc:
    src = self.linear(ly["in"], h, B * T)
    if isinstance(ly["spec"].mixer, AttentionMixer):
      q = self.rotate(ly, src, entry, col_ptr, starts, B, T)
      out = self.attend(ly, q, entry, col_ptr, starts, B, T)
    else:
      out = self.gate(ly, self.recur(ly, src, entry, col_ptr, starts, B, T), src, B * T)
    return self.linear(ly["out"], out, B * T)

  def gate_up(self, ly, h, M: int) -> torch.Tensor:
    f = ly["gu"]
    act = self._buf("act", ly["down"].Kp)
    if self.dtype == torch.float32:
      self.linear(f, h, M)
      ops.gelu_mul(self.y[:M * f.N].view(M, f.N), f.offsets[1], M, ly["spec"].mlp.ff, act)
    else:
      d = L.DenseDesc()
      d.M, d.K, d.N, d.dtype = M, f.Kp, f.N, self.code
      d.x, d.ldx, d.x_frag, d.w = h.data_ptr(), h.shape[1], 1 if self.frag else 0, f.w.data_ptr()
      d.epilogue, d.y, d.ldy, d.y_frag, d.split_k = L.TNX_EPI_GELU_MUL, act.data_ptr(), act.shape[1], 1 if self.frag else 0, 1
      ops.dense_linear(d)
    return act

  def forward_hidden(self, tokens, positions, col_ptr, cache, B=None, T=None, segment_ids=None, starts=None):
    """Runs all layers for tokens[b, col .. col+T) of each row from what `cache` holds of the columns
    before; leaves the final-normed hidden rows in self.xn[:B*T].  starts (int32 [B]): the column of
    each row's first token; positions count from there (`positions` is not read)."""
    if segment_ids is not None:
      raise ValueError("packed batches are not part of layer-list decoders: one sequence per row")
    m, cfg = self.model, self.cfg
    B = self.B if B is None else B
    T = self.T if T is None else T
    M = B * T
    starts = self.no_starts if starts is None else starts
    D = cfg.embed_dim
    cat = None if m.loop_in is None else self._buf("cat", m.loop_in.Kp)
    ops.embed_rows(m.embed, tokens, col_ptr, B, T, cfg.vocab_size, D, self.x, cat=cat, cat_off=D, cat_frag=self.frag)
    h = self._buf("h", m.Dp)
    pending, behind_layer = None, False

    def norm(w_next, out, frag):
      nonlocal behind_layer
      self.residual_norm(pending, w_next, out, M, frag)
      if behind_layer and self.residual_sink is not None:
        self.residual_sink(self.x[:M])
      behind_layer = False

    for (i, begins), entry in zip(cfg.layer_runs, cache.entries):
      ly = m.layers[i]
      if begins:   # a pass of the loop: x <- W [x; embedding output]
        norm(None, cat, self.frag)
        pending = ("set", self.linear(m.loop_in, cat, M, fp32_out=True), None)
      norm(ly["norm1"], h, self.frag)
      pending = ("add", self._mixer(ly, h, entry, col_ptr, starts, B, T), ly["norm1b"])
      if "gu" in ly:
        norm(ly["norm2"], h, self.frag)
        pending = ("add", self.linear(ly["down"], self.gate_up(ly, h, M), M), ly["norm2b"])
      behind_layer = True
    norm(m.final_norm, self.xn, False)
    return self.xn

  # ---- head ----------------------------------------------------------------------------------
  def run_head(self, x, rows, temperature=1.0, targets=None, best_id=None, best_logp=None, target_logp=None, lse=None,
               logits_out=None, forbidden=None, entropy=None, part_entropy=None, draw=None, logits_fp32=False):
    m = self.model
    if m.block_head:
      return super().run_head(x, rows, temperature=temperature, targets=targets, best_id=best_id, best_logp=best_logp,
                              target_logp=target_logp, lse=lse, logits_out=logits_out, forbidden=forbidden,
                              entropy=entropy, part_entropy=part_entropy, draw=draw, logits_fp32=logits_fp32)
    V, f = self.cfg.vocab_size, m.head_linear
    if logits_out is None:
      logits_out = (self._head_logits if rows <= self._head_logits.shape[0]
                    else torch.empty(rows, V, dtype=torch.float32, device=m.device))
    d = L.DenseDesc()
    d.M, d.K, d.N, d.dtype = rows, f.Kp, V, self.code
    d.x, d.ldx, d.w, d.epilogue = x.data_ptr(), x.shape[1], f.w.data_ptr(), L.TNX_EPI_F32
    d.y, d.ldy, d.split_k = logits_out.data_ptr(), V, 1
    ops.dense_linear(d)
    s = L.LogitsDesc()
    s.M, s.V, s.logits, s.temperature = rows, V, logits_out.data_ptr(), float(temperature)
    if forbidden is not None:
      s.forbidden, s.n_forbidden = forbidden.data_ptr(), forbidden.numel()
    for name, t in (("targets", targets), ("best_id", best_id), ("best_logp", best_logp), ("target_logp", target_logp),
                    ("lse", lse), ("entropy", entropy)):
      if t is not None:
        setattr(s, name, t.data_ptr())
    if draw is not None:
      s.draw_key0, s.draw_key1, s.draw_rng_variant = int(draw["key"][0]), int(draw["key"][1]), int(draw["variant"])
      s.draw_step_ptr, s.draw_id = draw["step"].data_ptr(), draw["ids"].data_ptr()
      if draw.get("logp") is not None:
        s.draw_logp = draw["logp"].data_ptr()
    if any(t is not None for t in (best_id, best_logp, target_logp, lse, entropy, draw)):
      ops.logits_stats(s)
