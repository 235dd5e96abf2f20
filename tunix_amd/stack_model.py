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
from .cache import BorrowedSpec, KVSpec, LatentSpec, PartsSpec, RingSpec, SequenceCache, StateSpec
from .config import AttentionMixer, ExpertsMlp, GatedStateMixer, LatentMixer, LightningMixer, MemoryMixer, MixedAttentionMixer, ParallelMixer, PolyNormMlp, SsdMixer, StackConfig
from .model import HeadRunner


def _up(n: int, m: int) -> int:
  return (n + m - 1) // m * m


# rows up to which a pass keeps its activations in fragment order for the few-row linear kernel
FRAG_ROWS = 512


class DenseLinear:
  """One dense projection, possibly several weights [N_i, K] that share an input.  A member is a name, or
  (name, first row, end row) for some rows of a weight.  Every member starts at a multiple of `align` (16) output
  columns (`offsets`), K is zero-padded to a multiple of 128.  Runs of 256 columns lie behind each other in memory: at an
  offset that is a multiple of 256 a call may begin or end.
  inputs: columns [first, end) of the members that take part, all by default.
  paired: two members of one shape whose rows alternate in blocks of 16 (gate | up), so that the
  kernel's epilogue finds both in one wave (bf16).  transpose: the members' transposes."""

  def __init__(self, members: list, weights: dict, dtype, device, paired: bool = False, transpose: bool = False, align: int = 16, inputs: tuple | None = None):
    self.members = [m if isinstance(m, tuple) else (m, 0, weights[m].shape[0]) for m in members]
    self.names, self.dtype, self.device, self.paired = [m[0] for m in self.members], dtype, device, paired
    self.transpose = transpose
    self.full_shapes = [tuple(weights[n].shape) for n in self.names]
    self.inputs = inputs or (0, self.full_shapes[0][1])
    self.shapes = [(r1 - r0, self.inputs[1] - self.inputs[0])[::-1 if transpose else 1] for (_, r0, r1), s in zip(self.members, self.full_shapes)]
    self.K = self.shapes[0][1]
    self.Kp = _up(self.K, 128)
    widths = [_up(s[0], align) for s in self.shapes]
    self.offsets = [sum(widths[:i]) for i in range(len(widths))]
    self.N = sum(widths)
    self.w = None
    self.load(weights)

  def check(self, weights: dict):
    for n, s in zip(self.names, self.full_shapes):
      if n not in weights:
        raise ValueError(f"New state must have the same structure as the old state: {n} is missing")
      if tuple(weights[n].shape) != s:
        raise ValueError(f"New state must have the same shape as the old state: {n} {tuple(weights[n].shape)} vs {s}")

  def load(self, weights: dict):
    self.check(weights)
    w = torch.zeros(self.N, self.Kp, dtype=self.dtype, device=self.device)
    for (n, r0, r1), off in zip(self.members, self.offsets):
      src = weights[n][r0:r1, self.inputs[0]:self.inputs[1]].to(self.device, self.dtype)
      src = src.T if self.transpose else src
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


class LinearBank:
  """Projections of one shape behind each other in memory: experts, or one per head."""

  def __init__(self, linears: list[DenseLinear]):
    self.linears = linears
    first = linears[0]
    self.w = torch.stack([f.w for f in linears])
    for f, w in zip(linears, self.w):   # (a member's load writes into the bank)
      f.w = w
    self.K, self.Kp, self.N, self.shapes, self.offsets = first.K, first.Kp, first.N, first.shapes, first.offsets
    self.stride = self.w[0].numel()

  def __len__(self) -> int:
    return len(self.linears)

  def nbytes(self) -> int:
    return sum(f.nbytes() for f in self.linears)


class LinearPart:
  """Some members of a projection, where a layer reads only them."""

  def __init__(self, linear: DenseLinear, first: int, count: int):
    self.linear, self.offsets = linear, linear.offsets[first:first + count]


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
    self.linears: dict[str, list[DenseLinear]] = {}    # the projections a weight takes part in
    self.transposed: set[str] = set()                  # vectors kept as [taps, channels]
    self.vectors: dict[str, torch.Tensor] = {"final.norm": self.final_norm}

    def linear(members, paired=False, transpose=False, align=16, inputs=None):
      f = DenseLinear(members, weights, dtype, dev, paired, transpose, align, inputs)
      for n in dict.fromkeys(f.names):
        self.linears.setdefault(n, []).append(f)
      return f

    def vector(name):
      self.vectors[name] = vec(name)
      return self.vectors[name]

    def taps(name, buf=None):
      """A convolution's weights [channels, taps] as [taps, channels], of their own or in given columns."""
      t = vec(name).T
      if buf is None:
        buf = torch.empty(t.shape, dtype=torch.float32, device=dev)
      buf.copy_(t)
      self.vectors[name] = buf
      self.transposed.add(name)
      return buf

    self.pos = torch.empty(cfg.max_positions, D, dtype=dtype, device=dev) if cfg.max_positions else None
    self.embed_norm = vector("embed.norm") if cfg.embed_norm else None
    looped = cfg.loop is not None
    self.loop_in = linear(["loop.in"]) if looped and not cfg.loop.step else None
    self.loop_step = vector("loop.step") if looped and cfg.loop.step else None
    self.layers = []
    for i, spec in enumerate(cfg.layers):
      p, m = f"l{i}.", spec.mixer
      ly = {"spec": spec, "norm1": vector(p + "norm1") if cfg.pre_norm else None, "post1": None if cfg.parallel else vector(p + cfg.post_norm(1))}
      if cfg.token_shift:
        ly["shift"] = vector(p + "shift")
      if cfg.depth_average:
        ly["dwa"] = vector(p + "dwa")
      if isinstance(m, SsdMixer):
        x = p + "mix."
        ly["in"] = linear([(x + "in", 0, m.inner), (x + "in", m.inner, m.inner + m.channels),
                           (x + "in", m.inner + m.channels, m.inner + m.channels + m.heads)])
        ly["conv"] = taps(x + "conv")
        for key, name in (("conv_b", "conv.b"), ("dt_bias", "dt_bias"), ("A_log", "A_log"), ("D", "D"), ("norm", "norm")):
          ly[key] = vector(x + name)
      elif isinstance(m, LatentMixer):
        x = p + "mix."
        ly["in"] = linear([x + "dq", x + "dkv", x + "g"])
        ly["uq"], ly["ukv"] = linear([x + "uq"]), linear([x + "uk", x + "uv"])
        # the key projection applied to a head's query, the value projection to its weighted latent
        ly["absorb_k"] = LinearBank([linear([(x + "uk", h * m.dim, (h + 1) * m.dim)], transpose=True) for h in range(m.heads)])
        ly["absorb_v"] = LinearBank([linear([(x + "uv", h * m.vdim, (h + 1) * m.vdim)]) for h in range(m.heads)])
        ly["q_norm"], ly["kv_norm"] = vector(x + "dq.norm"), vector(x + "dkv.norm")
        freq = np.float64(m.rot_base) ** (-2.0 * np.arange(m.rot_dim // 2) / max(m.rot_dim, 1))
        ly["inv_freq"] = torch.from_numpy(freq.astype(np.float32)).to(dev)
      elif isinstance(m, ParallelMixer):
        # everything that reads the input is one projection, but the memory's gates: they stay fp32
        a, b = p + "mix.left.", p + "mix.right."
        f = ly["in"] = linear([x + n for x in (a, b) for n in "qkvg"])
        left = {"spec": type(spec)(m.left, None), "in": LinearPart(f, 0, 4), "out": linear([a + "o"]), "post": vector(a + "out"), "talk": vector(a + "talk")}
        n_conv = f.offsets[3] - f.offsets[0]
        left["conv"] = torch.zeros(m.left.conv, n_conv, dtype=torch.float32, device=dev)
        for n, off, size in zip("qkv", f.offsets, f.shapes):
          taps(a + n + ".conv", left["conv"][:, off:off + size[0]])
        right = {"spec": type(spec)(m.right, None), "in": LinearPart(f, 4, 4), "out": linear([b + "o"]), "post": vector(b + "out"), "gates": linear([b + "i", b + "f"]),
                 "bias_i": vector(b + "i.b"), "bias_f": vector(b + "f.b"), "norm": vector(b + "norm")}
        ly["left"], ly["right"] = left, right
        ly["canon1"] = taps(p + "canon1")
        if spec.mlp is not None:
          ly["canon2"] = taps(p + "canon2")
      elif isinstance(m, GatedStateMixer):
        # (the gates' columns begin at a run of 256, so that a prompt pass can keep them, and only them, in fp32)
        ly["in"] = linear([p + "mix.q", p + "mix.v", p + "mix.f"], align=256)
        ly["bias"], ly["lower"], ly["norm"] = vector(p + "mix.f.b"), vector(p + "mix.lower"), vector(p + "mix.norm")
      elif isinstance(m, AttentionMixer):
        ly["in"] = linear([p + "mix.q"] if m.kv_from is not None else [p + "mix.q", p + "mix.k", p + "mix.v"])
        if m.row_norm:
          ly["q_norm"], ly["k_norm"] = vector(p + "mix.q.norm"), None if m.kv_from is not None else vector(p + "mix.k.norm")
        ly["slopes"] = torch.tensor(m.slopes, dtype=torch.float32, device=dev) if m.slopes else None
        ly["sink"] = vector(p + "mix.sink") if m.sink else None
        freq = np.float64(m.rot_base) ** (-2.0 * np.arange(m.rot_dims // 2) / max(m.rot_dims, 1))
        ly["inv_freq"] = torch.from_numpy(freq.astype(np.float32)).to(dev)
      else:
        ly["in"] = linear([p + "mix.q", p + "mix.k", p + "mix.v", p + "mix.g"])
        ly["norm"] = vector(p + "mix.norm")
        ly["decay"] = torch.tensor(m.decay, dtype=torch.float32, device=dev)
      if not isinstance(m, ParallelMixer):
        ly["out"] = linear([p + "mix.o"])
      if spec.mlp is not None and not cfg.parallel:
        ly["norm2"], ly["post2"] = vector(p + "norm2") if cfg.pre_norm else None, vector(p + cfg.post_norm(2))
      if isinstance(spec.mlp, ExpertsMlp):
        e = [p + f"mlp.e{j}." for j in range(spec.mlp.experts)]
        parts = [(j * spec.mlp.ff, (j + 1) * spec.mlp.ff) for j in range(spec.mlp.shared_routes)]   # of the shared expert
        ly["router"] = linear([p + "mlp.router"] + ([p + "mlp.shared.sg"] if spec.mlp.shared_ff else []))
        ly["gu"] = LinearBank([linear([n + "gate", n + "up"], paired=True) if spec.mlp.gated else linear([n + "up"]) for n in e] +
                              [linear([(p + "mlp.shared.up", *r)]) for r in parts])
        ly["down"] = LinearBank([linear([n + "down"]) for n in e] + [linear([p + "mlp.shared.down"], inputs=r) for r in parts])
        if spec.mlp.corrected:
          ly["correction"] = vector(p + "mlp.correction")
        if spec.mlp.shared_ff and not parts:
          ly["shared_up"], ly["shared_down"] = linear([p + "mlp.shared.up"]), linear([p + "mlp.shared.down"])
      elif isinstance(spec.mlp, PolyNormMlp):
        ly["gu"], ly["down"], ly["act"] = linear([p + "mlp.up"]), linear([p + "mlp.down"]), vector(p + "mlp.act")
      elif spec.mlp is not None:
        ly["gu"] = linear([p + "mlp.gate", p + "mlp.up"], paired=True)
        ly["down"] = linear([p + "mlp.down"])
      self.layers.append(ly)
    # the head (the embedding table, or a weight of its own) runs through the statistics head when its shape is
    # one that kernel takes, else as a plain linear into fp32 logits
    self.head = self.head_expanded = self.head_linear = None
    self.head_w = self.embed if cfg.tied_head else torch.zeros_like(self.embed)
    self.block_head = dtype == torch.bfloat16 and D % 128 == 0 and V % 16 == 0
    self._load_tables(weights)
    torch.cuda.synchronize(dev)

  def _load_tables(self, weights: dict):
    """The embedding table and the head, as far as `weights` has them."""
    head = "embed" if self.cfg.tied_head else "head"
    for name, table in (("embed", self.embed), ("pos", self.pos), (head, self.head_w)):
      if table is not None and name in weights:
        table.copy_(weights[name].to(self.device, self.dtype))
    if head not in weights:
      return
    if self.block_head:
      if self.head_expanded is None:
        self.head_expanded = ops.dense_expand(self.head_w)
      else:
        self.head_expanded.copy_(ops.dense_expand(self.head_w))
    elif self.head_linear is None:
      self.head_linear = DenseLinear([head], {head: self.head_w}, self.dtype, self.device)
    else:
      self.head_linear.load({head: self.head_w})

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
      if isinstance(m, AttentionMixer) and m.kv_from is not None:
        spec = BorrowedSpec(m.kv_from)   # (layers with borrowed keys run once: a layer is its run)
      elif isinstance(m, AttentionMixer):
        spec = KVSpec(m.kv_heads, ops.sink_attn_pad(m.dim, False, self.dtype),
                      ops.sink_attn_pad(m.vdim, True, self.dtype), self.dtype)
      elif isinstance(m, SsdMixer):
        spec = PartsSpec((("state", StateSpec(m.heads, m.state, m.vdim)), ("conv", RingSpec(m.conv, m.channels, self.dtype))))
      elif isinstance(m, LatentMixer):
        spec = LatentSpec(ops.latent_row(m.kv_rank, m.rot_dim, self.dtype), self.dtype)
      elif isinstance(m, ParallelMixer):
        a, b = m.left, m.right
        ring = self.layers[i]["left"]["conv"]
        left = PartsSpec((("kv", KVSpec(a.kv_heads, ops.sink_attn_pad(a.dim, True, self.dtype), ops.sink_attn_pad(a.vdim, True, self.dtype), self.dtype)),
                          ("conv", RingSpec(a.conv, ring.shape[1], self.dtype))))
        right = PartsSpec((("state", StateSpec(b.heads, b.dim, b.vdim)), ("sum", StateSpec(b.heads, b.dim, 1)), ("top", StateSpec(b.heads, 1, 1))))
        spec = PartsSpec((("left", left), ("right", right), ("input", RingSpec(max(self.cfg.input_conv - 1, 1), self.cfg.embed_dim, torch.float32))))
      else:
        spec = StateSpec(m.heads, m.dim, m.vdim)
      if self.cfg.token_shift:
        spec = PartsSpec((("mixer", spec), ("shift", RingSpec(1, self.cfg.embed_dim, torch.float32))))
      specs.append(spec)
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
    owners = {id(f): f for n, fs in self.linears.items() if n in new_state for f in fs}
    for f in owners.values():
      f.check(new_state)
    for f in owners.values():
      f.load(new_state)
    for n, t in new_state.items():
      if n in self.vectors:
        t = t.to(self.device, torch.float32)
        self.vectors[n].copy_(t.T if n in self.transposed else t)
    self._load_tables(new_state)
    torch.cuda.synchronize(self.device)

  def weight_bytes(self) -> dict:
    """Bytes one decode step reads: the linears (a looped layer's once per pass) and the head."""
    n = 0
    for i, begins in self.cfg.layer_runs:
      ly = self.layers[i]
      n += sum(part[k].nbytes() for part in (ly, ly.get("left", {}), ly.get("right", {}))
               for k in ("in", "uq", "absorb_k", "absorb_v", "out", "router", "gates", "gu", "down", "shared_up", "shared_down") if hasattr(part.get(k), "nbytes"))
      n += self.loop_in.nbytes() if begins and self.loop_in is not None else 0
    return {"dense": n, "head": self.head_w.numel() * self.head_w.element_size()}


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
    # the embedding output and every layer's result but the last one's, where they are averaged over depth
    self.hist = torch.empty(cfg.num_layers, M, D, dtype=torch.float32, device=dev) if cfg.depth_average else None
    self.first = None           # the embedding output, until a sublayer has been added
    # a token shift or an input convolution reads the rows in front of a row: over several tokens the new rows go to a
    # second buffer
    self.x_next = torch.empty_like(self.x) if (cfg.token_shift or cfg.input_conv > 1) and T > 1 else None
    self.tail = torch.empty(B * min(T, max(cfg.input_conv - 1, 1)), D, dtype=torch.float32, device=dev) if cfg.input_conv > 1 and T > 1 else None
    # the final-normed rows (row-major, zero columns behind the model width)
    width = D if model.block_head else model.Dp
    self.xn = torch.zeros(M, width, dtype=self.dtype, device=dev)
    self.split_k_override = dict(split_k_override or {})
    n_light = n_attn = n_routes = n_experts = 1
    n_y, n_ws = [1, 1, 1], [1, 1, 1]     # a projection's output, and those of some which run while the first is still read
    for i, begins in cfg.layer_runs:
      ly = model.layers[i]
      m = ly["spec"].mixer
      mlp_slot = 2 if cfg.parallel else 0
      uses = [(ly, k, s) for k, s in (("in", 0), ("out", 0), ("router", 0), ("gu", mlp_slot), ("down", mlp_slot), ("uq", 1), ("ukv", 1), ("shared_down", 0))]
      if cfg.parallel:
        uses += [(ly["right"], "gates", 1), (ly["left"], "out", 0), (ly["right"], "out", 1)]
      for part, key, slot in uses:
        f = part.get(key)
        if isinstance(f, DenseLinear):
          n_y[slot] = max(n_y[slot], M * f.N)
          n_ws[slot] = max(n_ws[slot], self._split(f) * M * f.N if self._split(f) > 1 or key in ("router", "gates") or
                         key == "in" and isinstance(m, GatedStateMixer) else 1)
      if begins and model.loop_in is not None:
        n_ws[0] = max(n_ws[0], self._split(model.loop_in) * M * model.loop_in.N)
      if isinstance(ly["spec"].mlp, ExpertsMlp):
        e = ly["spec"].mlp
        n_routes, n_experts = max(n_routes, M * e.routes), max(n_experts, len(ly["gu"]))
        if self.dtype == torch.float32:
          n_y[0] = max(n_y[0], M * e.routes * ly["gu"].N)
      if isinstance(m, LightningMixer):   # (a call may bring fewer rows, and cut them into more spans)
        n_light = max([n_light] + [ops.lightning_ws_bytes(b, T, m.heads, m.dim, m.vdim) // 4 for b in range(1, B + 1)])
      elif isinstance(m, GatedStateMixer):
        n_light = max([n_light] + [ops.gated_state_ws_bytes(b, T, m.heads, m.dim, m.vdim) // 4 for b in range(1, B + 1)])
      elif isinstance(m, SsdMixer):
        n_light = max([n_light] + [ops.ssd_ws_bytes(b, T, m.heads, m.groups, m.state, m.vdim) // 4 for b in range(1, B + 1)])
      elif isinstance(m, LatentMixer):
        if self.dtype == torch.bfloat16:
          n_attn = max(n_attn, ops.latent_attn_ws_bytes(B, T, S, m.heads, m.kv_rank, self._latent_chunk(m)) // 4)
      elif isinstance(m, ParallelMixer):
        a, r = m.left, m.right
        n_light = max([n_light] + [ops.memory_ws_bytes(b, T, r.heads, r.dim, r.vdim) // 4 for b in range(1, B + 1)])
        n_attn = max(n_attn, ops.mixed_attn_ws_bytes(B, T, S, a.heads, ops.sink_attn_pad(a.vdim, True, self.dtype), self._mixed_chunk(kv_chunk)) // 4)
      else:
        n_attn = max(n_attn, ops.sink_attn_ws_bytes(B, T, S, m.heads, ops.sink_attn_pad(m.vdim, True, self.dtype),
                                                    self._kv_chunk(m, kv_chunk)) // 4)
    self.kv_chunk_arg = kv_chunk
    self.y = [torch.empty(n, dtype=self.dtype, device=dev) for n in n_y]
    self.ws = [torch.empty(n, dtype=torch.float32, device=dev) for n in n_ws]
    if any(isinstance(ly.mlp, ExpertsMlp) for ly in cfg.layers):
      i32 = lambda n: torch.empty(n, dtype=torch.int32, device=dev)
      self.topk_id, self.counts, self.offsets, self.sorted_route = i32(n_routes), i32(n_experts), i32(n_experts + 1), i32(n_routes)
      self.topk_w = torch.empty(n_routes, dtype=torch.float32, device=dev)
      self.gate_w = torch.empty(M, dtype=torch.float32, device=dev)
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
  def _buf(self, name: str, cols: int, dtype=None, rows: int | None = None) -> torch.Tensor:
    """Activation buffer [rows, cols], zero where nothing is ever written (the padding columns of a
    linear's input must be zero); whole blocks of 128 rows for the fragment order."""
    key = (name, cols, rows)
    if key not in self._bufs:
      if rows is None:
        rows = _up(self.M, 128) if self.frag else self.M
      self._bufs[key] = torch.zeros(rows, cols, dtype=self.dtype if dtype is None else dtype, device=self.model.device)
    return self._bufs[key]

  def _kv_chunk(self, m: AttentionMixer, given) -> int:
    """Decode: split the key range only as far as needed to put about a thousand waves on the device."""
    if given is not None:
      return given
    waves = self.B * m.kv_heads * math.ceil(self.T * (m.heads // m.kv_heads) / 16)
    S = min(self.S, m.chunk + 31) if m.chunk else self.S      # (columns that one position may see, from a block's edge on)
    if self.dtype != torch.bfloat16 or self.T != 1 or waves >= 1024 or S <= 64:
      return 0
    n = min(math.ceil(1024 / waves), S // 32)
    chunk = max(32, _up(math.ceil(S / n), 32))
    return 0 if chunk >= S else chunk

  def _latent_chunk(self, m: LatentMixer) -> int:
    """The same for latent attention, whose work-groups have a compute unit to themselves."""
    groups = self.B * math.ceil(self.T * m.heads / 32)
    if self.T != 1 or groups >= 256 or self.S <= 256:
      return 0
    chunk = max(256, _up(math.ceil(self.S / math.ceil(256 / groups)), 64))
    return 0 if chunk >= self.S else chunk

  def _mixed_chunk(self, given) -> int:
    """Keys of a work-group in a decode step of mixed attention: as many as leave about two work-groups per compute unit."""
    if given:
      return given
    for chunk in (320, 256, 192, 128):
      if self.B * math.ceil(self.S / chunk) >= 512:
        return chunk
    return 64

  def _split(self, f: DenseLinear) -> int:
    """k split of a few-row linear whose reader sums fp32 planes."""
    key = f.names[0].split(".")[-1]
    if key in self.split_k_override:
      return self.split_k_override[key]
    if not self.frag or f.paired:
      return 1
    groups = math.ceil(f.N / 64) * math.ceil(self.M / 128)
    return int(max(1, min(8, (256 if self.M > 32 else 512) // groups, f.Kp // 512)))

  def linear(self, f: DenseLinear, x, M: int, fp32_out: bool = False, slot: int = 0, cols: tuple | None = None) -> L.RowsSrc:
    """Runs one projection of x [M, f.Kp], or its columns cols[0] .. cols[1] (runs of 256); returns its output as the reading
    kernel wants it.  It holds until the next projection of the same slot."""
    c0, c1 = cols or (0, f.N)
    N = c1 - c0
    d = L.DenseDesc()
    d.M, d.K, d.N, d.dtype = M, f.Kp, N, self.code
    d.x, d.ldx, d.x_frag, d.w = x.data_ptr(), x.shape[1], 1 if self.frag else 0, f.w.data_ptr() + c0 * f.Kp * f.w.element_size()
    d.ldy, d.split_k = N, self._split(f)
    src = L.RowsSrc()
    src.ld, src.plane, src.split_k = N, M * N, d.split_k
    if d.split_k > 1:
      d.epilogue, d.ws = L.TNX_EPI_F32, self.ws[slot].data_ptr()
      src.ws = d.ws
    elif fp32_out and self.dtype != torch.float32:
      d.epilogue, d.y = L.TNX_EPI_F32, self.ws[slot].data_ptr()
      src.ws = d.y
    else:
      d.epilogue, d.y = L.TNX_EPI_STORE, self.y[slot].data_ptr()
      src.y = d.y
    ops.dense_linear(d)
    return src

  def bank(self, f: LinearBank, x, ldx: int, x_stride: int, y, ldy: int, y_stride: int, M: int):
    """Every row of x through every projection of a bank: x + z x_stride -> y + z y_stride."""
    d = L.DenseDesc()
    d.M, d.K, d.N, d.dtype = M, f.Kp, f.N, self.code
    d.x, d.ldx, d.x_stride, d.w, d.w_stride = x.data_ptr(), ldx, x_stride, f.w.data_ptr(), f.stride
    d.epilogue, d.y, d.ldy, d.y_stride, d.split_k, d.batch = L.TNX_EPI_STORE, y.data_ptr(), ldy, y_stride, 1, len(f)
    ops.dense_linear(d)

  def residual_norm(self, pending, w_next, out, M: int, frag: bool, shift=None, behind=None):
    """x takes what is pending: None, ("add", rows, post-norm weight), ("set", rows, None), ("norm", None, weight) --
    x itself normed -- or ("routes", rows, post-norm weight, route weights, routes per row[, extra rows, their weights]);
    out = norm(x) . w_next, or x itself when w_next is None, or x moved towards the token before:
    shift = (weight, ring of the rows before, col_ptr, starts, B, T).
    behind: the layer that ends with what is pending, when results are averaged over depth."""
    cfg = self.cfg
    d = L.ResidualNormDesc()
    d.M, d.D, d.dtype, d.eps, d.w_offset, d.groups = M, cfg.embed_dim, self.code, cfg.norm_eps, cfg.norm_offset, cfg.norm_groups
    d.center, d.mult = 1 if cfg.center_norm else 0, cfg.residual_mult
    if pending is not None:
      kind, rows, w_post = pending[:3]
      d.mode = {"add": 1, "routes": 1, "set": 2, "norm": 3}[kind]
      if rows is not None:
        d.y = rows
      d.w_post = None if w_post is None else w_post.data_ptr()
      if kind == "routes":
        d.route_w, d.route_k = pending[3].data_ptr(), pending[4]
        if len(pending) > 5:
          d.extra, d.extra_w = pending[5], pending[6].data_ptr()
    d.x, d.w_next = self.x.data_ptr(), None if w_next is None else w_next.data_ptr()
    if self.first is not None:
      d.x = self.first.data_ptr()
      if pending is not None:
        d.x_out, self.first = self.x.data_ptr(), None
    if behind is not None:
      d.hist, d.hist_plane, d.hist_n, d.hist_w = self.hist.data_ptr(), self.M * cfg.embed_dim, behind + 1, self.model.layers[behind]["dwa"].data_ptr()
      d.hist_store = 1 if behind + 1 < cfg.num_layers else 0
    d.out, d.out_ld, d.out_frag = out.data_ptr(), out.shape[1], 1 if frag else 0
    if shift is not None:
      w, ring, col_ptr, starts, B, T = shift
      d.shift, d.before, d.starts, d.col_ptr, d.B, d.T = w.data_ptr(), ring.data_ptr(), starts.data_ptr(), col_ptr.data_ptr(), B, T
      if T > 1:
        d.x_out = self.x_next.data_ptr()
    ops.residual_norm(d)
    if shift is not None and T > 1:
      self.x, self.x_next = self.x_next, self.x
      ops.ring_write(ops.rows_src(y=self.x, ld=cfg.embed_dim), 0, B, T, col_ptr, ring)

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

  def norm_kv(self, ly, src, entry, col_ptr, starts, B, T):
    """Norms q and k over their projections and writes the cache (with borrowed keys: q alone); returns q."""
    m, f = ly["spec"].mixer, ly["in"]
    dkp, dvp = entry.k.shape[3], entry.v.shape[3]
    q = self._buf("q", m.heads * dkp)
    d = L.RowNormKvDesc()
    d.B, d.T, d.S, d.H, d.G = B, T, entry.k.shape[2], m.heads, m.kv_heads
    d.dk, d.dv, d.dkp, d.dvp, d.dtype, d.eps = m.dim, m.vdim, dkp, dvp, self.code, self.cfg.norm_eps
    d.w_q, d.y, d.col_ptr, d.q_out = ly["q_norm"].data_ptr(), src, col_ptr.data_ptr(), q.data_ptr()
    if m.kv_from is None:
      d.w_k, d.k_off, d.v_off = ly["k_norm"].data_ptr(), f.offsets[1], f.offsets[2]
      d.kcache, d.vcache = entry.k.data_ptr(), entry.v.data_ptr()
    ops.rownorm_kvwrite(d)
    return q

  def attend(self, ly, q, entry, col_ptr, starts, B, T) -> torch.Tensor:
    m = ly["spec"].mixer
    out = self._buf("attn", ly["out"].Kp)
    d = L.SinkAttnDesc()
    d.B, d.T, d.S, d.H, d.G = B, T, entry.k.shape[2], m.heads, m.kv_heads
    d.dk, d.dv, d.dkp, d.dvp, d.scale, d.dtype = m.dim, m.vdim, entry.k.shape[3], entry.v.shape[3], m.scale, self.code
    d.q, d.kcache, d.vcache = q.data_ptr(), entry.k.data_ptr(), entry.v.data_ptr()
    d.sinks = None if ly["sink"] is None else ly["sink"].data_ptr()
    d.slopes, d.chunk = None if ly["slopes"] is None else ly["slopes"].data_ptr(), m.chunk
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
    """norm(o) . weight * sigmoid(gate columns of the projection); a memory's heads are normed on their own."""
    m, out = ly["spec"].mixer, self._buf("gated", ly["out"].Kp)
    d = L.GatedNormDesc()
    d.M, d.W, d.dtype, d.eps, d.w_offset, d.groups = M, o.shape[1], self.code, self.cfg.norm_eps, 0.0, m.heads if isinstance(m, MemoryMixer) else 1
    d.o, d.o_ld, d.g, d.g_off, d.w = o.data_ptr(), o.shape[1], src, ly["in"].offsets[3], ly["norm"].data_ptr()
    d.out, d.out_ld, d.out_frag = out.data_ptr(), out.shape[1], 1 if self.frag else 0
    ops.gated_norm(d)
    return out

  # forget gates whose complement writes
  def gated_in(self, f: DenseLinear, h, M: int):
    """The projection of h as the recurrence reads it: (rows of q and v, whether they are fp32, rows of the gates -- fp32
    always --, the gates' first column)."""
    if self.dtype == torch.float32 or self.frag:
      src = self.fp32_rows(f, h, M, slot=0)
      return src, 1, src, f.offsets[2]
    return self.linear(f, h, M, cols=(0, f.offsets[2])), 0, self.fp32_rows(f, h, M, slot=0, cols=(f.offsets[2], f.N)), 0

  def gated_state(self, ly, rows, entry, col_ptr, starts, B, T) -> tuple:
    """The recurrence: (what the output projection reads, True), heads normed, or (fp32 [rows, heads * vdim], False)."""
    m, f = ly["spec"].mixer, ly["in"]
    d = L.GatedStateDesc()
    d.B, d.T, d.H, d.dk, d.dv, d.dtype = B, T, m.heads, m.dim, m.vdim, self.code
    d.y, d.y_f32, d.f, d.f_off = rows
    d.q_off, d.v_off, d.bias, d.lower = f.offsets[0], f.offsets[1], ly["bias"].data_ptr(), ly["lower"].data_ptr()
    d.starts, d.col_ptr, d.state, d.ws = starts.data_ptr(), col_ptr.data_ptr(), entry.s.data_ptr(), self.light_ws.data_ptr()
    if T == 1 and ops.gated_state_step_ok(m.dim, m.vdim):
      out = self._buf("gated", ly["out"].Kp)
      d.norm_w, d.eps, d.out, d.out_ld, d.out_frag = ly["norm"].data_ptr(), self.cfg.norm_eps, out.data_ptr(), out.shape[1], 1 if self.frag else 0
      ops.gated_state(d)
      return out, True
    o = self._buf("state_out", m.heads * m.vdim, torch.float32)
    d.o, d.o_ld = o.data_ptr(), o.shape[1]
    ops.gated_state(d)
    return o, False

  def head_norm(self, ly, o, M: int) -> torch.Tensor:
    """Heads of o normed on their own, with shared weights."""
    m, out = ly["spec"].mixer, self._buf("gated", ly["out"].Kp)
    d = L.GatedNormDesc()
    d.M, d.W, d.dtype, d.eps, d.groups, d.shared_w = M, o.shape[1], self.code, self.cfg.norm_eps, m.heads, 1
    d.o, d.o_ld, d.w = o.data_ptr(), o.shape[1], ly["norm"].data_ptr()
    d.out, d.out_ld, d.out_frag = out.data_ptr(), out.shape[1], 1 if self.frag else 0
    ops.gated_norm(d)
    return out

  # parallel layers
  def parallel_step(self, pending, ly, out, out2, at, entry, add=None):
    """x takes the pending sublayers (rows of the left and right mixer and of the feed-forward with their layer, or None)
    and the vector `add`; out, out2 = norm(x) behind the layer's input convolutions.  ly None: out = the final norm of x."""
    cfg, (col_ptr, starts, B, T) = self.cfg, at
    d = L.ParallelStepDesc()
    d.M, d.D, d.dtype, d.eps, d.mult, d.B, d.T = B * T, cfg.embed_dim, self.code, cfg.norm_eps, cfg.residual_mult, B, T
    if pending is not None:
      sides, mlp, before = pending
      for i, (side, rows) in enumerate(zip(("left", "right"), sides)):
        d.y[i], d.w_post[i], d.y_scale[i] = rows, before[side]["post"].data_ptr(), 0.5
      d.n_in = 2
      if mlp is not None:
        d.y[2], d.y_scale[2], d.n_in = mlp, 1.0, 3
    moved = ly is not None and cfg.input_conv > 1 and T > 1
    d.x, d.add = self.x.data_ptr(), None if add is None else add.data_ptr()
    if d.n_in or add is not None:
      d.x_out = (self.x_next if moved else self.x).data_ptr()
    d.out1, d.out_ld, d.out_frag = out.data_ptr(), out.shape[1], 1 if self.frag and ly is not None else 0
    if ly is None:
      d.w_next = self.model.final_norm.data_ptr()
    else:
      ring = entry["input"].r
      d.w_next, d.conv1, d.taps, d.slots, d.ring = ly["norm1"].data_ptr(), ly["canon1"].data_ptr(), cfg.input_conv, ring.shape[1], ring.data_ptr()
      if "canon2" in ly:
        d.conv2, d.out2 = ly["canon2"].data_ptr(), out2.data_ptr()
      d.starts, d.col_ptr = starts.data_ptr(), col_ptr.data_ptr()
      if moved:
        d.tail = self.tail.data_ptr()
    ops.parallel_step(d)
    if moved:
      if d.x_out:
        self.x, self.x_next = self.x_next, self.x
      keep = min(T, cfg.input_conv - 1)
      ops.ring_write(ops.rows_src(y=self.tail, ld=cfg.embed_dim), 0, B, keep, col_ptr, ring, t0=T - keep)

  def conv_kv(self, ly, src, entry, col_ptr, starts, B, T) -> torch.Tensor:
    """Convolution of q, k and v, query temperature, value norm, cache write; returns q."""
    m, f, kv, ring = ly["spec"].mixer, ly["in"], entry["kv"], entry["conv"].r
    dkp, dvp = kv.k.shape[3], kv.v.shape[3]
    q = self._buf("q", m.heads * dkp)
    d = L.ConvKvDesc()
    d.B, d.T, d.S, d.H, d.G = B, T, kv.k.shape[2], m.heads, m.kv_heads
    d.dk, d.dv, d.dkp, d.dvp, d.taps, d.slots, d.dtype = m.dim, m.vdim, dkp, dvp, m.conv, ring.shape[1], self.code
    d.temp_coef, d.temp_every, d.eps, d.value_norm = m.temp_coef, m.temp_every, self.cfg.norm_eps, 1 if m.value_norm else 0
    d.y, d.off, d.C = src, f.offsets[0], ring.shape[2]
    d.q_off, d.k_off, d.v_off = (o - f.offsets[0] for o in f.offsets[:3])
    d.w, d.ring, d.starts, d.col_ptr = ly["conv"].data_ptr(), ring.data_ptr(), starts.data_ptr(), col_ptr.data_ptr()
    d.q_out, d.kcache, d.vcache = q.data_ptr(), kv.k.data_ptr(), kv.v.data_ptr()
    ops.conv_kvwrite(d)
    if T > 1:
      ops.ring_write(src, f.offsets[0], B, T, col_ptr, ring)
    return q

  def mixed_attend(self, ly, q, src, entry, col_ptr, starts, B, T) -> torch.Tensor:
    """Attention with mixed heads and the output gate (the projection's fourth part)."""
    m, kv = ly["spec"].mixer, entry["kv"]
    out = self._buf("mixed", ly["out"].Kp)
    d = L.MixedAttnDesc()
    d.B, d.T, d.S, d.H, d.G = B, T, kv.k.shape[2], m.heads, m.kv_heads
    d.dk, d.dv, d.dkp, d.dvp, d.scale, d.dtype = m.dim, m.vdim, kv.k.shape[3], kv.v.shape[3], m.scale, self.code
    d.q, d.kcache, d.vcache, d.talk = q.data_ptr(), kv.k.data_ptr(), kv.v.data_ptr(), ly["talk"].data_ptr()
    d.starts, d.col_ptr, d.kv_chunk, d.ws = starts.data_ptr(), col_ptr.data_ptr(), self._mixed_chunk(self.kv_chunk_arg), self.attn_ws.data_ptr()
    d.gate, d.g_off = src, ly["in"].offsets[3]
    d.out, d.out_ld, d.out_frag = out.data_ptr(), out.shape[1], 1 if self.frag else 0
    ops.mixed_attn(d)
    return out

  def remember(self, ly, src, gates, entry, col_ptr, starts, B, T) -> torch.Tensor:
    """The matrix memory of a projection's rows: fp32 [rows, heads * vdim]."""
    m, f = ly["spec"].mixer, ly["in"]
    o = self._buf("state_out", m.heads * m.vdim, torch.float32)
    d = L.MemoryDesc()
    d.B, d.T, d.H, d.dk, d.dv, d.dtype, d.q_scale, d.cap = B, T, m.heads, m.dim, m.vdim, self.code, m.dim ** -0.5, m.gate_cap
    d.y, d.q_off, d.k_off, d.v_off = src, *f.offsets[:3]
    d.gates, d.i_off, d.f_off = gates, *ly["gates"].offsets
    d.bias_i, d.bias_f, d.starts, d.col_ptr = ly["bias_i"].data_ptr(), ly["bias_f"].data_ptr(), starts.data_ptr(), col_ptr.data_ptr()
    d.state, d.sum, d.top = (entry[n].s.data_ptr() for n in ("state", "sum", "top"))
    d.o, d.o_ld, d.ws = o.data_ptr(), o.shape[1], self.light_ws.data_ptr()
    ops.memory(d)
    return o

  def fp32_rows(self, f: DenseLinear, x, M: int, slot: int, cols: tuple | None = None) -> L.RowsSrc:
    """A projection whose rows stay fp32 (finished, or planes)."""
    src = self.linear(f, x, M, fp32_out=True, slot=slot, cols=cols)
    if src.split_k <= 1 and src.ws:
      src.y = src.ws
    return src

  def parallel_sublayers(self, ly, h, h2, entry, col_ptr, starts, B, T):
    """Both mixers of h and the feed-forward of h2, as `parallel_step` takes them."""
    M, at, left, right = B * T, (col_ptr, starts, B, T), ly["left"], ly["right"]
    src = self.linear(ly["in"], h, M)
    gates = self.fp32_rows(right["gates"], h, M, slot=1)
    a = self.mixed_attend(left, self.conv_kv(left, src, entry["left"], *at), src, entry["left"], *at)
    b = self.gate(right, self.remember(right, src, gates, entry["right"], *at), src, M)
    sides = self.linear(left["out"], a, M), self.linear(right["out"], b, M, slot=1)
    mlp = self.linear(ly["down"], self.gate_up(ly, h2, M, slot=2), M, slot=2) if "gu" in ly else None
    return sides, mlp, ly

  # state-space duality
  def convolve(self, ly, src, entry, col_ptr, starts, B, T) -> torch.Tensor:
    """silu(convolution) of x, B and C: [rows, channels]; the ring takes the last inputs."""
    m, ring = ly["spec"].mixer, entry["conv"].r
    u = self._buf("conv", _up(m.channels, 8), rows=self.M)
    d = L.ShortConvDesc()
    d.B, d.T, d.C, d.taps, d.slots, d.dtype = B, T, m.channels, m.conv, ring.shape[1], self.code
    d.y, d.off, d.w, d.bias, d.ring = src, ly["in"].offsets[1], ly["conv"].data_ptr(), ly["conv_b"].data_ptr(), ring.data_ptr()
    d.starts, d.col_ptr, d.out, d.out_ld = starts.data_ptr(), col_ptr.data_ptr(), u.data_ptr(), u.shape[1]
    ops.short_conv(d)
    ops.ring_write(src, ly["in"].offsets[1], B, T, col_ptr, ring)
    return u

  def ssd(self, ly, src, u, entry, col_ptr, starts, B, T) -> torch.Tensor:
    """The recurrence: fp32 [rows, heads * vdim].  u None: one token, the convolution inside."""
    m, f, ring = ly["spec"].mixer, ly["in"], entry["conv"].r
    o = self._buf("state_out", m.inner, torch.float32)
    d = L.SsdDesc()
    d.B, d.T, d.H, d.G, d.N, d.P, d.dtype = B, T, m.heads, m.groups, m.state, m.vdim, self.code
    d.A_log, d.dt_bias, d.D = ly["A_log"].data_ptr(), ly["dt_bias"].data_ptr(), ly["D"].data_ptr()
    d.y, d.c_off, d.dt_off = src, f.offsets[1], f.offsets[2]
    if u is not None:
      d.u, d.u_ld = u.data_ptr(), u.shape[1]
    d.taps, d.slots, d.conv_w, d.conv_b, d.ring = m.conv, ring.shape[1], ly["conv"].data_ptr(), ly["conv_b"].data_ptr(), ring.data_ptr()
    d.starts, d.col_ptr, d.state = starts.data_ptr(), col_ptr.data_ptr(), entry["state"].s.data_ptr()
    d.o, d.o_ld, d.ws = o.data_ptr(), o.shape[1], self.light_ws.data_ptr()
    ops.ssd(d)
    return o

  def ssd_gate(self, ly, o, src, M: int) -> torch.Tensor:
    """norm(o * silu(gate columns of the projection)) . weight, in the mixer's norm groups."""
    m, out = ly["spec"].mixer, self._buf("gated", ly["out"].Kp)
    d = L.GatedNormDesc()
    d.M, d.W, d.dtype, d.eps, d.gate_first, d.groups = M, m.inner, self.code, self.cfg.norm_eps, 1, m.norm_groups
    d.o, d.o_ld, d.g, d.g_off, d.w = o.data_ptr(), o.shape[1], src, ly["in"].offsets[0], ly["norm"].data_ptr()
    d.out, d.out_ld, d.out_frag = out.data_ptr(), out.shape[1], 1 if self.frag else 0
    ops.gated_norm(d)
    return out

  # latent attention
  def latent_prep(self, ly, src, entry, col_ptr, starts, B, T, expand: bool):
    """Norms the query latent (returned) and the key / value latent (returned with `expand`), fills the cache."""
    m, f, c = ly["spec"].mixer, ly["in"], entry.c
    cq = self._buf("cq", ly["uq"].Kp)
    ckv = self._buf("ckv", ly["ukv"].Kp) if expand else None
    d = L.LatentPrepDesc()
    d.B, d.T, d.S = B, T, c.shape[1]
    d.q_rank, d.rank, d.rot, d.rank_pad, d.row = m.q_rank, m.kv_rank, m.rot_dim, _up(m.kv_rank, 16), c.shape[2]
    d.dtype, d.eps, d.y, d.q_off, d.kv_off = self.code, self.cfg.norm_eps, src, f.offsets[0], f.offsets[1]
    d.w_q, d.w_kv, d.inv_freq = ly["q_norm"].data_ptr(), ly["kv_norm"].data_ptr(), ly["inv_freq"].data_ptr()
    d.starts, d.col_ptr, d.cache = starts.data_ptr(), col_ptr.data_ptr(), c.data_ptr()
    d.q_out, d.q_ld, d.q_frag = cq.data_ptr(), cq.shape[1], 1 if self.frag else 0
    if expand:
      d.c_out, d.c_ld, d.c_frag = ckv.data_ptr(), ckv.shape[1], 1 if self.frag else 0
    ops.latent_prep(d)
    return cq, ckv

  def latent_q(self, ly, src, col_ptr, starts, B, T, un, un_ld, un_pad, rot, rot_at, rot_ld, rot_pad):
    """Splits the heads of a query projection: the unrotated parts to `un`, the rotated ones to rot[rot_at ..]."""
    m = ly["spec"].mixer
    d = L.LatentQDesc()
    d.B, d.T, d.H, d.n, d.r, d.dtype, d.y = B, T, m.heads, m.dim, m.rot_dim, self.code, src
    d.inv_freq, d.starts, d.col_ptr = ly["inv_freq"].data_ptr(), starts.data_ptr(), col_ptr.data_ptr()
    d.un, d.un_ld, d.un_pad = un.data_ptr(), un_ld, un_pad
    d.rot, d.rot_ld, d.rot_pad = rot.data_ptr() + rot_at * rot.element_size(), rot_ld, rot_pad
    ops.latent_q(d)

  def gate_mul(self, ly, y, head: int, y_head: int, src, M: int) -> torch.Tensor:
    m, out = ly["spec"].mixer, self._buf("gated", ly["out"].Kp)
    d = L.GateMulDesc()
    d.M, d.W, d.head, d.dtype, d.y, d.y_ld, d.y_head = M, m.heads * head, head, self.code, y.data_ptr(), m.heads * y_head, y_head
    d.g, d.g_off, d.out, d.out_ld, d.out_frag = src, ly["in"].offsets[2], out.data_ptr(), out.shape[1], 1 if self.frag else 0
    ops.gate_mul(d)
    return out

  def plain_attention(self, m, q, k, v, dk, dv, starts, col_ptr, B, T, S, G, out, out_head):
    """softmax(scale q k) v over plain keys and values (one kv head per query head, or one for all)."""
    d = L.SinkAttnDesc()
    d.B, d.T, d.S, d.H, d.G = B, T, S, m.heads, G
    d.dk, d.dv, d.dkp, d.dvp, d.scale, d.dtype = dk, dv, k.shape[-1], v.shape[-1], m.scale, self.code
    d.q, d.kcache, d.vcache, d.starts, d.col_ptr = q.data_ptr(), k.data_ptr(), v.data_ptr(), starts.data_ptr(), col_ptr.data_ptr()
    d.ws, d.out, d.out_ld, d.out_head = self.attn_ws.data_ptr(), out.data_ptr(), m.heads * out_head, out_head
    ops.sink_attn(d)

  def latent_kv(self, ly, src, k, v, entry, B, T):
    """Lays the projected keys and values of a prompt out as plain attention reads them."""
    m, c = ly["spec"].mixer, entry.c
    d = L.LatentKvDesc()
    d.B, d.T, d.S, d.H, d.n, d.r, d.vd = B, T, c.shape[1], m.heads, m.dim, m.rot_dim, m.vdim
    d.dkp, d.dvp, d.rank_pad, d.row, d.dtype = k.shape[1], v.shape[1], _up(m.kv_rank, 16), c.shape[2], self.code
    d.y, d.v_off, d.cache, d.k, d.v = src, ly["ukv"].offsets[1], c.data_ptr(), k.data_ptr(), v.data_ptr()
    ops.latent_kv(d)

  def latent_prompt(self, ly, cq, ckv, entry, col_ptr, starts, B, T):
    """A prompt from its first column on: keys and values of all heads are formed for its tokens."""
    m, M = ly["spec"].mixer, B * T
    dkp, dvp = ops.sink_attn_pad(m.dim + m.rot_dim, False, self.dtype), ops.sink_attn_pad(m.vdim, True, self.dtype)
    q = self._buf("q", m.heads * dkp, rows=self.M)
    self.latent_q(ly, self.linear(ly["uq"], cq, M, slot=1), col_ptr, starts, B, T, q, dkp, m.dim, q, m.dim, dkp, dkp - m.dim)
    k, v = self._buf("k_full", dkp, rows=self.M * m.heads), self._buf("v_full", dvp, rows=self.M * m.heads)
    self.latent_kv(ly, self.linear(ly["ukv"], ckv, M, slot=1), k, v, entry, B, T)
    out = self._buf("heads", m.heads * m.vdim, rows=self.M)
    self.plain_attention(m, q, k, v, m.dim + m.rot_dim, m.vdim, starts, col_ptr, B, T, T, m.heads, out, m.vdim)
    return out, m.vdim

  def latent_rows(self, ly, cq, entry, col_ptr, starts, B, T):
    """Decoding and portions: the heads attend to the cache rows themselves."""
    m, M, c = ly["spec"].mixer, B * T, entry.c
    H, row, fk, fv = m.heads, c.shape[2], ly["absorb_k"], ly["absorb_v"]
    un, q = self._buf("q_un", H * fk.Kp, rows=self.M), self._buf("q", H * row, rows=self.M)
    self.latent_q(ly, self.linear(ly["uq"], cq, M, slot=1), col_ptr, starts, B, T, un, fk.Kp, fk.Kp, q, fk.N, row, row - fk.N)
    self.bank(fk, un, H * fk.Kp, fk.Kp, q, H * row, row, M)
    lat = self._buf("latent_out", H * fv.Kp, rows=self.M)
    self.latent_attend(ly, q, lat, fv.Kp, entry, col_ptr, starts, B, T)
    out = self._buf("heads", H * fv.N, rows=self.M)
    self.bank(fv, lat, H * fv.Kp, fv.Kp, out, H * fv.N, fv.N, M)
    return out, fv.N

  def latent_attend(self, ly, q, out, out_head, entry, col_ptr, starts, B, T):
    m, c = ly["spec"].mixer, entry.c
    S, row = c.shape[1], c.shape[2]
    if self.dtype != torch.bfloat16 or not ops.latent_attn_ok(m.kv_rank, row, S):
      self.plain_attention(m, q, c, c, _up(m.kv_rank, 16) + m.rot_dim, m.kv_rank, starts, col_ptr, B, T, S, 1, out, out_head)
      return
    d = L.LatentAttnDesc()
    d.B, d.T, d.S, d.H, d.rank, d.row, d.scale = B, T, S, m.heads, m.kv_rank, row, m.scale
    d.q, d.cache, d.starts, d.col_ptr = q.data_ptr(), c.data_ptr(), starts.data_ptr(), col_ptr.data_ptr()
    d.kv_chunk, d.ws, d.out, d.out_head = self._latent_chunk(m) if T == 1 else 0, self.attn_ws.data_ptr(), out.data_ptr(), out_head
    ops.latent_attn(d)

  def _mixer(self, ly, h, entry, col_ptr, starts, B, T) -> L.RowsSrc:
    m, M = ly["spec"].mixer, B * T
    at = (entry, col_ptr, starts, B, T)
    if isinstance(m, GatedStateMixer):
      out, normed = self.gated_state(ly, self.gated_in(ly["in"], h, M), *at)
      return self.linear(ly["out"], out if normed else self.head_norm(ly, out, M), M)
    src = self.linear(ly["in"], h, M)
    if isinstance(m, AttentionMixer):
      out = self.attend(ly, self.norm_kv(ly, src, *at) if m.row_norm else self.rotate(ly, src, *at), *at)
    elif isinstance(m, SsdMixer):
      u = None if T == 1 and ops.ssd_step_ok(m.state, m.vdim) else self.convolve(ly, src, *at)
      out = self.ssd_gate(ly, self.ssd(ly, src, u, *at), src, M)
    elif isinstance(m, LatentMixer):
      prompt = T > 1 and col_ptr is self.zero
      cq, ckv = self.latent_prep(ly, src, *at, expand=prompt)
      y, y_head = self.latent_prompt(ly, cq, ckv, *at) if prompt else self.latent_rows(ly, cq, *at)
      out = self.gate_mul(ly, y, m.vdim, y_head, src, M)
    else:
      out = self.gate(ly, self.recur(ly, src, *at), src, M)
    return self.linear(ly["out"], out, M)

  # experts
  def route(self, ly, h, M: int):
    """Chooses every row's experts and sorts the routes by expert."""
    e = ly["spec"].mlp
    src = self.fp32_rows(ly["router"], h, M, slot=0)
    ids = self.topk_id[:M * e.routes].view(M, e.routes)
    if e.corrected:
      ops.route_scores(src, M, e.experts, e.top, ly["correction"], e.scale, self.topk_w, ids, ly["router"].offsets[1] if e.shared_ff else 0,
                       self.gate_w if "shared_up" in ly else None, ld=e.routes)
    else:
      ops.route_softmax(src, M, e.experts, e.top, self.topk_w, ids)
    ops.moe_sort_routes(ids, len(ly["gu"]), self.counts, self.offsets, self.sorted_route)

  def experts_linear(self, f: LinearBank, x, x_frag: bool, x_div: int, routes: int, epilogue: int, y, ldy: int):
    d = L.DenseDesc()
    d.M, d.K, d.N, d.dtype = routes, f.Kp, f.N, self.code
    d.x, d.ldx, d.x_frag, d.w, d.w_stride = x.data_ptr(), x.shape[1], 1 if x_frag else 0, f.w.data_ptr(), f.stride
    d.epilogue, d.y, d.ldy, d.split_k = epilogue, y.data_ptr(), ldy, 1
    d.n_experts, d.x_div, d.offsets, d.sorted_route = len(f), x_div, self.offsets.data_ptr(), self.sorted_route.data_ptr()
    ops.dense_linear(d)

  def experts_gate_up(self, ly, h, M: int) -> torch.Tensor:
    e, f = ly["spec"].mlp, ly["gu"]
    act = self._buf("act", ly["down"].Kp, rows=self.M * e.routes)
    if not e.gated:
      self.experts_linear(f, h, self.frag, e.routes, M * e.routes, L.TNX_EPI_RELU2, act, act.shape[1])
    elif self.dtype == torch.float32:
      y = self.y[0][:M * e.routes * f.N].view(M * e.routes, f.N)
      self.experts_linear(f, h, False, e.routes, M * e.routes, L.TNX_EPI_STORE, y, f.N)
      ops.silu_mul(y, f.offsets[1], M * e.routes, e.ff, act)
    else:
      self.experts_linear(f, h, self.frag, e.routes, M * e.routes, L.TNX_EPI_SILU_MUL, act, act.shape[1])
    return act

  def experts_down(self, ly, act, M: int):
    """The routes' results, to be summed with their weights by the residual step."""
    e, f = ly["spec"].mlp, ly["down"]
    y = self._buf("routes", f.N, rows=self.M * e.routes)
    self.experts_linear(f, act, False, 1, M * e.routes, L.TNX_EPI_STORE, y, f.N)
    return ops.rows_src(y=y, ld=f.N)

  def _mlp(self, ly, h, M: int):
    """The feed-forward of h, as `residual_norm` takes it."""
    e = ly["spec"].mlp
    if isinstance(e, ExpertsMlp):
      self.route(ly, h, M)
      routes = ("routes", self.experts_down(ly, self.experts_gate_up(ly, h, M), M), ly["post2"], self.topk_w, e.routes)
      if "shared_up" in ly:
        routes += (self.linear(ly["shared_down"], self.shared_up(ly, h, M), M), self.gate_w)
      return routes
    if isinstance(e, PolyNormMlp):
      return ("add", self.linear(ly["down"], self.poly_up(ly, h, M), M), ly["post2"])
    return ("add", self.linear(ly["down"], self.gate_up(ly, h, M), M), ly["post2"])

  def shared_up(self, ly, h, M: int) -> torch.Tensor:
    """max(up h, 0)^2 of the expert that every token uses."""
    f, act = ly["shared_up"], self._buf("shared", ly["shared_down"].Kp)
    d = L.DenseDesc()
    d.M, d.K, d.N, d.dtype = M, f.Kp, f.N, self.code
    d.x, d.ldx, d.x_frag, d.w = h.data_ptr(), h.shape[1], 1 if self.frag else 0, f.w.data_ptr()
    d.epilogue, d.y, d.ldy, d.y_frag, d.split_k = L.TNX_EPI_RELU2, act.data_ptr(), act.shape[1], 1 if self.frag else 0, 1
    ops.dense_linear(d)
    return act

  def poly_up(self, ly, h, M: int) -> torch.Tensor:
    act = self._buf("act", ly["down"].Kp)
    ops.poly_norm(self.linear(ly["gu"], h, M), self.dtype, M, ly["spec"].mlp.ff, ly["act"], self.cfg.norm_eps, act, self.frag)
    return act

  def gate_up(self, ly, h, M: int, slot: int = 0) -> torch.Tensor:
    f = ly["gu"]
    act = self._buf("act", ly["down"].Kp)
    if self.dtype == torch.float32:
      self.linear(f, h, M, slot=slot)
      ops.gelu_mul(self.y[slot][:M * f.N].view(M, f.N), f.offsets[1], M, ly["spec"].mlp.ff, act)
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
    self.first = self.hist[0] if cfg.depth_average else None
    ops.embed_rows(m.embed, tokens, col_ptr, B, T, cfg.vocab_size, D, self.x if self.first is None else self.first, pos=m.pos, starts=starts, cat=cat, cat_off=D, cat_frag=self.frag, scale=cfg.embed_scale)
    h = self._buf("h", m.Dp)
    if cfg.parallel:
      return self._forward_parallel(h, col_ptr, cache, B, T, starts)
    pending, behind_layer = None if m.embed_norm is None else ("norm", None, m.embed_norm), False
    ended = None                                     # the layer that what is pending completes

    def norm(w_next, out, frag, shift=None):
      nonlocal behind_layer
      self.residual_norm(pending, w_next, out, M, frag, shift, behind=ended if behind_layer and cfg.depth_average else None)
      if behind_layer and self.residual_sink is not None:
        self.residual_sink(self.x[:M])
      behind_layer = False

    for (i, begins), entry in zip(cfg.layer_runs, cache.entries):
      ly = m.layers[i]
      if begins:   # a pass of the loop: x <- W [x; embedding output]
        norm(None, cat, self.frag)
        pending = ("set", self.linear(m.loop_in, cat, M, fp32_out=True), None)
      if cfg.token_shift:
        norm(None, h, self.frag, (ly["shift"], entry["shift"].r, col_ptr, starts, B, T))
        entry = entry["mixer"]
      else:
        norm(ly["norm1"], h, self.frag)
      pending = ("add", self._mixer(ly, h, entry, col_ptr, starts, B, T), ly["post1"])
      if "gu" in ly:
        norm(ly["norm2"], h, self.frag)
        pending = self._mlp(ly, h, M)
      behind_layer, ended = True, i
    norm(m.final_norm, self.xn, False)
    return self.xn

  def _forward_parallel(self, h, col_ptr, cache, B, T, starts):
    m, cfg, at = self.model, self.cfg, (col_ptr, starts, B, T)
    h2, pending, passes = self._buf("h2", m.Dp), None, 0
    for (i, begins), entry in zip(cfg.layer_runs, cache.entries):
      add = None
      if begins:   # a pass of the loop: x <- x + the pass's vector
        add, passes = m.loop_step[passes], passes + 1
      if self.residual_sink is not None and pending is not None:   # (the layer's own result is asked for, without what comes ahead of the next)
        self.parallel_step(pending, None, self.xn, None, at, None)
        self.residual_sink(self.x[:B * T])
        pending = None
      self.parallel_step(pending, m.layers[i], h, h2, at, entry, add)
      pending = self.parallel_sublayers(m.layers[i], h, h2, entry, *at)
    self.parallel_step(pending, None, self.xn, None, at, None)
    if self.residual_sink is not None:
      self.residual_sink(self.x[:B * T])
    return self.xn

  # ---- head ----------------------------------------------------------------------------------
  def head_desc(self, *args, **kw) -> L.LmHeadDesc:
    d = super().head_desc(*args, **kw)
    d.softcap = self.cfg.logit_softcap
    return d

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
    if self.cfg.logit_softcap > 0.0:
      ops.soft_cap(logits_out[:rows], self.cfg.logit_softcap)
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
