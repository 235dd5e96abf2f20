"""Model descriptions for the decode path: the three families the sampler runs
(tunix/models/llama3/model.py:85-187, qwen3/model.py ModelConfig, gemma3/model.py:93-300)
plus the qwix-style QLoRA settings (tunix/cli/utils/model.py:31-77).
"""
from __future__ import annotations

import dataclasses

Q_INT4, Q_NF4 = 0, 1
QTYPE_BY_NAME = {"int4": Q_INT4, "nf4": Q_NF4}

# 5 local sliding-window layers, then 1 global (tunix/models/gemma3/model.py:441-448)
GEMMA3_PATTERN_LEN = 6

ATTN_LINEARS = ("wq", "wk", "wv", "wo")
MLP_LINEARS = ("w_gate", "w_up", "w_down")


@dataclasses.dataclass
class ModelConfig:
  family: str                      # 'llama3' | 'qwen3' | 'gemma3'
  num_layers: int
  vocab_size: int
  embed_dim: int
  hidden_dim: int                  # dense MLP width, or per-expert width for MoE
  num_heads: int
  num_kv_heads: int
  head_dim: int
  norm_eps: float = 1e-6
  # RoPE base actually used.  Llama3 and Qwen3 attention call apply_rope without rope_theta
  # (llama3/model.py:356-365, qwen3/model.py:545-554), so the default 1e6 applies whatever the
  # checkpoint config says.
  rope_theta: float = 1_000_000.0
  tied_embedding: bool = False
  # quantisation of the linears (None: dense bf16, not built)
  qtype: int = Q_INT4
  group: int = 64
  int4_bound: float = 7.0          # int4 scale = group absmax / this bound (codes clamp to [-8, 7])
  quantize_head: bool = False      # lm_head stays bf16 unless set (module_path never matches it)
  # LoRA
  lora_rank: int = 0
  lora_alpha: float = 0.0
  lora_targets: tuple = ATTN_LINEARS + MLP_LINEARS
  head_lora: bool = False
  # MoE (qwen3)
  num_experts: int = 0
  num_experts_per_tok: int = 0
  # gemma3
  sliding_window: int = 0
  local_base_frequency: float = 10_000.0
  global_base_frequency: float = 1_000_000.0
  local_scale_factor: float = 1.0
  global_scale_factor: float = 1.0
  query_pre_attn_scalar: float = 0.0

  def __post_init__(self):
    if self.family not in ("llama3", "qwen3", "gemma3"):
      raise ValueError(f"unknown model family {self.family!r}")
    if self.family == "gemma3" and self.query_pre_attn_scalar == 0.0:
      self.query_pre_attn_scalar = self.head_dim ** -0.5
    if self.num_heads % self.num_kv_heads:
      raise ValueError("num_heads must be a multiple of num_kv_heads")

  # ---- helpers shared by the engine and by checkers ----------------------------------------
  def is_local_layer(self, i: int) -> bool:
    return self.family == "gemma3" and (i % GEMMA3_PATTERN_LEN) != GEMMA3_PATTERN_LEN - 1

  def rope_params(self, i: int) -> tuple[float, float]:
    """(base frequency, scale factor) of layer i (gemma3/model.py:838-846)."""
    if self.family != "gemma3":
      return float(self.rope_theta), 1.0
    if self.is_local_layer(i):
      return float(self.local_base_frequency), float(self.local_scale_factor)
    return float(self.global_base_frequency), float(self.global_scale_factor)

  def layer_linear_names(self, i: int) -> list[str]:
    p = f"l{i}."
    names = [p + n for n in ATTN_LINEARS]
    if self.num_experts:
      names += [p + "e_gate", p + "e_up", p + "e_down"]
    else:
      names += [p + n for n in MLP_LINEARS]
    return names

  def quantized_names(self) -> list[str]:
    names = []
    for i in range(self.num_layers):
      names += self.layer_linear_names(i)
    if self.quantize_head and not self.tied_embedding:
      names.append("lm_head")
    return names

  def lora_names(self) -> list[str]:
    if self.lora_rank <= 0:
      return []
    names = [f"l{i}.{n}" for i in range(self.num_layers) for n in self.lora_targets]
    if self.head_lora:
      names.append("lm_head")
    return names

  @property
  def q_dim(self) -> int:
    return self.num_heads * self.head_dim

  @property
  def kv_dim(self) -> int:
    return self.num_kv_heads * self.head_dim


# ---- decoders described as a list of layers (dense weights, fp32 residual stream) --------------
@dataclasses.dataclass(frozen=True)
class AttentionMixer:
  """Causal grouped-query attention: separate key and value head sizes, rotation of the first
  rot_dims dimensions of q and k, any score scale, optionally a learned sink per query head.
  row_norm: q and k are normed, each over all its heads together (then nothing rotates).  slopes: what a head takes off a
  score per position of distance (empty: nothing).  chunk > 0: a position sees its own chunk of that many positions only.
  kv_from: the layer whose keys and values (its cache entry) this one reads instead of its own."""
  heads: int
  kv_heads: int
  dim: int
  vdim: int
  rot_dims: int
  rot_base: float
  scale: float
  sink: bool = True
  row_norm: bool = False
  slopes: tuple = ()
  chunk: int = 0
  kv_from: int | None = None

  def __post_init__(self):
    if self.heads % self.kv_heads:
      raise ValueError("heads must be a multiple of kv_heads")
    if self.rot_dims % 2 or not 0 <= self.rot_dims <= self.dim:
      raise ValueError(f"rot_dims={self.rot_dims} must be even and at most the head size {self.dim}")
    if self.slopes and len(self.slopes) != self.heads:
      raise ValueError(f"{len(self.slopes)} slopes for {self.heads} heads")
    if self.chunk < 0:
      raise ValueError(f"chunk={self.chunk} must not be negative")
    if self.row_norm and self.rot_dims or self.kv_from is not None and not self.row_norm:
      raise ValueError("normed projections do not rotate, and only they may borrow keys and values")

  def weight_shapes(self, D: int) -> dict[str, tuple]:
    rows = {"q": self.heads * self.dim, "k": self.kv_heads * self.dim, "v": self.kv_heads * self.vdim}
    own = ("q",) if self.kv_from is not None else ("q", "k", "v")
    out = {n: (rows[n], D) for n in own}
    out["o"] = (D, self.heads * self.vdim)
    if self.row_norm:
      out.update({n + ".norm": (rows[n],) for n in own if n != "v"})
    if self.sink:
      out["sink"] = (self.heads,)
    return out


def distance_slopes(heads: int) -> tuple:
  """2^(-8 (h + 1) / heads) for head h."""
  return tuple(2.0 ** (-8.0 * (h + 1) / heads) for h in range(heads))


@dataclasses.dataclass(frozen=True)
class MixedAttentionMixer:
  """Causal grouped-query attention without rotation: q, k and v behind a short causal convolution of `conv`
  taps, queries scaled by 1 + temp_coef ln(floor((p + 1) / temp_every) + 1) at position p, value heads divided
  by their root mean square (value_norm), softmax weights mixed between the heads, output gate."""
  heads: int
  kv_heads: int
  dim: int
  vdim: int
  conv: int
  scale: float
  temp_coef: float = 0.0
  temp_every: float = 1.0
  value_norm: bool = True

  def __post_init__(self):
    if self.heads % self.kv_heads:
      raise ValueError("heads must be a multiple of kv_heads")
    if self.conv < 1:
      raise ValueError("the convolution needs a tap")
    if not self.temp_every > 0:
      raise ValueError(f"temp_every={self.temp_every} must be positive")

  def weight_shapes(self, D: int) -> dict[str, tuple]:
    H, rows = self.heads, {"q": self.heads * self.dim, "k": self.kv_heads * self.dim, "v": self.kv_heads * self.vdim}
    out = {n: (r, D) for n, r in rows.items()}
    out.update({n + ".conv": (r, self.conv) for n, r in rows.items()})
    out.update({"talk": (H, H), "g": (H * self.vdim, D), "o": (D, H * self.vdim)})
    return out


@dataclasses.dataclass(frozen=True)
class MemoryMixer:
  """Matrix memory with exponential gates (mLSTM): per head a matrix state [dim, vdim], a sum of keys and a
  running maximum; gates capped at gate_cap; heads normed on their own, gated and projected."""
  heads: int
  dim: int
  vdim: int
  gate_cap: float

  def __post_init__(self):
    if not self.gate_cap > 0:
      raise ValueError(f"gate_cap={self.gate_cap} must be positive")

  def weight_shapes(self, D: int) -> dict[str, tuple]:
    H, qk, v = self.heads, self.heads * self.dim, self.heads * self.vdim
    return {"q": (qk, D), "k": (qk, D), "v": (v, D), "g": (v, D), "i": (H, D), "i.b": (H,), "f": (H, D), "f.b": (H,), "norm": (v,), "o": (D, v)}


@dataclasses.dataclass(frozen=True)
class ParallelMixer:
  """Two mixers side by side that read one input; half the sum of their outputs, each normed over the width."""
  left: MixedAttentionMixer
  right: MemoryMixer

  @property
  def sides(self) -> tuple:
    return (("left", self.left), ("right", self.right))

  def weight_shapes(self, D: int) -> dict[str, tuple]:
    out = {}
    for side, m in self.sides:
      out.update({f"{side}.{k}": s for k, s in m.weight_shapes(D).items()})
      out[side + ".out"] = (D,)
    return out


@dataclasses.dataclass(frozen=True)
class LightningMixer:
  """Linear attention with one constant decay per head and a matrix state per head; the heads'
  outputs are normed together, gated and projected."""
  heads: int
  dim: int
  vdim: int
  decay: tuple

  def __post_init__(self):
    if len(self.decay) != self.heads:
      raise ValueError(f"{len(self.decay)} decays for {self.heads} heads")

  def weight_shapes(self, D: int) -> dict[str, tuple]:
    qk, v = self.heads * self.dim, self.heads * self.vdim
    return {"q": (qk, D), "k": (qk, D), "v": (v, D), "g": (v, D), "norm": (v,), "o": (D, v)}


@dataclasses.dataclass(frozen=True)
class GatedStateMixer:
  """Linear attention with a forget gate per head and channel, bounded below, whose complement writes (HGRN2): a matrix state
  [dim, vdim] per head; heads normed on their own with shared weights, then projected."""
  heads: int
  dim: int
  vdim: int

  def weight_shapes(self, D: int) -> dict[str, tuple]:
    qk, v = self.heads * self.dim, self.heads * self.vdim
    return {"q": (qk, D), "f": (qk, D), "f.b": (qk,), "lower": (qk,), "v": (v, D), "norm": (self.vdim,), "o": (D, v)}


@dataclasses.dataclass(frozen=True)
class SsdMixer:
  """State-space duality: per head a matrix state [state, vdim] whose decay depends on the token; inputs
  behind a short causal convolution, B and C shared by the heads of a group; the heads' outputs gated,
  then normed in norm_groups equal parts and projected."""
  heads: int
  vdim: int
  state: int
  groups: int
  conv: int
  norm_groups: int

  def __post_init__(self):
    if self.heads % self.groups:
      raise ValueError("heads must be a multiple of groups")
    if self.inner % self.norm_groups:
      raise ValueError(f"{self.inner} values do not divide into {self.norm_groups} norm groups")
    if self.conv < 1:
      raise ValueError("the convolution needs a tap")

  @property
  def inner(self) -> int:
    return self.heads * self.vdim

  @property
  def channels(self) -> int:
    """Of the convolution: x, B and C."""
    return self.inner + 2 * self.groups * self.state

  def weight_shapes(self, D: int) -> dict[str, tuple]:
    C, H = self.channels, self.heads
    return {"in": (self.inner + C + H, D), "conv": (C, self.conv), "conv.b": (C,), "dt_bias": (H,), "A_log": (H,), "D": (H,),
            "norm": (self.inner,), "o": (D, self.inner)}


@dataclasses.dataclass(frozen=True)
class LatentMixer:
  """Causal attention whose keys and values are linear in a normed latent of size kv_rank (all that is
  cached, beside one rotated key part shared by the heads); queries through a latent of size q_rank; `dim`
  unrotated and rot_dim rotated query / key dimensions per head; output gate."""
  heads: int
  dim: int
  rot_dim: int
  vdim: int
  q_rank: int
  kv_rank: int
  rot_base: float
  scale: float

  def __post_init__(self):
    if self.rot_dim % 2 or self.rot_dim < 0:
      raise ValueError(f"rot_dim={self.rot_dim} must be even")

  def weight_shapes(self, D: int) -> dict[str, tuple]:
    H = self.heads
    return {"dq": (self.q_rank, D), "dq.norm": (self.q_rank,), "uq": (H * (self.dim + self.rot_dim), self.q_rank),
            "dkv": (self.kv_rank + self.rot_dim, D), "dkv.norm": (self.kv_rank,), "uk": (H * self.dim, self.kv_rank),
            "uv": (H * self.vdim, self.kv_rank), "g": (H * self.vdim, D), "o": (D, H * self.vdim)}


@dataclasses.dataclass(frozen=True)
class GatedMlp:
  """down(gelu_tanh(gate h) * (up h))."""
  ff: int

  def weight_shapes(self, D: int) -> dict[str, tuple]:
    return {"gate": (self.ff, D), "up": (self.ff, D), "down": (D, self.ff)}


@dataclasses.dataclass(frozen=True)
class PolyNormMlp:
  """down(a norm(z) + b norm(z^2) + c norm(z^3) + e) with z = up h, norms over the row and four learned numbers."""
  ff: int

  def weight_shapes(self, D: int) -> dict[str, tuple]:
    return {"up": (self.ff, D), "down": (D, self.ff), "act": (4,)}


@dataclasses.dataclass(frozen=True)
class ExpertsMlp:
  """The weighted sum of the `top` chosen experts: down(silu(gate h) * (up h)), or down(max(up h, 0)^2) when not gated.
  Chosen are the largest router logits, weights the softmax over them; corrected: chosen are the largest of softmax over all
  logits + a correction per expert, weights the chosen scores over their sum, times scale.  shared_ff > 0: one more expert of
  that size for every token, times a sigmoid of its own (not gated and corrected experts only)."""
  ff: int
  experts: int
  top: int
  gated: bool = True
  corrected: bool = False
  scale: float = 1.0
  shared_ff: int = 0

  def __post_init__(self):
    if not 1 <= self.top <= self.experts:
      raise ValueError(f"{self.top} of {self.experts} experts")
    if self.shared_ff and (self.gated or not self.corrected) or not self.corrected and self.scale != 1.0:
      raise ValueError("a shared expert and a scale go with corrected scores")

  @property
  def shared_routes(self) -> int:
    """A shared expert of up to four times the others' size is as many more experts, to which every token is routed (0: it
    runs apart): the square is taken element by element."""
    n = self.shared_ff // self.ff
    return n if n * self.ff == self.shared_ff and n <= 4 else 0

  @property
  def routes(self) -> int:
    """Experts that a token is routed to."""
    return self.top + self.shared_routes

  def weight_shapes(self, D: int) -> dict[str, tuple]:
    out = {"router": (self.experts, D)}
    if self.corrected:
      out["correction"] = (self.experts,)
    sizes = [(f"e{e}", self.ff) for e in range(self.experts)] + ([("shared", self.shared_ff)] if self.shared_ff else [])
    for name, ff in sizes:
      out.update({f"{name}.{n}": (ff, D) for n in (("gate", "up") if self.gated else ("up",))})
      out[name + ".down"] = (D, ff)
    if self.shared_ff:
      out["shared.sg"] = (1, D)
    return out


@dataclasses.dataclass(frozen=True)
class LayerSpec:
  mixer: AttentionMixer | LightningMixer | SsdMixer | LatentMixer | ParallelMixer | GatedStateMixer
  mlp: GatedMlp | PolyNormMlp | ExpertsMlp | None


@dataclasses.dataclass(frozen=True)
class LayerLoop:
  """Layers start .. stop - 1 run `times` times; before each pass x <- W [x; embedding output], or with `step` x <- x + the
  pass's own vector."""
  start: int
  stop: int
  times: int
  step: bool = False


@dataclasses.dataclass(frozen=True)
class StackConfig:
  """A decoder given layer by layer.  Every sublayer is x += residual_mult norm(f(norm(x))), or x += norm(f(x)) without
  pre_norm, with norm weights stored as an offset from `norm_offset` and norms taken over norm_groups equal
  parts of the row.  embed_norm: the embedding is normed.  token_shift:
  what a mixer reads is first moved towards the same of the token before, per element.
  parallel: x += residual_mult (mixer(h1) + mlp(h2)) with h = norm(x) and h1, h2 = h + a causal convolution of input_conv
  taps of h, per sublayer.  center_norm: norms are layer norms.  max_positions > 0: a learned vector per position is added to the
  embedding, and a sequence has at most so many positions.  depth_average: behind layer i, x <- sum over j <= i + 1 of
  l<i>.dwa[j] X_j with X_0 the embedding output and X_(j+1) layer j's result.  tied_head: the head is the embedding table.  logit_softcap > 0: logits <- cap tanh(logits / cap)."""
  family: str
  vocab_size: int
  embed_dim: int
  layers: tuple
  norm_eps: float
  loop: LayerLoop | None = None
  norm_offset: float = 1.0
  norm_groups: int = 1
  pre_norm: bool = True
  embed_norm: bool = False
  token_shift: bool = False
  parallel: bool = False
  residual_mult: float = 1.0
  input_conv: int = 0
  embed_scale: float = 1.0
  tied_head: bool = True
  logit_softcap: float = 0.0
  center_norm: bool = False
  max_positions: int = 0
  depth_average: bool = False

  def __post_init__(self):
    n, lp = len(self.layers), self.loop
    if any(isinstance(ly.mixer, ParallelMixer) != self.parallel for ly in self.layers):
      raise ValueError("parallel layers are made of parallel mixers, and no others are")
    if self.parallel and (self.input_conv < 1 or self.norm_groups != 1 or self.norm_offset != 0.0 or not self.pre_norm or self.embed_norm or self.token_shift):
      raise ValueError("parallel layers have one plain norm in front and input convolutions")
    if lp is not None and lp.step != self.parallel:
      raise ValueError("a loop over parallel layers adds its pass's vector, no other does")
    if lp is not None and not (0 <= lp.start < lp.stop <= n and lp.times >= 1):
      raise ValueError(f"the loop {lp} does not fit {n} layers")
    if self.embed_dim % self.norm_groups:
      raise ValueError(f"width {self.embed_dim} does not divide into {self.norm_groups} norm groups")
    if self.token_shift and self.pre_norm:
      raise ValueError("a token shift goes with norms behind the sublayers only")
    if self.center_norm or self.depth_average or (self.residual_mult != 1.0 and not self.parallel):
      if self.parallel or self.token_shift or self.norm_groups != 1 or not self.pre_norm or self.embed_norm or lp is not None:
        raise ValueError("layer norms, a residual factor and the depth average go with plain pre-normed layers that run once")
    for i, ly in enumerate(self.layers):
      j = getattr(ly.mixer, "kv_from", None)
      if j is None:
        continue
      src = self.layers[j].mixer if 0 <= j < i else None
      if lp is not None or not isinstance(src, AttentionMixer) or src.kv_from is not None:
        raise ValueError(f"layer {i} reads the keys of layer {j}, which is no earlier attention layer with keys of its own")
      if any(getattr(src, n) != getattr(ly.mixer, n) for n in ("heads", "kv_heads", "dim", "vdim")):
        raise ValueError(f"layer {i} reads the keys of layer {j}, whose heads differ")

  def post_norm(self, n: int) -> str:
    """Name of the norm behind a layer's mixer (n = 1) or feed-forward (2)."""
    return f"norm{n}b" if self.pre_norm else f"norm{n}"

  @property
  def num_layers(self) -> int:
    return len(self.layers)

  @property
  def layer_runs(self) -> list[tuple[int, bool]]:
    """(layer, whether a pass of the loop begins with it) in running order: one cache entry each."""
    n, lp = self.num_layers, self.loop
    if lp is None:
      return [(i, False) for i in range(n)]
    one = [(i, i == lp.start) for i in range(lp.start, lp.stop)]
    return [(i, False) for i in range(lp.start)] + one * lp.times + [(i, False) for i in range(lp.stop, n)]

  def weight_shapes(self) -> dict[str, tuple]:
    """Name -> shape of every tensor; linear weights are [out, in]."""
    D = self.embed_dim
    out = {"embed": (self.vocab_size, D), "final.norm": (D,)}
    if self.embed_norm:
      out["embed.norm"] = (D,)
    if not self.tied_head:
      out["head"] = (self.vocab_size, D)
    if self.max_positions:
      out["pos"] = (self.max_positions, D)
    if self.loop is not None:
      out.update({"loop.step": (self.loop.times, D)} if self.loop.step else {"loop.in": (D, 2 * D)})
    for i, ly in enumerate(self.layers):
      p = f"l{i}."
      parts = [(1, "mix.", ly.mixer)] + ([(2, "mlp.", ly.mlp)] if ly.mlp is not None else [])
      if self.token_shift:
        out[p + "shift"] = (D,)
      if self.depth_average:
        out[p + "dwa"] = (i + 2,)
      for n, at, part in parts:
        if self.pre_norm and not (self.parallel and n == 2):
          out[p + f"norm{n}"] = (D,)
        if self.parallel:
          out[p + f"canon{n}"] = (D, self.input_conv)
        else:
          out[p + self.post_norm(n)] = (D,)
        out.update({p + at + k: s for k, s in part.weight_shapes(D).items()})
    return out


def lapevik_from_dict(d: dict) -> StackConfig:
  """Reads a Lapevik config.json."""
  layers = []
  for i, ly in enumerate(d["layers"]):
    m = ly["mixer"]
    if ly["type"] in ("mamba2", "mamba2_2"):
      mixer = SsdMixer(heads=int(m["heads"]), vdim=int(m["vdim"]), state=int(m["state"]), groups=int(m["groups"]),
                       conv=int(m["conv"]), norm_groups=int(m["norm_groups"]))
    elif ly["type"] == "latent_attention":
      rot = m["rot"] if int(m["rot_dim"]) else {"dims": 0, "base": 1.0}
      if int(rot["dims"]) != int(m["rot_dim"]):
        raise ValueError(f"layer {i}: rotation over {rot['dims']} of {m['rot_dim']} dimensions")
      mixer = LatentMixer(heads=int(m["heads"]), dim=int(m["dim"]), rot_dim=int(m["rot_dim"]), vdim=int(m["vdim"]),
                          q_rank=int(m["q_rank"]), kv_rank=int(m["kv_rank"]), rot_base=float(rot["base"]), scale=float(m["scale"]))
    else:
      raise ValueError(f"layer {i}: unknown mixer type {ly['type']!r}")
    mlp = ly.get("mlp")
    if mlp is not None:
      if mlp["kind"] != "moe":
        raise ValueError(f"layer {i}: unknown feed-forward kind {mlp['kind']!r}")
      mlp = ExpertsMlp(ff=int(mlp["expert"]["ff"]), experts=int(mlp["router"]["experts"]), top=int(mlp["router"]["top"]))
    layers.append(LayerSpec(mixer, mlp))
  return StackConfig(family="lapevik", vocab_size=int(d["vocab"]), embed_dim=int(d["width"]), layers=tuple(layers),
                     norm_eps=float(d["norm"]["eps"]), norm_offset=0.0, norm_groups=int(d["norm"]["groups"]), pre_norm=False,
                     embed_norm=True, token_shift=True)


def nunezen_from_dict(d: dict) -> StackConfig:
  """Reads a Nunezen config.json."""
  layers = []
  for i, ly in enumerate(d["layers"]):
    m = ly["mixer"]
    if ly["type"] == "attention":
      rot = m["rot"]
      mixer = AttentionMixer(heads=int(m["heads"]), kv_heads=int(m["kv_heads"]), dim=int(m["dim"]), vdim=int(m["vdim"]),
                             rot_dims=int(rot["dims"]), rot_base=float(rot["base"]), scale=float(m["scale"]))
    elif ly["type"] == "lightning":
      mixer = LightningMixer(heads=int(m["heads"]), dim=int(m["dim"]), vdim=int(m["vdim"]),
                             decay=tuple(float(x) for x in m["decay"]))
    else:
      raise ValueError(f"layer {i}: unknown mixer type {ly['type']!r}")
    mlp = ly.get("mlp")
    if mlp is not None and mlp["kind"] != "dense":
      raise ValueError(f"layer {i}: unknown feed-forward kind {mlp['kind']!r}")
    layers.append(LayerSpec(mixer, None if mlp is None else GatedMlp(int(mlp["ff"]))))
  lp = d.get("loop")
  return StackConfig(family="nunezen", vocab_size=int(d["vocab"]), embed_dim=int(d["width"]), layers=tuple(layers),
                     norm_eps=float(d["norm"]["eps"]),
                     loop=None if lp is None else LayerLoop(int(lp["start"]), int(lp["stop"]), int(lp["times"])))


def kuzezen_from_dict(d: dict) -> StackConfig:
  """Reads a Kuzezen config.json."""
  layers = []
  for i, ly in enumerate(d["layers"]):
    if ly["type"] != "parallel":
      raise ValueError(f"layer {i}: unknown mixer type {ly['type']!r}")
    a, b = ly["mixer"]["left"], ly["mixer"]["right"]
    left = MixedAttentionMixer(heads=int(a["heads"]), kv_heads=int(a["kv_heads"]), dim=int(a["dim"]), vdim=int(a["vdim"]), conv=int(a["conv"]),
                               scale=float(a["scale"]), temp_coef=float(a["q_temp"]["coef"]), temp_every=float(a["q_temp"]["every"]))
    right = MemoryMixer(heads=int(b["heads"]), dim=int(b["dim"]), vdim=int(b["vdim"]), gate_cap=float(b["gate_cap"]))
    mlp = ly.get("mlp")
    if mlp is not None and mlp["kind"] != "dense":
      raise ValueError(f"layer {i}: unknown feed-forward kind {mlp['kind']!r}")
    layers.append(LayerSpec(ParallelMixer(left, right), None if mlp is None else GatedMlp(int(mlp["ff"]))))
  lp = d.get("loop")
  return StackConfig(family="kuzezen", vocab_size=int(d["vocab"]), embed_dim=int(d["width"]), layers=tuple(layers), norm_eps=float(d["norm"]["eps"]),
                     loop=None if lp is None else LayerLoop(int(lp["start"]), int(lp["stop"]), int(lp["times"]), step=True), norm_offset=0.0,
                     parallel=True, residual_mult=float(d["residual_mult"]), input_conv=int(d["canon"]["taps"]),
                     embed_scale=float(d["embedding"]["scale"]), tied_head=False, logit_softcap=float(d["logit_softcap"]))


def kezolix_from_dict(d: dict) -> StackConfig:
  """Reads a Kezolix config.json."""
  layers = []
  for i, ly in enumerate(d["layers"]):
    m = ly["mixer"]
    if ly["type"] == "attention":
      heads, mask, kv_from = int(m["heads"]), m.get("mask"), m.get("kv_from")
      if mask is not None and int(mask["size"]) < 1:
        raise ValueError(f"layer {i}: a chunk of {mask['size']} positions")
      mixer = AttentionMixer(heads=heads, kv_heads=int(m["kv_heads"]), dim=int(m["dim"]), vdim=int(m["vdim"]), rot_dims=0, rot_base=1.0,
                             scale=float(m["scale"]), sink=False, row_norm=True, slopes=distance_slopes(heads),
                             chunk=0 if mask is None else int(mask["size"]), kv_from=None if kv_from is None else int(kv_from))
    elif ly["type"] == "hgrn2":
      mixer = GatedStateMixer(heads=int(m["heads"]), dim=int(m["dim"]), vdim=int(m["vdim"]))
    else:
      raise ValueError(f"layer {i}: unknown mixer type {ly['type']!r}")
    mlp = ly.get("mlp")
    if mlp is not None:
      if mlp["kind"] == "dense":
        mlp = PolyNormMlp(int(mlp["ff"]))
      elif mlp["kind"] == "moe":
        r, shared = mlp["router"], mlp.get("shared")
        mlp = ExpertsMlp(ff=int(mlp["expert"]["ff"]), experts=int(r["experts"]), top=int(r["top"]), gated=False, corrected=True,
                         scale=float(r["scale"]), shared_ff=0 if shared is None else int(shared["ff"]))
      else:
        raise ValueError(f"layer {i}: unknown feed-forward kind {mlp['kind']!r}")
    layers.append(LayerSpec(mixer, mlp))
  return StackConfig(family="kezolix", vocab_size=int(d["vocab"]), embed_dim=int(d["width"]), layers=tuple(layers), norm_eps=float(d["norm"]["eps"]),
                     norm_offset=0.0, residual_mult=float(d["residual_mult"]), tied_head=False, center_norm=True,
                     max_positions=int(d["max_positions"]), depth_average=True)


# ---- the shapes the headline metric and the parity cases are quoted on ------------------------
def tiny_qwen3(**kw) -> ModelConfig:
  """2-layer Qwen3-style decoder: D512, 8q/2kv, dh64, MLP 1536, V32000, int4 g64, LoRA r8."""
  d = dict(family="qwen3", num_layers=2, vocab_size=32000, embed_dim=512, hidden_dim=1536,
           num_heads=8, num_kv_heads=2, head_dim=64, norm_eps=1e-6, qtype=Q_INT4, group=64,
           lora_rank=8, lora_alpha=8.0)
  d.update(kw)
  return ModelConfig(**d)


def gemma3_1b(**kw) -> ModelConfig:
  """Gemma3-1B shape (gemma3/model.py:158-174): int4 g128, LoRA r16, tied embeddings."""
  d = dict(family="gemma3", num_layers=26, vocab_size=262144, embed_dim=1152, hidden_dim=6912,
           num_heads=4, num_kv_heads=1, head_dim=256, norm_eps=1e-6, tied_embedding=True,
           qtype=Q_INT4, group=128, lora_rank=16, lora_alpha=16.0, sliding_window=512,
           local_base_frequency=10_000.0, global_base_frequency=1_000_000.0)
  d.update(kw)
  return ModelConfig(**d)


def llama31_8b(**kw) -> ModelConfig:
  """Llama-3.1-8B shape (llama3/model.py:143-155): NF4 g64 with bf16 scales, LoRA r64."""
  d = dict(family="llama3", num_layers=32, vocab_size=128256, embed_dim=4096, hidden_dim=14336,
           num_heads=32, num_kv_heads=8, head_dim=128, norm_eps=1e-5, qtype=Q_NF4, group=64,
           lora_rank=64, lora_alpha=64.0)
  d.update(kw)
  return ModelConfig(**d)


def qwen3_30b_a3b(**kw) -> ModelConfig:
  """Qwen3-30B-A3B shape: 128 experts top-8, expert MLP 768, int4 g128, LoRA r16 on attention."""
  d = dict(family="qwen3", num_layers=48, vocab_size=151936, embed_dim=2048, hidden_dim=768,
           num_heads=32, num_kv_heads=4, head_dim=128, norm_eps=1e-6, qtype=Q_INT4, group=128,
           lora_rank=16, lora_alpha=16.0, lora_targets=ATTN_LINEARS, num_experts=128,
           num_experts_per_tok=8)
  d.update(kw)
  return ModelConfig(**d)


def nunezen_shape(width: int, heads: int, kv_heads: int, ff: int, vocab: int = 32768, dim: int = 128,
                  layers: int = 4) -> StackConfig:
  """A Nunezen decoder with layers of a real model's size: attention (+ feed-forward) and lightning
  layers in turn, the middle layers run twice."""
  attn = LayerSpec(AttentionMixer(heads, kv_heads, dim, dim, dim // 2, 500_000.0, dim ** -0.5), GatedMlp(ff))
  decay = tuple(1.0 - 2.0 ** (-1.0 - 8.0 * h / max(heads - 1, 1)) for h in range(heads))
  light = LayerSpec(LightningMixer(heads, dim, dim, decay), None)
  return StackConfig(family="nunezen", vocab_size=vocab, embed_dim=width, norm_eps=1e-6,
                     layers=tuple(attn if i % 2 == 0 else light for i in range(layers)),
                     loop=LayerLoop(1, layers - 1, 2) if layers > 2 else None)


def lapevik_shape(width: int, heads: int, experts: int, top: int, ff: int, vocab: int = 32768, layers: int = 4) -> StackConfig:
  """A Lapevik decoder with layers of a real model's size: state-space and latent-attention layers in turn, each
  with routed experts."""
  moe = ExpertsMlp(ff, experts, top)
  ssd = LayerSpec(SsdMixer(heads=width // 32, vdim=64, state=128, groups=8, conv=4, norm_groups=8), moe)
  attn = LayerSpec(LatentMixer(heads, 128, 64, 128, q_rank=3 * width // 8, kv_rank=512, rot_base=500_000.0, scale=192 ** -0.5), moe)
  return StackConfig(family="lapevik", vocab_size=vocab, embed_dim=width, norm_eps=1e-5, norm_offset=0.0, norm_groups=8, pre_norm=False,
                     embed_norm=True, token_shift=True, layers=tuple(ssd if i % 2 == 0 else attn for i in range(layers)))


def kuzezen_shape(width: int, heads: int, kv_heads: int, ff: int, vocab: int = 32768, dim: int = 128, layers: int = 4) -> StackConfig:
  """A Kuzezen decoder with layers of a real model's size: mixed attention and matrix memory side by side, each with as many
  heads, the middle layers run twice."""
  mixer = ParallelMixer(MixedAttentionMixer(heads, kv_heads, dim, dim, 4, dim ** -0.5, 0.1, 8192.0), MemoryMixer(heads, dim, dim, 15.0))
  return StackConfig(family="kuzezen", vocab_size=vocab, embed_dim=width, norm_eps=1e-6, layers=(LayerSpec(mixer, GatedMlp(ff)),) * layers,
                     loop=LayerLoop(1, layers - 1, 2, step=True) if layers > 2 else None, norm_offset=0.0, parallel=True, residual_mult=0.5,
                     input_conv=4, embed_scale=width ** 0.5, tied_head=False, logit_softcap=30.0)


def kezolix_shape(width: int, heads: int, kv_heads: int, ff: int, experts: int, top: int, expert_ff: int, vocab: int = 32768, dim: int = 128,
                  chunk: int = 2048, layers: int = 6, positions: int = 8192) -> StackConfig:
  """A Kezolix decoder with layers of a real model's size: recurrent and attention layers in turn, the first with a dense
  feed-forward, the others with routed and shared experts; the last attention layer reads the keys of the first."""
  moe = ExpertsMlp(expert_ff, experts, top, gated=False, corrected=True, scale=2.5, shared_ff=expert_ff)
  attn = lambda kv_from: AttentionMixer(heads, kv_heads, dim, dim, 0, 1.0, dim ** -0.5, sink=False, row_norm=True, slopes=distance_slopes(heads),
                                        chunk=chunk, kv_from=kv_from)
  out = []
  for i in range(layers):
    mixer = GatedStateMixer(heads, dim, dim) if i % 2 == 0 else attn(1 if i > 1 and i >= layers - 2 else None)
    out.append(LayerSpec(mixer, PolyNormMlp(ff) if i == 0 else moe))
  return StackConfig(family="kezolix", vocab_size=vocab, embed_dim=width, norm_eps=1e-6, layers=tuple(out), norm_offset=0.0, residual_mult=0.5,
                     tied_head=False, center_norm=True, max_positions=positions, depth_average=True)
