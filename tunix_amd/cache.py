"""What a batch of sequences carries from one forward pass to the next: one entry per layer run,
a key / value slab (attention), a slab of latents, a recurrent state, a ring of the last columns' rows,
or several of these.  A layer that runs several times has one entry per run; one that reads another layer's keys
and values has that layer's entry.

Slabs are [B, heads, S, size] or [B, S, size] in the model's dtype, states [B, heads, dim, vdim] in fp32,
rings [B, slots, width] with slot = column % slots.  Rows of
a batch are slots: a slot whose sequence has ended may be given to another one.  Nothing has to be
cleared for that: attention reads no slot in front of the new sequence's first column or behind
its last token, a recurrence starts from zero at a sequence's first column, and no ring slot of a column in
front of it is read.
"""
from __future__ import annotations

import dataclasses

import torch


@dataclasses.dataclass(frozen=True)
class KVSpec:
  """Keys and values of one attention layer run."""
  heads: int
  k_dim: int
  v_dim: int
  dtype: torch.dtype = torch.bfloat16

  def allocate(self, B: int, S: int, device) -> "KVEntry":
    z = lambda d: torch.zeros(B, self.heads, S, d, dtype=self.dtype, device=device)
    return KVEntry(z(self.k_dim), z(self.v_dim))


@dataclasses.dataclass(frozen=True)
class StateSpec:
  """Matrix state of one recurrent layer run (always fp32)."""
  heads: int
  dim: int
  vdim: int

  def allocate(self, B: int, S: int, device) -> "StateEntry":
    return StateEntry(torch.zeros(B, self.heads, self.dim, self.vdim, dtype=torch.float32, device=device))


@dataclasses.dataclass(frozen=True)
class LatentSpec:
  """One row per position of a latent-attention layer run."""
  row: int
  dtype: torch.dtype = torch.bfloat16

  def allocate(self, B: int, S: int, device) -> "LatentEntry":
    return LatentEntry(torch.zeros(B, S, self.row, dtype=self.dtype, device=device))


@dataclasses.dataclass(frozen=True)
class RingSpec:
  """Rows of the last `slots` columns: what a short convolution or a token shift looks back to."""
  slots: int
  width: int
  dtype: torch.dtype = torch.bfloat16

  def allocate(self, B: int, S: int, device) -> "RingEntry":
    return RingEntry(torch.zeros(B, self.slots, self.width, dtype=self.dtype, device=device))


@dataclasses.dataclass(frozen=True)
class PartsSpec:
  """Several things one layer run keeps: ((name, spec), ...)."""
  parts: tuple

  def allocate(self, B: int, S: int, device) -> "PartsEntry":
    return PartsEntry({name: spec.allocate(B, S, device) for name, spec in self.parts})


@dataclasses.dataclass(frozen=True)
class BorrowedSpec:
  """Nothing of its own: the entry of an earlier layer run."""
  run: int


@dataclasses.dataclass
class KVEntry:
  k: torch.Tensor
  v: torch.Tensor

  def rows(self, b0: int, n: int) -> "KVEntry":
    return KVEntry(self.k[b0:b0 + n], self.v[b0:b0 + n])

  def grow(self, S: int):
    for name in ("k", "v"):
      old = getattr(self, name)
      new = torch.zeros(*old.shape[:2], S, old.shape[3], dtype=old.dtype, device=old.device)
      new[:, :, :old.shape[2]].copy_(old)
      setattr(self, name, new)


@dataclasses.dataclass
class StateEntry:
  s: torch.Tensor

  def rows(self, b0: int, n: int) -> "StateEntry":
    return StateEntry(self.s[b0:b0 + n])

  def grow(self, S: int):
    pass   # a state does not depend on the number of columns


@dataclasses.dataclass
class LatentEntry:
  c: torch.Tensor

  def rows(self, b0: int, n: int) -> "LatentEntry":
    return LatentEntry(self.c[b0:b0 + n])

  def grow(self, S: int):
    new = torch.zeros(self.c.shape[0], S, self.c.shape[2], dtype=self.c.dtype, device=self.c.device)
    new[:, :self.c.shape[1]].copy_(self.c)
    self.c = new


@dataclasses.dataclass
class RingEntry:
  r: torch.Tensor

  def rows(self, b0: int, n: int) -> "RingEntry":
    return RingEntry(self.r[b0:b0 + n])

  def grow(self, S: int):
    pass


@dataclasses.dataclass
class PartsEntry:
  parts: dict

  def __getitem__(self, name: str):
    return self.parts[name]

  def rows(self, b0: int, n: int) -> "PartsEntry":
    return PartsEntry({k: e.rows(b0, n) for k, e in self.parts.items()})

  def grow(self, S: int):
    for e in self.parts.values():
      e.grow(S)


class SequenceCache:
  """The entries of one batch.  shared=True: layer runs with equal specs use one buffer (a scratch
  cache for passes that never come back to it), but those whose entry a later run reads."""

  def __init__(self, specs: list, B: int, S: int, device, shared: bool = False):
    self.B, self.S = B, S
    made: dict = {}
    self.entries = []
    lent = {spec.run for spec in specs if isinstance(spec, BorrowedSpec)}
    for i, spec in enumerate(specs):
      if isinstance(spec, BorrowedSpec):
        self.entries.append(self.entries[spec.run])
        continue
      if shared and spec in made and i not in lent:
        self.entries.append(made[spec])
        continue
      entry = spec.allocate(B, S, device)
      if i not in lent:
        made[spec] = entry
      self.entries.append(entry)

  @property
  def kcache(self) -> list:
    return [e.k for e in self.entries if isinstance(e, KVEntry)]

  @property
  def vcache(self) -> list:
    return [e.v for e in self.entries if isinstance(e, KVEntry)]

  def rows(self, b0: int, n: int) -> "SequenceCache":
    """A view of the slots b0 .. b0 + n - 1."""
    view = object.__new__(SequenceCache)
    view.B, view.S = n, self.S
    view.entries = [e.rows(b0, n) for e in self.entries]
    return view

  def grow(self, S: int):
    """More columns, the ones in use kept."""
    if S > self.S:
      for e in {id(e): e for e in self.entries}.values():
        e.grow(S)
      self.S = S
