"""Replays recorded token streams through a model, step by step, and hands back logits: the
sampler's prompt and decode passes with the tokens given instead of sampled.

A step is {"entries": [{"id", "tokens", "want"}], "end": [ids]}.  The entries of a step are one batch:
new requests, each with its whole first portion (left-padded to one width, as the sampler pads
prompts), or the requests of a running batch, one token each.  Requests of `end` give their slot
back; a batch whose requests have all ended frees its cache.
"""
from __future__ import annotations

import numpy as np
import torch

from . import utils
from .sampler import CacheConfig, Sampler, _SamplingState

PAD_ID = -1          # no token: every id of the vocabulary may occur in a recorded stream
HEAD_ROWS = 256      # rows of one head call


class _Batch:
  def __init__(self, ids: list[str], st: _SamplingState):
    self.rows = {r: i for i, r in enumerate(ids)}     # live request -> slot
    self.st = st
    self.column = st.num_input_tokens                 # column of the next token
    self.first = st.starts.tolist()                   # column of each row's first token
    self.runner = None


class Replay:
  def __init__(self, model):
    self.model = model
    self.sampler = Sampler(model, utils.IdTokenizer(model.cfg.vocab_size, pad_id=PAD_ID), CacheConfig(0))
    self.batches: list[_Batch] = []

  def _logits(self, runner, hidden: torch.Tensor) -> np.ndarray:
    """Logits of the given final hidden rows."""
    V = self.model.cfg.vocab_size
    n = hidden.shape[0]
    out = torch.empty(n, V, dtype=torch.float32, device=self.model.device)
    keep = runner.part
    runner.part = torch.empty(min(n, HEAD_ROWS) * runner.nvb * 4, dtype=torch.float32, device=self.model.device)
    for r0 in range(0, n, HEAD_ROWS):
      rows = hidden[r0:r0 + HEAD_ROWS].contiguous()
      runner.run_head(rows, rows.shape[0], logits_out=out[r0:r0 + HEAD_ROWS])
    res = out.cpu().numpy()
    runner.part = keep
    return res

  def _check(self, entries: list[dict]):
    V = self.model.cfg.vocab_size
    for e in entries:
      if not e["tokens"]:
        raise ValueError(f"request {e['id']} brings no token")
      if min(e["tokens"]) < 0 or max(e["tokens"]) >= V:
        raise ValueError(f"request {e['id']} has a token outside the vocabulary of {V}")
      if any(not 0 <= w < len(e["tokens"]) for w in e["want"]):
        raise ValueError(f"request {e['id']} wants a place it has no token for")

  def _start(self, entries: list[dict]) -> list[np.ndarray]:
    lengths = [len(e["tokens"]) for e in entries]
    P = max(lengths)
    utils.check_positions(self.model, P)
    ids = np.array([utils.pad_to_length(np.asarray(e["tokens"], dtype=np.int32), P, PAD_ID, left=True) for e in entries])
    S = utils.next_power_of_2(P + 64)
    st = _SamplingState(self.model, ids, S, S, PAD_ID, False, False, lengths=lengths)
    batch = _Batch([e["id"] for e in entries], st)
    out: list = [None] * len(entries)

    def on_rows(b0, nb, runner, xn):
      for i in range(b0, b0 + nb):
        if entries[i]["want"]:
          first = (i - b0) * P + P - lengths[i]
          at = torch.tensor([first + w for w in entries[i]["want"]], device=self.model.device)
          out[i] = self._logits(runner, xn.index_select(0, at))

    self.sampler.forward_prompt(st, on_rows)
    self.batches.append(batch)
    return [o for o in out if o is not None]

  def _advance(self, batch: _Batch, entries: list[dict]) -> list[np.ndarray]:
    if set(batch.rows) != {e["id"] for e in entries} or any(len(e["tokens"]) != 1 for e in entries):
      raise ValueError("the requests of a running batch go on together, one token each")
    st, model = batch.st, self.model
    B, S = st.token_buffer.shape
    for e in entries:
      utils.check_positions(model, batch.column + 1 - batch.first[batch.rows[e["id"]]])
    if batch.column >= S:
      S *= 2
      st.cache.grow(S)
      grown = torch.full((B, S), PAD_ID, dtype=torch.int32, device=model.device)
      grown[:, :st.token_buffer.shape[1]] = st.token_buffer
      st.token_buffer = grown
      st.positions = torch.cat([st.positions, torch.zeros_like(st.positions)], dim=1)   # (read by token-masked models)
      st.positions[:, S // 2:] = st.positions[:, S // 2 - 1:S // 2] + torch.arange(1, S // 2 + 1, device=model.device, dtype=torch.int32)
      batch.runner = None
    if batch.runner is None:
      batch.runner = model.new_runner(B, 1, S, PAD_ID)
    column = np.full(B, PAD_ID, dtype=np.int32)
    for e in entries:
      column[batch.rows[e["id"]]] = e["tokens"][0]
    st.token_buffer[:, batch.column] = torch.from_numpy(column).to(model.device)
    st.step.fill_(batch.column)
    xn = self.sampler.forward_step(batch.runner, st)
    batch.column += 1
    want = [batch.rows[e["id"]] for e in entries for _ in e["want"]]
    if not want:
      return []
    return [self._logits(batch.runner, xn.index_select(0, torch.tensor(want, device=model.device)))]

  def step(self, step: dict) -> np.ndarray | None:
    """Runs one step; the wanted logits [n, vocab] in the order of the entries and their places."""
    entries = step["entries"]
    self._check(entries)
    live = {r: b for b in self.batches for r in b.rows}
    parts: list[np.ndarray] = []
    fresh = [e for e in entries if e["id"] not in live]
    if fresh and len(fresh) != len(entries):
      raise ValueError("a step either starts requests or continues running ones")
    if fresh:
      parts = self._start(fresh)
    elif entries:
      owners = {id(live[e["id"]]) for e in entries}
      if len(owners) != 1:
        raise ValueError("the entries of a step belong to one batch")
      parts = self._advance(live[entries[0]["id"]], entries)
    for r in step.get("end", []):
      for b in self.batches:
        b.rows.pop(r, None)
    self.batches = [b for b in self.batches if b.rows]
    return np.concatenate(parts) if parts else None
