"""Requests on top of MaxEngine.step: slots for live requests, prompts in portions beside decoded tokens, one batch per step.

The reference leaves this to its serving glue (jetstream's orchestrator around maxengine.py:533-936); here it is a small class so that a mixed
batch -- portions of some prompts beside single tokens of running sequences -- reaches the engine as ONE pass over the weights."""
from __future__ import annotations

from typing import Any, Dict, Hashable, Iterable, List, Sequence, Tuple

import torch


class StepScheduler:
  """Maps request ids to decode slots.  A request is admitted by its first tokens and keeps its slot until `release`."""

  def __init__(self, engine: Any):
    self.engine = engine
    self._free: List[int] = list(range(engine.max_concurrent_decodes))[::-1]
    self._slot: Dict[Hashable, int] = {}
    self._length: Dict[Hashable, int] = {}

  @property
  def live(self) -> List[Hashable]:
    return list(self._slot)

  def length(self, request: Hashable) -> int:
    return self._length.get(request, 0)

  def step(self, entries: Iterable[Tuple[Hashable, Sequence[int], Sequence[int]]], want_logits: bool = True):
    """entries: (request id, its next tokens, the places among them whose logits are wanted).  All of them run as one batch from where each request
    stands.  -> (logits f32 [wanted, vocab] or None, their greedy tokens int32 [wanted]), in the order of the entries and their places."""
    batch, seen = [], set()
    for request, tokens, want in entries:
      tokens = list(tokens)
      if request in seen:
        raise ValueError(f"request {request!r} has two entries in one step")
      seen.add(request)
      if not tokens:
        raise ValueError(f"request {request!r} brings no tokens")
      if request not in self._slot:
        if not self._free:
          raise ValueError(f"no free slot for request {request!r} ({len(self._slot)} live)")
        self._slot[request], self._length[request] = self._free.pop(), 0
      batch.append((self._slot[request], self._length[request], tokens, list(want)))
      self._length[request] += len(tokens)
    return self.engine.step(batch, want_logits=want_logits)

  def release(self, request: Hashable) -> None:
    """The request is finished: its pages go back to the pool, its slot can be taken again."""
    if request not in self._slot:
      raise ValueError(f"request {request!r} is not live")
    slot = self._slot.pop(request)
    del self._length[request]
    self.engine.release_pages(slot)
    self._free.append(slot)

  def generate(self, prompts: Dict[Hashable, Sequence[int]], max_new_tokens: int, portion: int = 0) -> Dict[Hashable, List[int]]:
    """Greedy generation for any number of prompts: as many run at a time as there are slots, a prompt's portions (`portion` tokens; 0: whole prompts)
    beside the decoded tokens of the others."""
    waiting = [(r, list(p)) for r, p in prompts.items()]
    out: Dict[Hashable, List[int]] = {r: [] for r, _ in waiting}
    rest: Dict[Hashable, List[int]] = {}
    while waiting or rest:
      while waiting and len(rest) < self.engine.max_concurrent_decodes:
        r, p = waiting.pop(0)
        rest[r] = p
      entries = []
      for r, todo in rest.items():
        now = todo[:portion] if portion > 0 else todo
        entries.append((r, now, [len(now) - 1] if len(now) == len(todo) else []))
      _, tokens = self.step(entries, want_logits=False)
      tokens = tokens.cpu().tolist() if isinstance(tokens, torch.Tensor) else list(tokens)
      for r, now, want in entries:
        rest[r] = rest[r][len(now):]
        if want:
          out[r].append(int(tokens.pop(0)))
          rest[r] = [out[r][-1]]
          if len(out[r]) >= max_new_tokens:
            del rest[r]
            self.release(r)
    return out
