"""Requests on the slots of a decoder-only model's cache: who holds which slot, how
far each request has come, and steps that feed several requests their next
tokens at once.

`Sequences` is what serves requests that arrive token by token or portion by
portion (bin/trace_run); models.DecoderOnlyModel drives whole batches over the
same step function.
"""

from typing import Any, Iterable, Optional, Sequence, Tuple


class Sequences:
  """Live requests of a module (hybrid.HybridDecoder) over `slots` slots of up to
  `max_len` positions each.  A request takes a slot with its first tokens and
  gives it back when it ends; a slot needs no clearing in between."""

  def __init__(self, module, params, slots: int, max_len: int):
    self.module, self.params, self.max_len = module, params, int(max_len)
    self.cache = module.init_cache(int(slots), self.max_len)
    self._free = list(range(int(slots)))[::-1]
    self._live = {}  # request -> [slot, positions held]

  def __len__(self):
    return len(self._live)

  def length(self, request) -> int:
    """Positions the request holds (0 before its first tokens)."""
    return self._live[request][1] if request in self._live else 0

  def step(self, entries: Iterable[Tuple[Any, Sequence[int], Sequence[int]]],
           trace: Optional[list] = None):
    """entries: (request, its next tokens, places among them whose logits are
    wanted), one per request.  Returns the wanted logits [n, vocab] in the order
    of the entries and places, or None."""
    entries = [(r, list(t), list(w)) for r, t, w in entries]
    names = [r for r, _, _ in entries]
    if len(set(names)) != len(names):
      raise ValueError('a request appears twice in one step')
    for request, tokens, want in entries:
      if any(not 0 <= k < len(tokens) for k in want):
        raise ValueError(f'request {request!r}: wanted places {want} of '
                         f'{len(tokens)} tokens')
      if self.length(request) + len(tokens) > self.max_len:
        raise ValueError(f'request {request!r} grows beyond {self.max_len} '
                         'positions')
    new = [r for r, t, _ in entries if t and r not in self._live]
    if len(new) > len(self._free):
      raise RuntimeError(f'{len(new)} new requests and {len(self._free)} free '
                         'slots')
    for request in new:
      self._live[request] = [self._free.pop(), 0]
    portions, wanted = [], []
    for request, tokens, want in entries:
      if tokens:
        slot, held = self._live[request]
        portions.append((slot, held, tokens))
        wanted.append(want)
    logits = None
    if portions:
      logits = self.module.advance(self.params, self.cache, portions, wanted,
                                   trace)
    for request, tokens, _ in entries:
      if tokens:
        self._live[request][1] += len(tokens)
    return logits

  def end(self, request):
    """The request is finished; its slot is free."""
    slot = self._live.pop(request, None)
    if slot is not None:
      self._free.append(slot[0])
