"""What a decoder keeps of the tokens it has seen, for a batch of sequences that advance together.

``StepCache`` is the part every model's cache shares: a capacity, the number of tokens held
(a host integer that the driver of the steps moves on, since a replayed HIP graph runs no
Python), and giving it all back. ``MixerCache`` holds whatever the layers of a model with
different sequence mixers declare: rows per position, recurrent states, rings. ``RequestCaches`` lends
caches to requests and takes them back.
"""

from __future__ import annotations

from typing import Callable, Dict, List

import torch
from torch import Tensor


class StepCache:
    def __init__(self, batch: int, max_len: int, device):
        self.batch, self.max_len, self.device = batch, max_len, torch.device(device)
        self.tokens = 0

    def next_positions(self, n: int) -> Tensor:
        """Positions of the next ``n`` tokens, ``[n]`` int64 on the device."""
        if n < 1 or self.tokens + n > self.max_len:
            raise ValueError(f"{n} tokens after {self.tokens} do not fit a cache of {self.max_len}")
        return torch.arange(self.tokens, self.tokens + n, device=self.device)

    def advance(self, n: int) -> None:
        """``n`` more tokens have been run through the model with this cache."""
        self.tokens += n

    def reset(self) -> None:
        """Forget everything: the next token is at position 0."""
        self.tokens = 0


class MixerCache(StepCache):
    """Per layer, what its mixer carries from token to token. ``slot`` is the layer's number, or (layer, pass)
    where layers run several times: every pass keeps its own.

      ``rows[slot]``   ``[batch, max_len, cols]`` in the model's dtype, one row per position: latents, keys
                       and values (rows at or past ``tokens`` are never read, so they need no clearing);
      ``state[slot]``  fp32 ``[batch, ...]``, zero before the first token;
      ``ring[slot]``   ``[batch, n, cols]`` in the model's dtype, the last inputs of a short convolution, the
                       one of position p in row p mod n (positions below 0 are not read: no clearing).

    ``rotary[key]`` are the rotary tables of the layers' rotations, ``[max_len, pairs, 2]``, one per
    distinct rotation.
    """

    def __init__(self, batch: int, max_len: int, device, dtype):
        super().__init__(batch, max_len, device)
        self.dtype = dtype
        self.rows: Dict[object, Tensor] = {}
        self.state: Dict[object, Tensor] = {}
        self.ring: Dict[object, Tensor] = {}
        self.rotary: Dict[object, Tensor] = {}

    def add_rows(self, slot, cols: int) -> None:
        self.rows[slot] = torch.zeros((self.batch, self.max_len, cols), device=self.device, dtype=self.dtype)

    def add_state(self, slot, *shape: int) -> None:
        self.state[slot] = torch.zeros((self.batch, *shape), device=self.device, dtype=torch.float32)

    def add_ring(self, slot, n: int, cols: int) -> None:
        self.ring[slot] = torch.zeros((self.batch, n, cols), device=self.device, dtype=self.dtype)

    def add_rotary(self, key, build: Callable[..., Tensor]) -> None:
        if key not in self.rotary:
            self.rotary[key] = build(self.max_len, self.device)

    def reset(self) -> None:
        super().reset()
        for s in self.state.values():
            s.zero_()


class RequestCaches:
    """One cache per live request, made by ``new_cache()`` on first use; ``end`` takes a request's
    cache back for the next request."""

    def __init__(self, new_cache: Callable[[], StepCache]):
        self._new_cache = new_cache
        self._live: Dict[object, StepCache] = {}
        self._free: List[StepCache] = []

    def of(self, request) -> StepCache:
        cache = self._live.get(request)
        if cache is None:
            cache = self._free.pop() if self._free else self._new_cache()
            self._live[request] = cache
        return cache

    def end(self, request) -> None:
        cache = self._live.pop(request, None)
        if cache is not None:
            cache.reset()
            self._free.append(cache)
