"""Decoders without a grammar: free generation and sequences fed from outside.

A decoder tells the engine what a request samples from and when it is done
(``planner.grammar`` has the constrained ones).  The two flags the engine reads
here are ``dense`` (the allowed set is the whole vocabulary: the step computes
full logits) and ``samples`` (False: the request never samples, its tokens come
from ``LLMEngine.feed``).
"""
from __future__ import annotations

from typing import List, Optional, Sequence


class TokenDecoder:
    """Up to ``max_new`` tokens from the whole vocabulary, ending early at
    ``eos``; ``result()`` is the list of sampled ids."""

    dense = True

    def __init__(self, max_new: int, eos: Optional[int] = None):
        self.max_new, self.eos = int(max_new), eos
        self.out: List[int] = []
        self._new: List[int] = []
        self.done = self.max_new <= 0

    def advance(self) -> List[int]:
        new, self._new = self._new, []
        return [] if self.done else new

    def allowed(self) -> Sequence[int]:
        return (-1,)                       # the whole vocabulary (ops.sample_dense)

    def feed(self, token: int) -> None:
        self.out.append(token)
        self.done = len(self.out) >= self.max_new or token == self.eos
        self._new = [token]

    def result(self) -> List[int]:
        return self.out


class FedDecoder:
    """A request whose tokens are given (``LLMEngine.feed``): never samples,
    stays admitted until ``LLMEngine.close``."""

    samples = False
    done = False

    def advance(self) -> List[int]:
        return []

    def allowed(self) -> Sequence[int]:
        return ()

    def result(self):
        return None
