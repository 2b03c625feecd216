"""Scheduler and sequence-state manager: requests in, greedy tokens out, over any model of the registry.

A model holds cache for a fixed number of sequences, its slots.  `SequenceStates` gives slots to requests and takes them
back; `Engine` admits requests first come first served while slots are free and lets the live ones take turns: a portion of
the prompt, or a burst of decode steps (each burst one run of graph replays, the token and the position stay on the
device)."""
from __future__ import annotations

from collections import deque
from dataclasses import dataclass, field
from typing import Dict, Hashable, Iterable, List, Optional, Sequence

import torch


class SequenceStates:
    """Which sequence holds which slot, and how many of its positions the slot's cache has seen."""

    def __init__(self, slots: int, capacity: int):
        self.capacity = capacity
        self._free = list(range(slots))[::-1]
        self._slot: Dict[Hashable, int] = {}
        self._pos: Dict[Hashable, int] = {}

    def __contains__(self, key) -> bool:
        return key in self._slot

    @property
    def free(self) -> int:
        return len(self._free)

    def open(self, key) -> int:
        if key in self._slot:
            raise ValueError(f"sequence {key!r} is open already")
        if not self._free:
            raise RuntimeError("no free slot")
        self._slot[key], self._pos[key] = self._free.pop(), 0
        return self._slot[key]

    def close(self, key) -> None:
        self._free.append(self._slot.pop(key))
        del self._pos[key]

    def slot(self, key) -> int:
        return self._slot[key]

    def position(self, key) -> int:
        return self._pos[key]

    def advance(self, key, n: int) -> None:
        if self._pos[key] + n > self.capacity:
            raise RuntimeError(f"sequence {key!r} would go beyond its {self.capacity} positions")
        self._pos[key] += n


@dataclass
class Request:
    id: Hashable
    prompt: List[int]
    max_new: int
    stop: frozenset = frozenset()
    tokens: List[int] = field(default_factory=list)     # generated so far
    done: bool = False


class Engine:
    def __init__(self, model, portion: int = 2048, burst: int = 32):
        if portion < 1 or burst < 1:
            raise ValueError("portion and burst must be positive")
        self.model, self.portion, self.burst = model, portion, burst
        self.states = SequenceStates(model.slots, model.capacity)
        self._waiting: deque = deque()
        self._live: deque = deque()

    # ---- one sequence at a time, tokens given by the caller
    def feed(self, key, tokens: Sequence[int], want: Iterable[int] = ()) -> torch.Tensor:
        """Runs the sequence's next tokens and returns the logits at the places `want` among them.  An unknown key opens a
        sequence."""
        new = key not in self.states
        slot = self.states.open(key) if new else self.states.slot(key)
        pos = self.states.position(key)
        try:
            self.states.advance(key, len(tokens))
            return self.model.forward(slot, tokens, pos, list(want))
        except Exception:
            if new:
                self.states.close(key)
            raise

    def finish(self, key) -> None:
        """Gives back what the sequence holds."""
        self.states.close(key)

    # ---- generation
    def add(self, request: Request) -> Request:
        if not request.prompt:
            raise ValueError("a prompt has at least one token")
        if request.max_new < 0:
            raise ValueError("max_new is negative")
        # the last token generated is not run
        if len(request.prompt) + max(request.max_new - 1, 0) > self.model.capacity:
            raise ValueError(f"request {request.id!r} needs more than {self.model.capacity} positions")
        self._waiting.append(request)
        return request

    def step(self) -> Optional[Request]:
        """One turn of one request; None when there is nothing to do."""
        while self._waiting and self.states.free:
            r = self._waiting.popleft()
            self.states.open(r.id)
            self._live.append(r)
        if not self._live:
            return None
        r = self._live.popleft()
        pos = self.states.position(r.id)
        if pos < len(r.prompt):
            part = r.prompt[pos:pos + self.portion]
            whole = pos + len(part) == len(r.prompt)
            logits = self.feed(r.id, part, [len(part) - 1] if whole and r.max_new else [])
            if whole:
                self._take(r, [int(logits[0].argmax())] if r.max_new else [])
        else:
            n = min(self.burst, r.max_new - len(r.tokens))
            slot = self.states.slot(r.id)
            self.states.advance(r.id, n)
            self._take(r, self.model.decode(slot, r.tokens[-1], pos, n))
        if r.done:
            self.finish(r.id)
        else:
            self._live.append(r)
        return r

    def _take(self, r: Request, tokens: List[int]) -> None:
        for t in tokens:
            r.tokens.append(t)
            if t in r.stop:
                r.done = True
                break
        r.done = r.done or len(r.tokens) >= r.max_new

    def run(self) -> None:
        """Turns until every request is done."""
        while self.step() is not None:
            pass

    def generate(self, prompts: Sequence[Sequence[int]], max_new: int, stop: Iterable[int] = ()) -> List[List[int]]:
        """Greedy continuation of every prompt."""
        rs = [self.add(Request(("generate", i), list(p), max_new, frozenset(stop))) for i, p in enumerate(prompts)]
        self.run()
        return [r.tokens for r in rs]
