"""Serves requests over one model: admission, prompt portions, token-by-token decoding, sampling.

A step of the model runs one sequence, so the scheduler interleaves: requests are admitted first come,
first served while the state pool has slots; every tick either runs one portion of the oldest unfinished
prompt or, every other tick, one token of each running sequence, so that long prompts do not stall those.
"""
from __future__ import annotations

import itertools
from collections import deque
from dataclasses import dataclass, field
from typing import Optional, Sequence

from . import sampling


def _scatter(seed: int, index: int) -> int:
    """The index-th output of the splitmix64 generator started at `seed`, as a positive 63-bit integer."""
    mask = (1 << 64) - 1
    z = (seed + (index + 1) * 0x9E3779B97F4A7C15) & mask
    z = ((z ^ (z >> 30)) * 0xBF58476D1CE4E5B9) & mask
    z = ((z ^ (z >> 27)) * 0x94D049BB133111EB) & mask
    return ((z ^ (z >> 31)) >> 1) or 1


@dataclass
class Request:
    id: int
    prompt: list[int]
    max_new_tokens: int
    params: sampling.Params
    stop_tokens: frozenset
    tokens: list[int] = field(default_factory=list)  # generated so far
    finished: bool = False
    # scheduler state
    sequence: object = None
    prompt_done: int = 0


class Engine:
    def __init__(self, model, portion: int = 2048):
        if portion < 1:
            raise ValueError("a prompt portion has at least one token")
        self.model, self.portion = model, portion
        self._ids = itertools.count()
        self._waiting: deque[Request] = deque()
        self._active: list[Request] = []
        self._decode_turn = False

    def submit(self, prompt: Sequence[int], max_new_tokens: int = 16, params: Optional[sampling.Params] = None,
               stop_tokens: Sequence[int] = ()) -> Request:
        prompt = [int(token) for token in prompt]
        if not prompt:
            raise ValueError("a prompt has at least one token")
        if any(not 0 <= token < self.model.vocabulary for token in prompt):
            raise ValueError("a prompt token is outside the vocabulary")
        if max_new_tokens < 1:
            raise ValueError("a request generates at least one token")
        request = Request(next(self._ids), prompt, max_new_tokens, params or sampling.Params.greedy(),
                          frozenset(stop_tokens))
        self._waiting.append(request)
        return request

    @property
    def busy(self) -> bool:
        return bool(self._waiting or self._active)

    def tick(self) -> None:
        """One scheduling decision and its model steps."""
        while self._waiting and self.model.state.free_slots:
            request = self._waiting.popleft()
            request.sequence = self.model.open()
            self._active.append(request)
        prompts = [r for r in self._active if r.prompt_done < len(r.prompt)]
        running = [r for r in self._active if r.prompt_done == len(r.prompt)]
        self._decode_turn = bool(running) and (not prompts or not self._decode_turn)
        try:
            if self._decode_turn:
                for request in running:
                    self._decode(request)
            elif prompts:
                self._prefill(prompts[0])
        except Exception:
            self._abandon()
            raise
        for request in [r for r in self._active if r.finished]:
            self._active.remove(request)
            self.model.close(request.sequence)

    def run(self) -> None:
        while self.busy:
            self.tick()

    def _prefill(self, request: Request) -> None:
        # a rest of one token would cost a step of its own
        left = len(request.prompt) - request.prompt_done
        count = left if left <= self.portion + 1 else self.portion
        part = request.prompt[request.prompt_done:request.prompt_done + count]
        last = count == left
        logits = self.model.step(request.sequence, part, [count - 1] if last else [])
        request.prompt_done += count
        if last:
            self._accept(request, sampling.sample_f32(self._step_params(request), logits[0]))

    def _decode(self, request: Request) -> None:
        token = self.model.decode(request.sequence, request.tokens[-1])
        if not request.params.is_greedy():
            token = sampling.sample_f32(self._step_params(request), self.model.logits_row())
        self._accept(request, token)

    @staticmethod
    def _step_params(request: Request) -> sampling.Params:
        """A seed gives one sequence of draws: every token a seed of its own, scattered (the sampler's
        generator gives neighbouring seeds neighbouring first draws); 0 stays 0, the clock."""
        p = request.params
        seed = _scatter(p.seed, len(request.tokens)) if p.seed else 0
        return sampling.Params(p.temperature, p.top_k, p.top_p, p.min_p, seed)

    @staticmethod
    def _accept(request: Request, token: int) -> None:
        request.tokens.append(token)
        request.finished = len(request.tokens) >= request.max_new_tokens or token in request.stop_tokens

    def _abandon(self) -> None:
        """A model step failed: nothing live can be trusted to be where its request thinks it is."""
        for request in self._active:
            request.finished = True
            self.model.close(request.sequence)
        self._active.clear()

    def generate(self, prompts: Sequence[Sequence[int]], max_new_tokens: int = 16,
                 params: Optional[sampling.Params] = None, stop_tokens: Sequence[int] = ()) -> list[list[int]]:
        requests = [self.submit(p, max_new_tokens, params, stop_tokens) for p in prompts]
        self.run()
        return [r.tokens for r in requests]
