"""Batches of requests over a model's streams: every live request owns one stream (its cache rows and recurrent state), a step
feeds any number of requests their next tokens as one batch, a finished request gives its stream back.

    sched = Scheduler(model)
    logits = sched.step([("a", prompt_a, [len(prompt_a) - 1]), ("b", prompt_b, [])])
    sched.finish(["a"])

generate() runs a set of prompts to completion: prompts in one ragged step, then one token per live request and step.
"""
from __future__ import annotations

from typing import Dict, Hashable, List, Optional, Sequence, Tuple

import numpy as np

from .model import HipModel


class Scheduler:
    def __init__(self, model: HipModel):
        self.model = model
        self._free = list(range(model.max_streams - 1, -1, -1))
        self._live: Dict[Hashable, List[int]] = {}      # request -> [stream, next position]

    def live(self) -> List[Hashable]:
        return list(self._live)

    def position(self, request: Hashable) -> int:
        return self._live[request][1]

    def step(self, entries: Sequence[Tuple[Hashable, Sequence[int], Sequence[int]]]) -> List[np.ndarray]:
        """entries: (request, its next tokens, places among them whose logits are wanted).  A request that is not live starts.
        Returns [wanted, vocab] per entry."""
        names = [e[0] for e in entries]
        if len(set(names)) != len(names):
            raise ValueError("a request appears twice in one step")
        new = [r for r in names if r not in self._live]
        if len(new) > len(self._free):
            raise RuntimeError(f"{len(new)} new requests, {len(self._free)} of {self.model.max_streams} streams are free")
        batch = []
        for r, tokens, want in entries:
            if not len(tokens):
                raise ValueError(f"request {r!r} brings no tokens")
            if r not in self._live:
                self._live[r] = [self._free.pop(), 0]
                self.model.reset(self._live[r][0])
            stream, pos = self._live[r]
            batch.append((stream, tokens, pos, want))
        out = self.model.step(batch)
        for r, tokens, _ in entries:
            self._live[r][1] += len(tokens)
        return out

    def finish(self, requests: Sequence[Hashable]) -> None:
        for r in requests:
            stream, _ = self._live.pop(r)
            self.model.reset(stream)
            self._free.append(stream)

    def generate(self, prompts: Sequence[Sequence[int]], max_tokens: int, eos_id: int = -1, sampler=None) -> List[List[int]]:
        """Continues every prompt by up to max_tokens ids (the EOS included).  sampler(logits) -> id; default: argmax."""
        pick = sampler or (lambda row: int(np.argmax(row)))
        out: List[List[int]] = [[] for _ in prompts]
        waiting, active = list(range(len(prompts)))[::-1], []
        tag = object()
        while waiting or active:
            step: List[Tuple[int, List[int], List[int]]] = [(i, [out[i][-1]], [0]) for i in active]
            if step:
                rows = self.step([((tag, i), t, w) for i, t, w in step])
            else:
                while waiting and len(step) < len(self._free):
                    i = waiting.pop()
                    step.append((i, list(prompts[i]), [len(prompts[i]) - 1]))
                if not step:
                    raise RuntimeError("no free stream")
                rows = self.step([((tag, i), t, w) for i, t, w in step])
            active = []
            for (i, _, _), row in zip(step, rows):
                out[i].append(pick(row[-1]))
                if len(out[i]) >= max_tokens or out[i][-1] == eos_id or self.position((tag, i)) >= self.model.config.seq_len:
                    self.finish([(tag, i)])
                else:
                    active.append(i)
        return out
