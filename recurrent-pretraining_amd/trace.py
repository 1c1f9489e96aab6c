"""Replays a trace of given tokens through a model: steps come as JSON lines, each bringing the next tokens of one or more
requests, and the logits at the asked-for places are written out.  Nothing is sampled.

The model is loaded as always (registry.load_model), every request has a cache from RequestCaches, portions of several tokens
go through forward() and single tokens through the decode runner (its graph included), as in generation."""

from __future__ import annotations

import json
import os
from typing import Iterable, List, Optional, TextIO

import torch

from .cache import RequestCaches


class TraceReplay:
    def __init__(self, model, max_tokens: Optional[int] = None):
        self.model = model
        self.max_tokens = max_tokens
        self.caches = RequestCaches(lambda: model.new_cache(max_tokens))
        self._runners: dict = {}  # id(cache) -> decode runner: a cache that is used again keeps its captured step

    def feed(self, request, tokens: List[int], want: List[int]) -> torch.Tensor:
        """The next tokens of a request; returns the logits [len(want), vocab] at the places `want` among them."""
        cache = self.caches.get(request)
        if len(tokens) == 1:
            if id(cache) not in self._runners:
                self._runners[id(cache)] = self.model.decode_runner(cache, 1, None, greedy=True, use_graph=True)
            logits, _, _ = self._runners[id(cache)].step(torch.tensor(tokens, device=self.model.device), None, 0.0)
            return logits[[0] * len(want)]
        out = self.model.forward(torch.tensor([tokens], device=self.model.device), past_key_values=cache, use_cache=True, init_scale=0.0,
                                 logit_positions=want)
        rows = out.logits[0]
        return rows if rows.shape[0] == len(want) else rows[want]  # a family that returns every position's logits

    def end(self, request) -> None:
        self.caches.release(request)

    def step(self, entries: Iterable[dict], end: Iterable) -> Optional[torch.Tensor]:
        """One step of a trace; the wanted logits of all entries in order ([n, vocab] float on the CPU), or None."""
        rows = [self.feed(e["id"], e["tokens"], e["want"]) for e in entries]
        rows = [r for r in rows if r.shape[0]]
        out = torch.cat(rows).float().cpu() if rows else None
        for request in end:
            self.end(request)
        return out


def replay(model, lines: TextIO, out_dir: str, done: TextIO, max_tokens: Optional[int] = None) -> None:
    """Runs the steps on `lines`; step n's logits go to <out_dir>/<n>.f32 (little-endian), its "done n" to `done`."""
    trace = TraceReplay(model, max_tokens)
    for line in lines:
        if not line.strip():
            continue
        step = json.loads(line)
        logits = trace.step(step["entries"], step.get("end", []))
        if logits is not None:
            path = os.path.join(out_dir, f"{step['step']}.f32")
            logits.contiguous().numpy().astype("<f4", copy=False).tofile(path)
        else:
            torch.cuda.synchronize()
        print(f"done {step['step']}", file=done, flush=True)
