"""Requests over one driver: pages, recurrent-state slots and batch construction.

Plays the part of the serving runtime above the driver boundary: it owns which physical pages and
which state slot a request holds, gives them back when the request ends, and turns one step's
entries (prompt portions beside single decoded tokens) into one forward request.  The cache, the
state and the arithmetic are the driver's.
"""
from __future__ import annotations

from dataclasses import dataclass, field
from typing import Hashable, List, Optional, Sequence, Tuple

import numpy as np

from . import driver as drv

SAMPLER_RAW_LOGITS = 7
GREEDY = dict(kind=drv.SAMPLER_TOP_P, temperature=0.0, p=1.0)


class OutOfPages(RuntimeError):
    pass


@dataclass
class Request:
    pages: List[int] = field(default_factory=list)
    slot: Optional[int] = None
    length: int = 0    # tokens in the cache


class Engine:
    def __init__(self, driver: drv.Driver):
        self.driver = driver
        caps = driver.capabilities()
        self.page_size = caps["kv_page_size"]
        self.max_tokens = caps["max_forward_tokens"]
        # handed out lowest first, taken back last in first out
        self._free_pages = list(range(caps["total_pages"]))[::-1]
        self._free_slots = list(range(caps["rs_cache_slots"]))[::-1]
        self._recurrent = bool(caps["rs_cache_required"])
        self.requests: dict = {}

    def _admit(self, rid: Hashable) -> Request:
        req = Request()
        if self._recurrent:
            if not self._free_slots:
                raise OutOfPages("no recurrent-state slot is free")
            req.slot = self._free_slots.pop()
        self.requests[rid] = req
        return req

    def finish(self, rid: Hashable) -> None:
        """Gives back what the request holds."""
        req = self.requests.pop(rid)
        self._free_pages.extend(reversed(req.pages))
        if req.slot is not None:
            self._free_slots.append(req.slot)

    def _forward(self, entries, samplers_of) -> drv.ForwardResult:
        tokens, positions, pages, page_indptr, last = [], [], [], [0], []
        qo, samp, samp_indptr, samplers, slots = [0], [], [0], [], []
        for rid, toks, want in entries:
            req = self.requests.get(rid) or self._admit(rid)
            end = req.length + len(toks)
            need = -(-end // self.page_size) - len(req.pages)
            if need > len(self._free_pages):
                raise OutOfPages(f"request {rid!r} needs {need} more pages, {len(self._free_pages)} are free")
            req.pages.extend(self._free_pages.pop() for _ in range(need))
            tokens.extend(toks)
            positions.extend(range(req.length, end))
            used = -(-end // self.page_size)
            pages.extend(req.pages[:used])
            page_indptr.append(len(pages))
            last.append(end - (used - 1) * self.page_size)
            qo.append(len(tokens))
            samp.extend(want)
            samp_indptr.append(len(samp))
            samplers.extend(samplers_of(rid, want))
            slots.append(req.slot)
        frame = drv.ForwardFrame(tokens, positions, pages, page_indptr, last, qo, sampling_indices=samp,
                                 sampling_indptr=samp_indptr, samplers=samplers, sampler_indptr=samp_indptr,
                                 rs_slot_ids=slots if self._recurrent else None)
        res = self.driver.forward(frame)
        if res.num_requests != len(entries):
            raise RuntimeError("forward failed: " + self.driver.last_error())
        for (rid, toks, _), start in zip(entries, qo):
            self.requests[rid].length += len(toks)
        return res

    def step(self, entries: Sequence[Tuple[Hashable, Sequence[int], Sequence[int]]]) -> List[np.ndarray]:
        """One batch of (request, its next tokens, places among them); returns per entry the fp32
        logits [places, vocab].  A request is admitted at its first entry."""
        res = self._forward(entries, lambda rid, want: [dict(kind=SAMPLER_RAW_LOGITS)] * len(want))
        return [np.stack(res.logits_of(r)) if want else np.zeros((0, 0), np.float32)
                for r, (_, _, want) in enumerate(entries)]

    def step_sampled(self, entries, sampler: dict = GREEDY) -> List[int]:
        """One batch of (request, its next tokens); the token sampled after each entry's last one."""
        full = [(rid, toks, [len(toks) - 1]) for rid, toks in entries]
        res = self._forward(full, lambda rid, want: [sampler])
        return [int(res.tokens_of(r)[0]) for r in range(len(full))]

    def generate(self, prompts: dict, max_new: int, portion: Optional[int] = None, sampler: dict = GREEDY) -> dict:
        """Continuous batching: every step runs one portion of each prompt still being read beside
        one decoded token of each other request.  {request: prompt} -> {request: tokens}."""
        left = {rid: list(p) for rid, p in prompts.items()}
        out = {rid: [] for rid in prompts}
        while any(len(o) < max_new for o in out.values()):
            entries, budget = [], self.max_tokens
            live = [rid for rid in prompts if len(out[rid]) < max_new]
            for rid in sorted(live, key=lambda r: bool(left[r])):   # decoded tokens first
                n = min(len(left[rid]) or 1, budget, portion or self.max_tokens)
                if n <= 0:
                    continue
                entries.append((rid, left[rid][:n] if left[rid] else [out[rid][-1]]))
                budget -= n
            toks = self.step_sampled(entries, sampler)
            for (rid, part), tok in zip(entries, toks):
                if left[rid]:
                    left[rid] = left[rid][len(part):]
                    if left[rid]:
                        continue
                out[rid].append(tok)
                if len(out[rid]) == max_new:
                    self.finish(rid)
        return out
