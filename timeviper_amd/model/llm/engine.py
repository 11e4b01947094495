"""Text requests on a causal LM: steps over a changing set of requests, and a greedy scheduler on top of them.

`TextEngine.step` takes the next tokens of any of the live requests (a new name starts a request) and returns the logits
at the places asked for; `end` gives a request's state back.  Models with `supports_ragged` run a step's requests as one
packed batch on a `SlotStateCache`; the others keep a cache per request and run one after the other.

`generate` admits prompts as others finish, up to `max_batch` at a time.  While the set of running requests does not
change, the single-token step is captured once and replayed as one hipGraph launch (decode_graph.py)."""
from __future__ import annotations

import os
from collections import deque
from typing import Dict, Hashable, List, Optional, Sequence, Tuple

import torch

from .decode_graph import GraphedDecodeStep

Entry = Tuple[Hashable, Sequence[int], Sequence[int]]       # request, its next tokens, places among them whose logits are asked for


class TextEngine:
    def __init__(self, llm, max_tokens: Optional[int] = None, slots: int = 1):
        self.llm, self.device = llm, llm.device
        self.ragged = bool(getattr(llm, "supports_ragged", False))
        self._live: Dict[Hashable, object] = {}             # request -> slot, or (cache, tokens seen) of its own
        self.cache, self.limit = None, None                 # limit: the most tokens of one request
        if self.ragged:
            self.cache = llm.new_cache(0)
            self.limit = self.cache.limit
            # (max_tokens bounds the longest request as well; buffers grow when a step needs more)
            self.cache._resize(slots, min(int(max_tokens or 0), 4096, self.limit or 4096))

    def _check(self, tokens):
        if not len(tokens) or min(tokens) < 0 or max(tokens) >= self.llm.config.vocab_size:
            raise ValueError("a request's tokens: at least one, each within the vocabulary")

    @torch.inference_mode()
    def step(self, entries: Sequence[Entry]) -> torch.Tensor:
        """fp32 logits (wanted places, vocab), in the order of the entries and of their places."""
        if not entries:
            return torch.empty((0, self.llm.config.vocab_size), device=self.device)
        for rid, tokens, want in entries:
            self._check(tokens)
            if self.limit is not None and (self.cache.length(self._live[rid]) if rid in self._live else 0) + len(tokens) > self.limit:
                raise ValueError(f"request {rid!r}: this model takes at most {self.limit} tokens a request")
            if any(not 0 <= w < len(tokens) for w in want):
                raise ValueError("a wanted place lies outside the step's tokens")
        return self._step_packed(entries) if self.ragged else self._step_each(entries)

    def _step_packed(self, entries):
        slots, counts, ids, at = [], [], [], []
        for rid, tokens, want in entries:
            if rid not in self._live:
                self._live[rid] = self.cache.alloc()
            slots.append(self._live[rid])
            counts.append(len(tokens))
            at += [len(ids) + w for w in want]
            ids += list(tokens)
        plan = self.cache.plan(slots, counts)
        i64 = lambda v: torch.tensor(v, dtype=torch.int64).to(self.device)
        return self.llm.step(i64(ids), self.cache, plan, logits_at=i64(at))

    def _step_each(self, entries):
        out = []
        for rid, tokens, want in entries:
            cache, seen = self._live.get(rid) or (self.llm.new_cache(1), 0)
            pos = torch.arange(seen, seen + len(tokens))
            r = self.llm(input_ids=torch.tensor([list(tokens)], device=self.device), past_key_values=cache, use_cache=True,
                         cache_position=pos, position_ids=pos[None].to(self.device), logits_to_keep=0)
            self._live[rid] = (cache, seen + len(tokens))
            out.append(r.logits[0].float()[list(want)])
        return torch.cat(out)

    def end(self, rid):
        """The request is finished: its slot (or cache) is given back."""
        if rid in self._live:
            held = self._live.pop(rid)
            if self.ragged:
                self.cache.free(held)

    # ------------------------------------------------------------------ greedy generation
    @torch.inference_mode()
    def generate(self, prompts: Sequence[Sequence[int]], max_new_tokens: int = 128, eos_token_id=(), max_batch: int = 16) -> List[List[int]]:
        eos = {int(e) for e in (eos_token_id if isinstance(eos_token_id, (list, tuple, set)) else [eos_token_id])}
        waiting = deque(enumerate(prompts))
        out: List[List[int]] = [[] for _ in prompts]
        running: List[int] = []

        def most(i):                                         # new tokens request i may get: one behind its last place is never fed back
            return max_new_tokens if self.limit is None else min(max_new_tokens, self.limit - len(prompts[i]) + 1)

        def take(i, token):                                  # True: request i goes on
            out[i].append(token)
            return token not in eos and len(out[i]) < most(i)

        if max_new_tokens < 1:
            return out
        while waiting or running:
            fresh = []
            while waiting and len(running) + len(fresh) < max_batch:
                fresh.append(waiting.popleft())
            if fresh:
                best = self.step([(("gen", i), list(p), [len(p) - 1]) for i, p in fresh]).argmax(-1).tolist()
                for (i, _), t in zip(fresh, best):
                    if take(i, t):
                        running.append(i)
                    else:
                        self.end(("gen", i))
                continue
            left = max(most(i) - len(out[i]) for i in running)
            stepper = self._stepper(running, left) if not waiting else None
            if stepper is not None:                          # nobody joins any more: finished requests ride along
                self._replay(stepper, running, take, out)
                for i in running:
                    self.end(("gen", i))
                running = []
                continue
            best = self.step([(("gen", i), [out[i][-1]], [0]) for i in running]).argmax(-1).tolist()
            going = []
            for i, t in zip(running, best):
                if take(i, t):
                    going.append(i)
                else:
                    self.end(("gen", i))
            running = going
        return out

    def _stepper(self, running, left):
        if (not self.ragged or left < 8 or self.device.type != "cuda" or os.environ.get("TV_DECODE_GRAPH", "1") == "0"
                or not self.llm.graph_decode_supported(self.cache)):
            return None
        if self.limit is not None and max(self.cache.length(self._live[("gen", i)]) for i in running) + left > self.limit:
            return None                                      # (finished requests ride along: not past the last place)
        cache, vocab = self.cache, self.llm.config.vocab_size
        cache.default_slots = tuple(self._live[("gen", i)] for i in running)
        cache.begin_static_decode(left)
        slots, ones = cache.default_slots, [1] * len(running)
        step = lambda ids: self.llm.step(ids.view(-1), cache, cache.plan(slots, ones)).view(-1, 1, vocab)
        return GraphedDecodeStep(step, cache, len(running), self.device)

    def _replay(self, stepper, running, take, out):
        alive = {i: True for i in running}
        tok = torch.tensor([[out[i][-1]] for i in running], dtype=torch.int64).to(self.device)
        while any(alive.values()):
            tok = stepper.step(tok)
            for i, t in zip(running, tok.view(-1).tolist()):
                if alive[i]:
                    alive[i] = take(i, t)
        self.cache.end_static_decode()
        self.cache._decode_plan = None
