"""Causal language models whose steps are PACKED: the new tokens of all sequences of a step are consecutive rows, without
padding; `cache.StepPlan` says which sequence and which cache rows they belong to.  A model brings its layers (`hidden`), its
cache (`new_cache`) and its output layer (`logits`); the step and the usual (batch, tokens) call of the framework's other models
are here."""
from __future__ import annotations

from typing import Any, Optional

import torch
import torch.nn as nn
import torch.nn.functional as F

from ... import kernels as K
from .cache import SlotStateCache
from .nano import CausalLMOutputWithPast


def vocabulary_logits(h, table):
    """fp32 logits of rows in the model's dtype against a (vocab, width) matrix"""
    if K.gemv_post_takes(h.shape[0], h.shape[1], h.dtype):
        return K.gemv_post(h, table, out_dtype=torch.float32)
    return F.linear(h, table).float()


class PackedCausalLM(nn.Module):
    supports_ragged = True       # sequences of different lengths share a step (engine.py)

    def graph_decode_supported(self, cache) -> bool:
        """A decode step has fixed launch parameters: positions and key counts are read on the device."""
        return isinstance(cache, SlotStateCache)

    def hidden(self, ids, cache: SlotStateCache, plan, logits_at=None, embeds=None, trace: Optional[list] = None):
        """The step's rows (ids (T) int64, or embeds (T, width)) behind the last layer at `logits_at` (int64 tensor; None: every row), in
        the form the model's `logits` takes.  `trace` gets the stream in front of the layers and behind each of them."""
        raise NotImplementedError

    # ---- one packed step
    def step(self, ids, cache: SlotStateCache, plan, logits_at=None, embeds=None, trace: Optional[list] = None):
        """New tokens of the sequences of `plan` (ids (T) int64, or embeds (T, width)): logits fp32 at the rows `logits_at`
        (int64 tensor; None: every row)."""
        x = self.hidden(ids, cache, plan, logits_at, embeds, trace)
        cache.commit(plan)
        return self.logits(x)

    # ---- the (batch, tokens) call of the framework's other models
    def forward(self, input_ids=None, inputs_embeds=None, attention_mask=None, position_ids=None, past_key_values=None,
                labels=None, use_cache=None, cache_position=None, logits_to_keep=None, output_hidden_states=None,
                train_pdrop_args: Any = None, **kwargs):
        """input_ids (B, L) or inputs_embeds (B, L, width): the next L tokens of every sequence of the cache (a new one without
        `past_key_values`).  attention_mask (B, L) with zeros marks padding rows on either side: they are left out, and their
        logits are zero.  logits_to_keep: the last n positions (default `num_logits_to_keep`; 0: all)."""
        if (input_ids is None) == (inputs_embeds is None):
            raise ValueError("You must specify exactly one of input_ids or inputs_embeds")
        if labels is not None:
            raise NotImplementedError("loss computation is a training feature")
        src = input_ids if inputs_embeds is None else inputs_embeds
        B, L = src.shape[:2]
        cache = past_key_values if past_key_values is not None else self.new_cache(B)
        if len(cache.default_slots) != B:
            raise ValueError(f"the cache holds {len(cache.default_slots)} sequences, the call {B}")
        keep = None
        flat = src.reshape(B * L, *src.shape[2:])
        counts = [L] * B
        if attention_mask is not None and not bool(attention_mask.all()):
            m = attention_mask.bool()
            counts = [int(c) for c in m.sum(1)]
            keep = m.reshape(-1).nonzero().flatten()
            flat = flat.index_select(0, keep)
        plan = cache.plan(cache.default_slots, counts)
        trace = [] if output_hidden_states else None
        n = self.config.num_logits_to_keep if logits_to_keep is None else int(logits_to_keep)
        kw = dict(ids=flat.contiguous()) if inputs_embeds is None else dict(ids=None, embeds=flat)
        if keep is None:
            at = None
            if 0 < n < L:
                at = (torch.arange(B, device=src.device)[:, None] * L + torch.arange(L - n, L, device=src.device)).flatten()
            logits = self.step(cache=cache, plan=plan, logits_at=at, trace=trace, **kw).view(B, -1, self.vocab_size)
        else:
            packed = self.step(cache=cache, plan=plan, trace=trace, **kw)
            logits = packed.new_zeros((B * L, self.vocab_size)).index_copy_(0, keep, packed).view(B, L, -1)
            logits = logits[:, -n:] if n > 0 else logits
        return CausalLMOutputWithPast(loss=None, logits=logits, past_key_values=cache if use_cache is not False else None,
                                      hidden_states=None if trace is None else tuple(trace))
