"""Token mixers of the layer-list models (fasovik.py, fogorax.py): linear attention with a constant decay per head, latent
attention with sinks, and attention in a sliding window with kept first tokens.  A mixer reads the packed rows of a step (`cache.StepPlan`), keeps its state in a `SlotStateCache`
layer and returns one row per token; every constant is a constructor argument.

A mixer offers
    cache_spec()                      what the cache holds for one layer that uses it
    forward(h, cache, layer, plan)    h (T, width) in the model's dtype -> (T, width)
    decode(stream, cache, layer, plan)   the same for a few single tokens, on the fused matrix-vector kernels (`DecodeStream`)
    checkpoint_tensors()              (name in a checkpoint, view of a parameter) pairs: projections that share their input
                                      are one stacked parameter

A mixer of a layer whose sublayers run in parallel (`WindowAttention`, parallel.py) has no parameters of its own: its
projections are rows and columns of the layer's stacked matrices."""
from __future__ import annotations

from typing import Optional, Sequence

import torch
import torch.nn as nn
import torch.nn.functional as F

from ... import kernels as K


def _weight(*shape) -> nn.Parameter:
    return nn.Parameter(torch.empty(shape))


class DecodeStream:
    """The residual stream of a few single tokens between fused launches.  A sublayer's output waits (`push`) until the next
    product reads the stream: its norm and the residual add run in that product's prologue (kernels.gemv_post)."""

    def __init__(self, x, h, eps, weight_offset, mult):
        self.x, self.h, self.eps, self.offset, self.mult = x, h, eps, weight_offset, mult
        self.pending = None                     # (sublayer output, norm weight)

    def push(self, u, norm_weight):
        self.pending = (u, norm_weight)

    def project(self, weight, out_dtype=torch.bfloat16):
        if self.pending is None:
            return K.gemv_post(self.h, weight, out_dtype=out_dtype)
        (u, nw), self.pending = self.pending, None
        y, self.x, self.h = K.gemv_post(u, weight, K.GEMV_POSTNORM, residual=self.x, norm_weight=nw, eps=self.eps,
                                        weight_offset=self.offset, mult=self.mult, out_dtype=out_dtype)
        return y

    def flush(self):
        """(x, h) with nothing waiting"""
        if self.pending is not None:
            (u, nw), self.pending = self.pending, None
            self.h, self.x = K.rms_norm_ex(u, nw, self.eps, self.offset, residual=self.x, mult=self.mult)
        return self.x, self.h


class LightningAttention(nn.Module):
    """S_t = decay_h S_{t-1} + k_t v_t^T, o_t = S_t^T q_t with q, k, v = SiLU of projections; the concatenated heads are RMS-
    normed together (plain weight), multiplied by a sigmoid gate and projected."""

    def __init__(self, width: int, heads: int, dim: int, vdim: int, decay: Sequence[float], eps: float):
        super().__init__()
        if len(decay) != heads:
            raise ValueError(f"lightning attention: {len(decay)} decays for {heads} heads")
        self.heads, self.dim, self.vdim, self.eps = heads, dim, vdim, eps
        self.decay = tuple(float(d) for d in decay)
        self.nq, self.nv = heads * dim, heads * vdim
        self.qkvg = _weight(2 * self.nq + 2 * self.nv, width)       # q | k | v | gate
        self.norm = _weight(self.nv)
        self.o = _weight(width, self.nv)
        self._decay_on = {}

    def decay_on(self, device) -> torch.Tensor:
        """fp32 on the device whatever dtype the model's parameters are converted to"""
        if device not in self._decay_on:
            self._decay_on[device] = torch.tensor(self.decay, dtype=torch.float32, device=device)
        return self._decay_on[device]

    def cache_spec(self):
        return ("state", (self.heads, self.dim, self.vdim))

    def checkpoint_tensors(self):
        q, k, v, g = self.qkvg.split([self.nq, self.nq, self.nv, self.nv])
        return [("q", q), ("k", k), ("v", v), ("g", g), ("norm", self.norm), ("o", self.o)]

    def split(self, p):
        return p.split([self.nq, self.nq, self.nv, self.nv], dim=1)

    def forward(self, h, cache, layer, plan):
        q, k, v, g = self.split(F.linear(h, self.qkvg))
        y = K.lightning_attention(q, k, v, self.decay_on(h.device), cache.state(layer), plan.cu, plan.slot, self.heads,
                                  max_len=max(plan.counts), silu=True)
        return F.linear(K.rms_norm_ex(y, self.norm, self.eps, gate=g), self.o)

    def decode_takes(self, rows, dtype):
        return K.gemv_post_takes(rows, self.nv, dtype)

    def decode(self, stream, cache, layer, plan):
        q, k, v, g = self.split(stream.project(self.qkvg))
        y = K.lightning_attention(q, k, v, self.decay_on(q.device), cache.state(layer), plan.cu, plan.slot, self.heads, max_len=1, silu=True)
        return K.gemv_post(y, self.o, K.GEMV_NORMGATE, norm_weight=self.norm, eps=self.eps, gate=g)


class LatentAttention(nn.Module):
    """Causal softmax attention whose keys and values are products of one normed latent per token, without positions, with a
    learned sink logit per head in the denominator.  The cache holds the latents.  Prompts: keys and values are expanded once
    per step.  Single tokens: the queries are taken to the latents instead (W_uk^T q) and the weighted latents back (W_uv)."""

    def __init__(self, width: int, heads: int, dim: int, vdim: int, kv_rank: int, scale: float, eps: float):
        super().__init__()
        self.heads, self.dim, self.vdim, self.rank, self.scale, self.eps = heads, dim, vdim, kv_rank, float(scale), eps
        self.nq, self.nk, self.nv = heads * dim, heads * dim, heads * vdim
        self.q_dkv = _weight(self.nq + kv_rank, width)              # q | down projection
        self.c_norm = _weight(kv_rank)
        self.ukv = _weight(self.nk + self.nv, kv_rank)              # key | value up projections
        self.sink = _weight(heads)
        self.o = _weight(width, self.nv)

    def cache_spec(self):
        return ("tokens", self.rank)

    def checkpoint_tensors(self):
        q, dkv = self.q_dkv.split([self.nq, self.rank])
        uk, uv = self.ukv.split([self.nk, self.nv])
        return [("q", q), ("dkv", dkv), ("dkv.norm", self.c_norm), ("uk", uk), ("uv", uv), ("sink", self.sink), ("o", self.o)]

    def sink32(self) -> torch.Tensor:
        key = K.param_key((self.sink,))
        if getattr(self, "_sink_key", None) != key:
            self._sink_val, self._sink_key = self.sink.detach().float().contiguous(), key
        return self._sink_val

    def forward(self, h, cache, layer, plan):
        q, c = F.linear(h, self.q_dkv).split([self.nq, self.rank], dim=1)
        buf = cache.tokens(layer)
        T = h.shape[0]
        if plan.decode:
            return F.linear(self._single(q, c, cache, layer, plan), self.o)
        c = K.rms_norm_ex(c, self.c_norm, self.eps, y2=cache.token_rows(layer), y2_rows=plan.rows)
        q = q.unflatten(1, (self.heads, self.dim))
        if plan.fresh:                                              # the step's own tokens are all the keys there are
            o = self._attend(q, F.linear(c, self.ukv), plan.cu, plan.cu, plan.start, plan.counts, plan.starts)
        else:
            o, r = torch.empty((T, self.heads, self.vdim), dtype=h.dtype, device=h.device), 0
            for b, (s, a, n) in enumerate(zip(plan.slots, plan.starts, plan.counts)):
                o[r:r + n] = self._attend(q[r:r + n], F.linear(buf[s, :a + n], self.ukv), *plan.alone(b), (n,), (a,))
                r += n
        return F.linear(o.reshape(T, self.nv), self.o)

    def _single(self, q, c, cache, layer, plan):
        return K.latent_decode(q, self.ukv[:self.nk], self.ukv[self.nk:], cache.tokens(layer), plan.keys, plan.slot, self.heads,
                               self.scale, self.sink32(), new=(c, self.c_norm, self.eps, plan.rows))

    def decode_takes(self, rows, dtype):
        return dtype == torch.bfloat16 and self.nv % 8 == 0 and rows * self.nv * 2 <= 128 * 1024

    def decode(self, stream, cache, layer, plan):
        q, c = stream.project(self.q_dkv).split([self.nq, self.rank], dim=1)
        return K.gemv_post(self._single(q, c, cache, layer, plan), self.o)

    def _attend(self, q, kv, cu_q, cu_k, start, counts, starts):
        """q (T, H, dim) against the expanded rows kv of the sequences' keys"""
        k, v = kv.split([self.nk, self.nv], dim=1)
        k, v = k.unflatten(1, (self.heads, self.dim)), v.unflatten(1, (self.heads, self.vdim))
        return K.attention_sink(q, k, v, cu_q, cu_k, start, counts, starts, self.scale, self.sink32())


class WindowAttention:
    """Softmax attention without positions; query heads share key / value heads in groups.  The query at position p sees the last
    `window` keys up to its own and the first `keep_first` of the sequence (window None: all); the concatenated heads are
    multiplied by a sigmoid gate.  The cache holds keys and values side by side; a mixer without `own_kv` has no key and value
    projections and reads another layer's rows, which the step has already written.

    Its projections q | k | v | gate are `in_rows` rows of the layer's input matrix, the output projection `out_cols` columns of
    the output matrix."""

    def __init__(self, heads: int, kv_heads: int, dim: int, vdim: int, scale: float, window: Optional[int] = None, keep_first: int = 0,
                 own_kv: bool = True):
        if heads % kv_heads or (window is not None and window < 1) or keep_first < 0:
            raise ValueError(f"window attention: {heads} heads on {kv_heads} key / value heads, window {window}, {keep_first} kept")
        self.heads, self.kv_heads, self.dim, self.vdim, self.scale, self.own_kv = heads, kv_heads, dim, vdim, float(scale), own_kv
        self.window, self.keep_first = K.NO_WINDOW if window is None else int(window), int(keep_first)
        self.nq, self.nv = heads * dim, heads * vdim
        self.cache_width = kv_heads * (dim + vdim)
        self.parts = [self.nq, self.cache_width if own_kv else 0, self.nv]
        self.in_rows, self.out_cols = sum(self.parts), self.nv

    def checkpoint_tensors(self, inp, out):
        q, kv, g = inp.split(self.parts)
        got = [("q", q), ("g", g), ("o", out)]
        if self.own_kv:
            k, v = kv.split([self.kv_heads * self.dim, self.kv_heads * self.vdim])
            got += [("k", k), ("v", v)]
        return got

    def attend(self, p, rows, plan, out=None):
        """p (T, in_rows): the projections; rows: the cache entry of the layer's keys and values -> the gated heads (T, out_cols)"""
        q, kv, g = p.split(self.parts, dim=1)
        q, g = q.unflatten(1, (self.heads, self.dim)), g.unflatten(1, (self.heads, self.vdim))
        o = None if out is None else out.unflatten(1, (self.heads, self.vdim))
        how = dict(window=self.window, keep_first=self.keep_first, gate=g, out=o)
        if plan.decode:
            o = K.attention_window_decode(q, rows, plan, self.kv_heads, self.scale, fresh=kv if self.own_kv else None, **how)
        else:
            if self.own_kv:
                K.scatter_rows(kv, plan.rows, rows.view(-1, self.cache_width))
            o = K.attention_window(q, rows, plan, self.kv_heads, self.scale, **how)
        return o.flatten(1) if out is None else out
