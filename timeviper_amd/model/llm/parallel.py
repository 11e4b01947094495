"""Layers whose mixer and feed-forward read one norm and run side by side on a 32-bit residual stream:

    h = norm(x),   hs = h + (h_before - h) * shift,   x <- x + (mixer(hs) + ff(h)),   x <- x + side(x)

norm: RMS norm with one gain for all coordinates; h_before: the h of the sequence's previous token (token shift, only in front of
the mixer); side: what the tokens' own rows of a second table add behind the layer.

The projections of both sublayers are stacked: one input matrix (the mixer's rows, then the feed-forward's) and one output matrix
whose columns meet the concatenated inner activations, so that mixer(hs) + ff(h) is one product with one 32-bit sum.  What
`TokenSide` returns waits, with its norm and residual add, for the next layer's norm (kernels.norm_shift)."""
from __future__ import annotations

from typing import Optional

import torch
import torch.nn as nn
import torch.nn.functional as F

from ... import kernels as K
from .mixers import _weight


class GatedFeedForward:
    """gelu_tanh(W_gate h + b) * (W_up h + b), then W_down and its bias: `in_rows` rows (gate | up) and `out_cols` columns of a parallel
    layer's matrices."""

    def __init__(self, ff: int):
        self.ff, self.in_rows, self.out_cols = ff, 2 * ff, ff

    def checkpoint_tensors(self, inp, inp_bias, out, out_bias):
        (gate, up), (gb, ub) = inp.split(self.ff), inp_bias.split(self.ff)
        return [("gate", gate), ("gate.b", gb), ("up", up), ("up.b", ub), ("down", out), ("down.b", out_bias)]

    def split(self, p):
        return p.split(self.ff, dim=1)


class TokenSide(nn.Module):
    """side(x) = norm(proj (gelu_tanh(gate x) * e)) with e the token's row of a table of its own (a slice of it per layer) and an RMS norm
    with a plain weight.  Returns what stands in front of that norm."""

    def __init__(self, width: int, dim: int):
        super().__init__()
        self.dim = dim
        self.gate, self.proj, self.norm = _weight(dim, width), _weight(width, dim), _weight(width)

    def checkpoint_tensors(self):
        return [("gate", self.gate), ("proj", self.proj), ("norm", self.norm)]

    def forward(self, h, ids, rows):
        """h: the stream in the model's dtype; rows (vocab, dim): this layer's slice of the table"""
        return F.linear(K.gated_mul(F.linear(h, self.gate), rows, K.ACT_GELU_TANH, ids=ids), self.proj)

    def decode(self, h, ids, rows):
        return K.gemv_glu(K.gemv_post(h, self.gate), rows, self.proj, ids=ids)


class ParallelLayer(nn.Module):
    def __init__(self, width: int, eps: float, mixer, mlp: Optional[GatedFeedForward], side: TokenSide):
        super().__init__()
        self.eps, self.mixer, self.mlp, self.side = eps, mixer, mlp, side
        self.n1, self.k1 = mixer.in_rows, mixer.out_cols
        n2, k2 = (mlp.in_rows, mlp.out_cols) if mlp is not None else (0, 0)
        self.gain = _weight()
        self.shift = _weight(width)
        self.inp, self.out = _weight(self.n1 + n2, width), _weight(width, self.k1 + k2)
        self.inp_bias = _weight(n2) if mlp is not None else None
        self.out_bias = _weight(width) if mlp is not None else None

    def checkpoint_tensors(self):
        got = [("norm1", self.gain), ("shift", self.shift)]
        got += [("mix." + n, t) for n, t in self.mixer.checkpoint_tensors(self.inp[:self.n1], self.out[:, :self.k1])]
        if self.mlp is not None:
            got += [("mlp." + n, t) for n, t in self.mlp.checkpoint_tensors(self.inp[self.n1:], self.inp_bias, self.out[:, self.k1:], self.out_bias)]
        return got + [("side." + n, t) for n, t in self.side.checkpoint_tensors()]

    def forward(self, x, pending, ids, side_rows, state, kv_rows, plan):
        """x (T, width) fp32 and what waits for it ((output, norm weight) or None) -> the same behind the layer.  state: the layer's shift
        rows, kv_rows: the cache entry of the mixer's keys and values."""
        y, w = pending or (None, None)
        x, h, hs = K.norm_shift(x, self.gain, self.eps, y, w, self.shift, state, plan, need_h=self.mlp is not None)
        u = torch.empty((x.shape[0], self.out.shape[1]), dtype=hs.dtype, device=hs.device)
        self.mixer.attend(F.linear(hs, self.inp[:self.n1]), kv_rows, plan, out=u[:, :self.k1])
        if self.mlp is not None:
            K.gated_mul(*self.mlp.split(F.linear(h, self.inp[self.n1:], self.inp_bias)), K.ACT_GELU_TANH, out=u[:, self.k1:])
        x, h = K.residual_add(x, F.linear(u, self.out, self.out_bias))
        return x, (self.side(h, ids, side_rows), self.side.norm)

    def decode_takes(self, rows, dtype):
        return all(K.gemv_rows_take(rows, n, dtype) for n in (self.shift.numel(), self.out.shape[1], self.side.dim)) and self.k1 % 8 == 0

    def decode(self, x, pending, ids, side_rows, state, kv_rows, plan):
        """The same for a few single tokens on matrix-vector kernels: both input products and the activation in one launch, the residual
        add behind the output product."""
        y, w = pending or (None, None)
        x, h, hs = K.norm_shift(x, self.gain, self.eps, y, w, self.shift, state, plan, need_h=self.mlp is not None)
        u = torch.empty((x.shape[0], self.out.shape[1]), dtype=hs.dtype, device=hs.device)
        p = K.gemv_pair(hs, h, self.inp, self.n1, self.inp_bias, act_out=u[:, self.k1:])
        self.mixer.attend(p, kv_rows, plan, out=u[:, :self.k1])
        x, h = K.gemv_add(u, self.out, x, self.out_bias)
        return x, (self.side.decode(h, ids, side_rows), self.side.norm)
