"""Fogorax: a decoder-only language model given by a list of parallel layers (parallel.py) — attention in a sliding window with
kept first tokens beside a gated feed-forward or none — with learned positions, a norm with one gain, a token shift in front of
every mixer and a second table of token rows that enters behind every layer.  A layer may read the keys and values of an
earlier one ("kv_from") instead of having its own.  Steps are packed (packed.py)."""
from __future__ import annotations

import os
from typing import Optional, Sequence

import torch
import torch.nn as nn

from ... import kernels as K
from .cache import SlotStateCache
from .mixers import WindowAttention, _weight
from .packed import PackedCausalLM, vocabulary_logits
from .parallel import GatedFeedForward, ParallelLayer, TokenSide


def _attention(m):
    mask = m.get("mask") or {}
    return WindowAttention(m["heads"], m["kv_heads"], m["dim"], m["vdim"], m["scale"], mask.get("size"), mask.get("keep_first", 0),
                           own_kv=m.get("kv_from") is None)


MIXERS = {"attention": _attention}
FEED_FORWARDS = {"dense": lambda m: GatedFeedForward(m["ff"])}


class FogoraxConfig:
    """Configuration: the keys of a checkpoint's config.json (`from_dict`)."""

    model_type = "fogorax"
    architecture = "Fogorax"

    def __init__(self, vocab_size: int, hidden_size: int, layers: Sequence[dict], side_dim: int, max_positions: int, norm_eps: float = 1e-6,
                 num_logits_to_keep: int = 1, use_cache: bool = True, pad_token_id: Optional[int] = None, **kwargs):
        self.vocab_size, self.hidden_size = int(vocab_size), int(hidden_size)
        self.layers = [dict(l) for l in layers]
        self.side_dim, self.max_positions, self.norm_eps = int(side_dim), int(max_positions), float(norm_eps)
        self.num_logits_to_keep, self.use_cache, self.pad_token_id = num_logits_to_keep, use_cache, pad_token_id
        self.tie_word_embeddings = False
        self.use_pdrop, self.pdrop_type, self.merge_module = False, None, "no_merge"
        self._attn_implementation = "flash_attention_2"
        self.num_hidden_layers = len(self.layers)
        for i, l in enumerate(self.layers):
            if l.get("type") not in MIXERS:
                raise ValueError(f"layer {i}: unknown mixer type {l.get('type')!r} (known: {sorted(MIXERS)})")
            if l.get("mlp") is not None and l["mlp"].get("kind") not in FEED_FORWARDS:
                raise ValueError(f"layer {i}: unknown feed-forward {l['mlp'].get('kind')!r} (known: {sorted(FEED_FORWARDS)})")
            j = l["mixer"].get("kv_from")
            if j is not None:
                if not 0 <= j < i or self.layers[j]["mixer"].get("kv_from") is not None:
                    raise ValueError(f"layer {i}: kv_from {j} is not an earlier layer with keys and values of its own")
                if any(l["mixer"][k] != self.layers[j]["mixer"][k] for k in ("heads", "kv_heads", "dim", "vdim")):
                    raise ValueError(f"layer {i}: its heads are not those of layer {j}, whose keys and values it reads")
        for k, v in kwargs.items():
            setattr(self, k, v)

    @classmethod
    def from_dict(cls, d: dict, **over) -> "FogoraxConfig":
        kw = dict(vocab_size=d["vocab"], hidden_size=d["width"], layers=d["layers"], side_dim=d["token_side"]["dim"],
                  max_positions=d["max_positions"], norm_eps=d["norm"]["eps"])
        kw.update(over)
        return cls(**kw)

    def kv_owner(self, i: int) -> int:
        """The layer whose keys and values layer i reads."""
        j = self.layers[i]["mixer"].get("kv_from")
        return i if j is None else int(j)


class TokenEmbedding(nn.Module):
    """Rows of the table as they are (without positions, which a step adds)."""

    def __init__(self, vocab: int, width: int):
        super().__init__()
        self.weight = _weight(vocab, width)

    def forward(self, ids):
        return K.embed_scaled(ids, self.weight)[1].view(*ids.shape, -1)


class FogoraxModel(nn.Module):
    def __init__(self, config: FogoraxConfig):
        super().__init__()
        self.config = config
        D = config.hidden_size
        self.embed = TokenEmbedding(config.vocab_size, D)
        self.positions = _weight(config.max_positions, D)
        self.side_embed = _weight(config.vocab_size, config.num_hidden_layers * config.side_dim)
        self.layers = nn.ModuleList(
            ParallelLayer(D, config.norm_eps, MIXERS[l["type"]](l["mixer"]),
                          FEED_FORWARDS[l["mlp"]["kind"]](l["mlp"]) if l.get("mlp") is not None else None, TokenSide(D, config.side_dim))
            for l in config.layers)
        # cache entries: the shift rows of all layers, then keys and values of the layers that have their own
        own = [i for i in range(len(self.layers)) if config.kv_owner(i) == i]
        self.kv_entry = [1 + own.index(config.kv_owner(i)) for i in range(len(self.layers))]
        self.cache_layers = [("state", (len(self.layers), 2, D))] + [("tokens", self.layers[i].mixer.cache_width) for i in own]
        self.final_gain = _weight()

    def _fused(self, ids, plan) -> bool:
        """Single tokens of up to four sequences run on the matrix-vector kernels, with activations and residual adds inside them; TV_DECODE_FUSED=0 keeps the general operators."""
        return (plan.decode and os.environ.get("TV_DECODE_FUSED", "1") != "0"
                and all(l.decode_takes(ids.numel(), self.final_gain.dtype) for l in self.layers))

    def forward(self, ids, cache: SlotStateCache, plan, trace: Optional[list] = None):
        """x (T, width) fp32 and what still waits for it"""
        x = K.embed_scaled(ids, self.embed.weight, positions=self.positions, plan=plan, need_h=False)[0]
        pending, side = None, self.side_embed.split(self.config.side_dim, dim=1)
        fused = trace is None and self._fused(ids, plan)
        if trace is not None:
            trace.append(x)
        for i, layer in enumerate(self.layers):
            run = layer.decode if fused else layer
            x, pending = run(x, pending, ids, side[i], cache.state(0)[:, i], cache.tokens(self.kv_entry[i]), plan)
            if trace is not None:
                trace.append(K.norm_shift(x, self.final_gain, self.config.norm_eps, *pending)[0])
        return x, pending


class FogoraxForCausalLM(PackedCausalLM):
    def __init__(self, config: FogoraxConfig):
        super().__init__()
        if config.use_pdrop or config.merge_module != "no_merge":
            raise NotImplementedError("token drop ranks with a backbone's full-attention layers: not defined for Fogorax")
        self.config = config
        self.backbone = FogoraxModel(config)
        self.head = _weight(config.vocab_size, config.hidden_size)
        self.vocab_size = config.vocab_size

    @torch.no_grad()
    def init_random(self, seed: int = 0, std: float = 0.02):
        """Random parameters (no checkpoint): N(0, std) matrices, gains and norms at one, no shift, no biases."""
        g = torch.Generator(device=self.device).manual_seed(seed)
        for name, p in self.named_parameters():
            leaf = name.rsplit(".", 1)[-1]
            if leaf in ("gain", "final_gain", "norm"):
                p.fill_(1.0)
            elif leaf in ("shift", "inp_bias", "out_bias"):
                p.zero_()
            else:
                p.normal_(0.0, std, generator=g)
        return self

    @property
    def device(self):
        return self.head.device

    @property
    def dtype(self):
        return self.head.dtype

    def get_input_embeddings(self):
        return self.backbone.embed

    def checkpoint_tensors(self):
        """(name in model.safetensors, view of a parameter) for every tensor of the model."""
        b = self.backbone
        out = [("embed", b.embed.weight), ("pos", b.positions), ("side.embed", b.side_embed), ("final.norm", b.final_gain), ("head", self.head)]
        for i, layer in enumerate(b.layers):
            out += [(f"l{i}.{n}", t) for n, t in layer.checkpoint_tensors()]
        return out

    def new_cache(self, batch_size: int = 1, dtype=None, device=None, capacity: int = 0) -> SlotStateCache:
        cache = SlotStateCache(self.backbone.cache_layers, max(batch_size, 1), dtype or self.dtype, device or self.device, capacity,
                               limit=self.config.max_positions)
        cache.alloc_batch(batch_size)
        return cache

    def hidden(self, ids, cache, plan, logits_at=None, embeds=None, trace=None):
        """Rows behind the last layer, and what waits for them."""
        if embeds is not None:
            raise NotImplementedError("Fogorax reads a second table by token id behind every layer: spliced embeddings have no ids")
        x, (y, w) = self.backbone(ids, cache, plan, trace)
        return (x, y, w) if logits_at is None else (x.index_select(0, logits_at), y.index_select(0, logits_at), w)

    def logits(self, hidden):
        x, y, w = hidden
        return vocabulary_logits(K.norm_shift(x, self.backbone.final_gain, self.config.norm_eps, y, w)[1], self.head)
