"""Fasovik: a decoder-only language model given by a list of layers — each with a mixer (linear attention with constant
decays, or latent attention with sinks; mixers.py) and optionally a mixture-of-experts feed-forward (moe.py) — on a 32-bit
residual stream; only what a sublayer returns is normalised:

    x <- x + m norm1(mixer(x)),   x <- x + m norm2(ff(x)),   norm(u) = u / sqrt(mean(u^2) + eps) * (1 + w)

Layers may share one set of parameters ("weights_of"); their caches and states stay separate.  Embedding rows are scaled on
the way in; the logits use the table as it is.

Steps are packed (packed.py)."""
from __future__ import annotations

import os
from typing import List, Optional, Sequence

import torch
import torch.nn as nn

from ... import kernels as K
from .cache import SlotStateCache
from .mixers import DecodeStream, LatentAttention, LightningAttention, _weight
from .moe import MixtureOfExperts
from .packed import PackedCausalLM, vocabulary_logits

NORM_OFFSET = 1.0            # the norms' weights are stored around zero

MIXERS = {
    "lightning": lambda c, m: LightningAttention(c.hidden_size, m["heads"], m["dim"], m["vdim"], m["decay"], c.norm_eps),
    "latent_attention": lambda c, m: LatentAttention(c.hidden_size, m["heads"], m["dim"], m["vdim"], m["kv_rank"], m["scale"],
                                                     c.norm_eps),
}


def _moe(c, m):
    r = m["router"]
    return MixtureOfExperts(c.hidden_size, r["experts"], m["expert"]["ff"], r["top"], r.get("identity", 0))


FEED_FORWARDS = {"moe": _moe}


class FasovikConfig:
    """Configuration: the keys of a checkpoint's config.json (`from_dict`)."""

    model_type = "fasovik"
    architecture = "Fasovik"

    def __init__(self, vocab_size: int, hidden_size: int, layers: Sequence[dict], norm_eps: float = 1e-6,
                 residual_mult: float = 1.0, embedding_scale: float = 1.0, num_logits_to_keep: int = 1, use_cache: bool = True,
                 pad_token_id: Optional[int] = None, **kwargs):
        self.vocab_size, self.hidden_size = int(vocab_size), int(hidden_size)
        self.layers = [dict(l) for l in layers]
        self.norm_eps, self.residual_mult, self.embedding_scale = float(norm_eps), float(residual_mult), float(embedding_scale)
        self.num_logits_to_keep, self.use_cache, self.pad_token_id = num_logits_to_keep, use_cache, pad_token_id
        self.tie_word_embeddings = True
        self.use_pdrop, self.pdrop_type, self.merge_module = False, None, "no_merge"
        self._attn_implementation = "flash_attention_2"
        self.num_hidden_layers = len(self.layers)
        for i, l in enumerate(self.layers):
            if l.get("type") not in MIXERS:
                raise ValueError(f"layer {i}: unknown mixer type {l.get('type')!r} (known: {sorted(MIXERS)})")
            if l.get("mlp") is not None and l["mlp"].get("kind", "moe") not in FEED_FORWARDS:
                raise ValueError(f"layer {i}: unknown feed-forward {l['mlp'].get('kind')!r} (known: {sorted(FEED_FORWARDS)})")
        for k, v in kwargs.items():
            setattr(self, k, v)

    @classmethod
    def from_dict(cls, d: dict, **over) -> "FasovikConfig":
        kw = dict(vocab_size=d["vocab"], hidden_size=d["width"], layers=d["layers"], norm_eps=d["norm"]["eps"],
                  residual_mult=d.get("residual_mult", 1.0), embedding_scale=d.get("embedding", {}).get("scale", 1.0))
        kw.update(over)
        return cls(**kw)

    def owner(self, i: int) -> int:
        """The layer whose parameters layer i uses."""
        seen = set()
        while self.layers[i].get("weights_of") is not None:
            if i in seen:
                raise ValueError("weights_of: a circle of layers")
            seen.add(i)
            i = int(self.layers[i]["weights_of"])
        return i


class FasovikLayer(nn.Module):
    def __init__(self, config: FasovikConfig, spec: dict):
        super().__init__()
        self.eps, self.mult = config.norm_eps, config.residual_mult
        self.mixer = MIXERS[spec["type"]](config, spec["mixer"])
        self.norm1 = _weight(config.hidden_size)
        self.mlp = self.norm2 = None
        if spec.get("mlp") is not None:
            self.mlp = FEED_FORWARDS[spec["mlp"].get("kind", "moe")](config, spec["mlp"])
            self.norm2 = _weight(config.hidden_size)

    def checkpoint_tensors(self):
        out = [("norm1", self.norm1)] + [("mix." + n, t) for n, t in self.mixer.checkpoint_tensors()]
        if self.mlp is not None:
            out += [("norm2", self.norm2)] + [("mlp." + n, t) for n, t in self.mlp.checkpoint_tensors()]
        return out

    def forward(self, x, h, cache, layer, plan):
        """x: fp32 residual rows, h: the same in the model's dtype.  Returns both behind the layer."""
        u = self.mixer(h, cache, layer, plan)
        h, x = K.rms_norm_ex(u, self.norm1, self.eps, NORM_OFFSET, residual=x, mult=self.mult)
        if self.mlp is not None:
            h, x = self.mlp.forward_norm(h, x, self.norm2, self.eps, NORM_OFFSET, self.mult)
        return x, h

    def decode_takes(self, rows, dtype):
        return self.mixer.decode_takes(rows, dtype) and (self.mlp is None or self.mlp.decode_takes(rows, dtype))

    def decode(self, stream, cache, layer, plan):
        """A few single tokens on the fused kernels; the layer's last norm and add wait in the stream."""
        stream.push(self.mixer.decode(stream, cache, layer, plan), self.norm1)
        if self.mlp is not None:
            stream.push(self.mlp.decode(stream), self.norm2)


class ScaledEmbedding(nn.Module):
    """Embedding rows times a constant, in the table's dtype (what a caller that splices embeddings takes)."""

    def __init__(self, vocab: int, width: int, scale: float):
        super().__init__()
        self.weight, self.scale = _weight(vocab, width), scale

    def forward(self, ids):
        return K.embed_scaled(ids, self.weight, self.scale)[1].view(*ids.shape, -1)

    def rows(self, ids):
        """(fp32, table dtype) rows of flat ids"""
        return K.embed_scaled(ids, self.weight, self.scale)


class FasovikModel(nn.Module):
    def __init__(self, config: FasovikConfig):
        super().__init__()
        self.config = config
        self.embed = ScaledEmbedding(config.vocab_size, config.hidden_size, config.embedding_scale)
        owners = [config.owner(i) for i in range(config.num_hidden_layers)]
        self.layers = nn.ModuleDict({str(i): FasovikLayer(config, config.layers[i]) for i in sorted(set(owners))})
        self.order: List[str] = [str(i) for i in owners]            # parameters of every layer run
        self.final_norm = _weight(config.hidden_size)

    def _fused(self, h, plan) -> bool:
        """Single tokens of up to four sequences run on the matrix-vector kernels, with norms, residual adds, gates and the choice
        of the experts inside their neighbours; TV_DECODE_FUSED=0 keeps the general operators."""
        c = self.config
        return (plan.decode and os.environ.get("TV_DECODE_FUSED", "1") != "0" and K.gemv_post_takes(h.shape[0], c.hidden_size, h.dtype)
                and all(l.decode_takes(h.shape[0], h.dtype) for l in self.layers.values()))

    def forward(self, x, h, cache: SlotStateCache, plan, trace: Optional[list] = None):
        if trace is None and self._fused(h, plan):
            stream = DecodeStream(x, h, self.config.norm_eps, NORM_OFFSET, self.config.residual_mult)
            for i, owner in enumerate(self.order):
                self.layers[owner].decode(stream, cache, i, plan)
            return stream.flush()
        for i, owner in enumerate(self.order):
            x, h = self.layers[owner](x, h, cache, i, plan)
            if trace is not None:
                trace.append(x)
        return x, h


class FasovikForCausalLM(PackedCausalLM):
    def __init__(self, config: FasovikConfig):
        super().__init__()
        if config.use_pdrop or config.merge_module != "no_merge":
            raise NotImplementedError("token drop ranks with a backbone's attention layers: not defined for Fasovik")
        self.config = config
        self.backbone = FasovikModel(config)
        self.vocab_size = config.vocab_size

    @torch.no_grad()
    def init_random(self, seed: int = 0, std: float = 0.02):
        """Random parameters (no checkpoint): N(0, std) matrices, norms at their neutral value, zero corrections and sinks."""
        g = torch.Generator(device=self.device).manual_seed(seed)
        for name, p in self.named_parameters():
            leaf = name.rsplit(".", 1)[-1]
            if leaf in ("norm", "c_norm"):
                p.fill_(1.0)
            elif leaf in ("norm1", "norm2", "final_norm", "correction", "sink"):
                p.zero_()
            else:
                p.normal_(0.0, std, generator=g)
        return self

    @property
    def device(self):
        return self.backbone.final_norm.device

    @property
    def dtype(self):
        return self.backbone.final_norm.dtype

    def get_input_embeddings(self):
        return self.backbone.embed

    def checkpoint_tensors(self):
        """(name in model.safetensors, view of a parameter) for every tensor of the model."""
        out = [("embed", self.backbone.embed.weight), ("final.norm", self.backbone.final_norm)]
        for i, layer in self.backbone.layers.items():
            out += [(f"l{i}.{n}", t) for n, t in layer.checkpoint_tensors()]
        return out

    def new_cache(self, batch_size: int = 1, dtype=None, device=None, capacity: int = 0) -> SlotStateCache:
        specs = [self.backbone.layers[o].mixer.cache_spec() for o in self.backbone.order]
        cache = SlotStateCache(specs, max(batch_size, 1), dtype or self.dtype, device or self.device, capacity)
        cache.alloc_batch(batch_size)
        return cache

    def hidden(self, ids, cache, plan, logits_at=None, embeds=None, trace=None):
        if embeds is None:
            x, h = self.backbone.embed.rows(ids)
        else:
            x, h = embeds.float(), embeds.to(self.dtype)
        if trace is not None:
            trace.append(x)
        x, h = self.backbone(x, h, cache, plan, trace)
        return x if logits_at is None else x.index_select(0, logits_at)

    def logits(self, x):
        return vocabulary_logits(K.rms_norm_ex(x, self.backbone.final_norm, self.config.norm_eps, NORM_OFFSET), self.backbone.embed.weight)
