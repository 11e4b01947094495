"""`GenericLLMBackbone` (reference timeviper/model/llm/llm_factory.py:41-198): thin
wrapper owning `.llm` (the causal LM), the tokenizer and the `<image>` token.  There is
no network here, so instead of `from_pretrained` the backbone is built from a config
(random init, the reference's `_from_config` branch :101) and the tokenizer is either
handed in or a minimal stand-in that only knows the special-token ids."""
from __future__ import annotations

from typing import Optional

import torch
import torch.nn as nn

from .fasovik import FasovikConfig, FasovikForCausalLM
from .fogorax import FogoraxConfig, FogoraxForCausalLM
from .nano import NemotronHConfig, NemotronHForCausalLM
from .qwen2 import Qwen2Config, Qwen2ForCausalLM

# family -> (configuration, causal LM): everything that builds or loads a language model goes through this table
LLM_FAMILIES = {
    "nano": (NemotronHConfig, NemotronHForCausalLM),
    "qwen2": (Qwen2Config, Qwen2ForCausalLM),
    "fasovik": (FasovikConfig, FasovikForCausalLM),
    "fogorax": (FogoraxConfig, FogoraxForCausalLM),
}

MODEL_REGISTRY = {
    # llm_registry.py:64-97 — ids the reference accepts for the nano family
    "nanov2-9b": "nvidia/NVIDIA-Nemotron-Nano-9B-v2",
    "nanov2-9b-base": "nvidia/NVIDIA-Nemotron-Nano-9B-v2-Base",
}
QWEN2_REGISTRY = {
    # llm_registry.py:65-77.  Only the 7B geometries have a config preset here (public
    # config.json values); the other ids need an explicit `config=`.
    "qwen2-7b": "Qwen/Qwen2-7B", "qwen2-7b-instruct": "Qwen/Qwen2-7B-Instruct",
    "qwen2-1.5b": "Qwen/Qwen2-1.5B", "qwen2-1.5b-instruct": "Qwen/Qwen2-1.5B-Instruct",
    "qwen2.5-7b-instruct": "Qwen/Qwen2.5-7B-Instruct", "qwen2.5-7b-base": "Qwen/Qwen2.5-7B-Base",
    "qwen2.5-3b-instruct": "Qwen/Qwen2.5-3B-Instruct", "qwen2.5-3b-base": "Qwen/Qwen2.5-3B-Base",
}
# layer-list designs: sizes come with a configuration (`config=`, or a checkpoint folder)
LAYER_LIST_REGISTRY = {"fasovik": "Fasovik", "fogorax": "Fogorax"}
_QWEN2_7B = ("qwen2-7b", "qwen2-7b-instruct", "qwen2.5-7b-instruct", "qwen2.5-7b-base")
DEFAULT_TOKEN = "<image>"


def llm_family_of(llm_backbone_id: str) -> str:
    if llm_backbone_id in MODEL_REGISTRY:
        return "nano"
    if llm_backbone_id in QWEN2_REGISTRY:
        return "qwen2"
    if llm_backbone_id in LAYER_LIST_REGISTRY:
        return llm_backbone_id
    raise ValueError(f"LLM backbone `{llm_backbone_id}` is not supported!")


def get_llm_config(llm_backbone_id: str, **over):
    family = llm_family_of(llm_backbone_id)
    if family == "nano":
        return NemotronHConfig.nemotron_nano_9b_v2(**over)
    if llm_backbone_id in _QWEN2_7B:
        return Qwen2Config.qwen2_5_7b(**over)
    raise ValueError(f"no built-in geometry for `{llm_backbone_id}`; pass config={LLM_FAMILIES[family][0].__name__}(...)")


def config_from_dict(d: dict):
    """Configuration object of a checkpoint's config.json: "architecture" names a design of this framework, "model_type" one of
    the mirrored families."""
    for config_cls, _ in LLM_FAMILIES.values():
        if d.get("architecture") is not None and d["architecture"] == getattr(config_cls, "architecture", None):
            return config_cls.from_dict(d)
    kind = d.get("model_type")
    if kind in LLM_FAMILIES and not hasattr(LLM_FAMILIES[kind][0], "architecture"):
        return LLM_FAMILIES[kind][0](**{k: v for k, v in d.items() if k not in ("model_type", "architecture", "architectures")})
    raise ValueError(f"config.json: unknown architecture {d.get('architecture')!r} / model_type {kind!r}")


def llm_class(config):
    return LLM_FAMILIES[config.model_type][1]


class SyntheticTokenizer:
    """Stand-in used for synthetic benchmarks/tests (no tokenizer files offline)."""

    def __init__(self, vocab_size: int):
        self.vocab_size = vocab_size
        self.image_token_id = vocab_size - 1
        self.eos_token_id = 2
        self.pad_token_id = 0

    def convert_tokens_to_ids(self, tok):
        return self.image_token_id if tok == DEFAULT_TOKEN else 3

    def decode(self, ids, skip_special_tokens: bool = False) -> str:
        """ids -> text: one `<id>` word per token (there is no vocabulary offline)."""
        return " ".join(f"<{int(i)}>" for i in ids)

    def __call__(self, text: str, add_special_tokens: bool = False, return_tensors: str = "pt"):
        """text -> ids, one id per whitespace-separated word (a `<id>` word maps back to its id,
        anything else to a stable id in [3, vocab-1)) — the call shape of
        `tokenizer(answer_prompt, add_special_tokens=False, return_tensors="pt").input_ids`
        (generic_vlm.py:774-776)."""
        import types
        import zlib
        out = []
        for w in text.split():
            if w.startswith("<") and w.endswith(">") and w[1:-1].isdigit():
                out.append(int(w[1:-1]))
            else:
                out.append(3 + zlib.crc32(w.encode()) % max(1, self.vocab_size - 4))
        return types.SimpleNamespace(input_ids=torch.tensor([out], dtype=torch.long))

    def __len__(self):
        return self.vocab_size


class GenericLLMBackbone(nn.Module):
    def __init__(self, llm_backbone_id: str, config=None,
                 tokenizer=None, llm_max_length: Optional[int] = None, inference_mode: bool = True,
                 attn_implementation: str = "flash_attention_2", merge_module: str = "no_merge",
                 use_pdrop: bool = False, pdrop_type: Optional[str] = None) -> None:
        super().__init__()
        self.identifier = llm_backbone_id
        self.llm_family = llm_family_of(llm_backbone_id)
        self.llm_max_length = llm_max_length
        self.inference_mode = inference_mode
        if config is None:
            config = get_llm_config(llm_backbone_id, merge_module=merge_module, use_pdrop=use_pdrop,
                                    pdrop_type=pdrop_type)
        else:
            config.merge_module, config.use_pdrop, config.pdrop_type = merge_module, use_pdrop, pdrop_type
        config._attn_implementation = attn_implementation
        want, llm_cls = LLM_FAMILIES[self.llm_family]
        if not isinstance(config, want):
            raise TypeError(f"`{llm_backbone_id}` needs a {want.__name__}, got {type(config).__name__}")
        self.llm = llm_cls(config)
        self.tokenizer = tokenizer or SyntheticTokenizer(config.vocab_size)
        self.terminators = [self.tokenizer.eos_token_id]

    @property
    def embed_dim(self) -> int:
        return self.llm.config.hidden_size

    @property
    def half_precision_dtype(self) -> torch.dtype:
        return torch.bfloat16

    @classmethod
    def from_folder(cls, folder, dtype=torch.bfloat16, device=None, tokenizer=None) -> "GenericLLMBackbone":
        """Backbone of a checkpoint folder (config.json + model.safetensors; checkpoint.py)."""
        from .checkpoint import load_llm
        llm = load_llm(folder, dtype, device)
        self = cls.__new__(cls)
        nn.Module.__init__(self)
        self.identifier, self.llm_family = llm.config.model_type, llm.config.model_type
        self.llm_max_length, self.inference_mode, self.llm = None, True, llm
        self.tokenizer = tokenizer or SyntheticTokenizer(llm.config.vocab_size)
        self.terminators = [self.tokenizer.eos_token_id]
        return self

    def generate(self, prompts, max_new_tokens: int = 128, eos_token_id=None, max_batch: int = 16):
        """Greedy continuation of token-id prompts through the batch scheduler (engine.py): list of new-token lists."""
        from .engine import TextEngine
        eos = self.terminators if eos_token_id is None else eos_token_id
        return TextEngine(self.llm).generate(prompts, max_new_tokens, eos, max_batch)

    def embed_input_ids(self, input_ids: torch.LongTensor) -> torch.Tensor:
        return self.llm.get_input_embeddings()(input_ids)

    def forward(self, input_ids=None, attention_mask=None, position_ids=None, past_key_values=None,
                inputs_embeds=None, labels=None, use_cache=None, output_attentions=None,
                output_hidden_states=None, return_dict=None, inference_params=None,
                num_last_tokens: int = 0, cache_position=None, logits_to_keep=None, seq_idx=None,
                train_pdrop_args=None):
        """llm_factory.py:177-198."""
        return self.llm(input_ids=input_ids, attention_mask=attention_mask,
                        position_ids=position_ids, past_key_values=past_key_values,
                        inputs_embeds=inputs_embeds, labels=labels, use_cache=use_cache,
                        output_hidden_states=output_hidden_states, cache_position=cache_position,
                        logits_to_keep=logits_to_keep, train_pdrop_args=train_pdrop_args)
