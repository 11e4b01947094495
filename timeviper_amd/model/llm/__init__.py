from .cache import SlotStateCache
from .checkpoint import load_llm
from .engine import TextEngine
from .fasovik import FasovikConfig, FasovikForCausalLM
from .fogorax import FogoraxConfig, FogoraxForCausalLM
from .llm_factory import GenericLLMBackbone, get_llm_config
from .nano import (HybridMambaAttentionDynamicCache, NemotronHConfig, NemotronHForCausalLM,
                   NemotronHModel)

__all__ = ["GenericLLMBackbone", "get_llm_config", "NemotronHConfig", "NemotronHForCausalLM",
           "FasovikConfig", "FasovikForCausalLM", "FogoraxConfig", "FogoraxForCausalLM", "SlotStateCache", "TextEngine", "load_llm",
           "NemotronHModel", "HybridMambaAttentionDynamicCache"]
