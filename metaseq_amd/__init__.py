"""MI355X-native incremental decoding: OPT (drop-in for metaseq's TransformerDecoder.forward /
SequenceGenerator on one gfx950 GPU) and hybrid decoders."""
from .config import HybridConfig, OPTConfig, config_from_state_dict, opt_config
from .dictionary import Dictionary
from .hub_utils import GeneratorInterface
from .hybrid_decoder import HybridDecoder
from .kv_cache import HybridCache, KVCache
from .registry import load_model
from .sequence_generator import SequenceGenerator
from .synthetic import (iter_random_state_dict, random_hybrid_state_dict, random_prompts,
                        random_state_dict)
from .transformer_decoder import ModelParallelTransformerDecoder, TransformerDecoder
from .transformer_lm import TransformerLanguageModel

__all__ = [
    "OPTConfig", "HybridConfig", "HybridDecoder", "HybridCache", "load_model", "opt_config",
    "config_from_state_dict", "Dictionary", "GeneratorInterface", "KVCache",
    "SequenceGenerator", "random_prompts", "random_state_dict", "random_hybrid_state_dict",
    "iter_random_state_dict", "TransformerDecoder", "ModelParallelTransformerDecoder",
    "TransformerLanguageModel",
]
