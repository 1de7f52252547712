"""The model registry: architecture name (config.json's "architecture") -> configuration reader
and decoder class, and the loading of a model folder (config.json + model.safetensors)."""
import json
import os
from dataclasses import fields
from typing import Callable, Dict, NamedTuple

import torch

from .checkpoint_utils import read_safetensors
from .config import HybridConfig, OPTConfig
from .hybrid_decoder import HybridDecoder
from .transformer_decoder import TransformerDecoder


class Architecture(NamedTuple):
    config_class: type
    read_config: Callable    # parsed config.json -> configuration
    decoder_class: type
    dtypes: tuple            # compute formats, the serving one first


def _opt_config(obj):
    known = {f.name for f in fields(OPTConfig)}
    return OPTConfig(**{k: v for k, v in obj.items() if k in known})


ARCHITECTURES: Dict[str, Architecture] = {
    "OPT": Architecture(OPTConfig, _opt_config, TransformerDecoder, (torch.float16,)),
    "Sinulorn": Architecture(HybridConfig, HybridConfig.from_json, HybridDecoder,
                             (torch.bfloat16, torch.float32)),
    "Nomalorn": Architecture(HybridConfig, HybridConfig.from_json, HybridDecoder,
                             (torch.bfloat16, torch.float32)),
}


def register(name: str, architecture: Architecture):
    if name in ARCHITECTURES:
        raise ValueError("architecture %r is registered already" % name)
    ARCHITECTURES[name] = architecture


def decoder_class(cfg):
    """The decoder class of a configuration object."""
    for a in ARCHITECTURES.values():
        if isinstance(cfg, a.config_class):
            return a.decoder_class
    raise NotImplementedError("no decoder for a %s" % type(cfg).__name__)


def read_config(folder: str):
    """(architecture, configuration) of a model folder."""
    with open(os.path.join(folder, "config.json")) as f:
        obj = json.load(f)
    name = obj.get("architecture")
    if name not in ARCHITECTURES:
        raise NotImplementedError("unknown architecture %r (known: %s)"
                                  % (name, ", ".join(sorted(ARCHITECTURES))))
    a = ARCHITECTURES[name]
    return a, a.read_config(obj)


def load_model(folder: str, device="cuda", dtype=None):
    """A ready model (``TransformerLanguageModel``) from a folder with config.json and
    model.safetensors.  ``dtype``: one of the architecture's compute formats (default: the one it
    is served in)."""
    from .transformer_lm import TransformerLanguageModel

    a, cfg = read_config(folder)
    dtype = dtype or a.dtypes[0]
    if dtype not in a.dtypes:
        raise ValueError("this architecture does not run in %s" % dtype)
    state = read_safetensors(os.path.join(folder, "model.safetensors"))
    kw = {"dtype": dtype} if len(a.dtypes) > 1 else {}
    return TransformerLanguageModel.build_model(cfg, state, device=device, **kw)
