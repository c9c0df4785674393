"""Model registry: a folder's config.json chooses the model class.

``load_pretrained(folder)`` reads config.json, builds the registered class
and fills it from the folder's *.safetensors.  The architecture is named by
``architecture`` or by the first of ``architectures``.
"""

import json
import os
from dataclasses import dataclass
from typing import Callable, Dict

import torch

from ..utils.safetensors_utils import load_safetensors


@dataclass(frozen=True)
class ModelEntry:
    config_from_dict: Callable[[dict], object]
    build: Callable[[object], torch.nn.Module]
    load_weights: Callable[[torch.nn.Module, Dict[str, torch.Tensor]], None]


_REGISTRY: Dict[str, ModelEntry] = {}


def register_model(name: str, entry: ModelEntry):
    _REGISTRY[name] = entry


def registered_models():
    return sorted(_REGISTRY)


def architecture_of(config: dict) -> str:
    name = config.get("architecture") or \
        (config.get("architectures") or [None])[0]
    if name not in _REGISTRY:
        raise ValueError(f"no model is registered for architecture "
                         f"{name!r}; known: {', '.join(registered_models())}")
    return name


def read_config(folder: str) -> dict:
    with open(os.path.join(folder, "config.json")) as f:
        return json.load(f)


def read_tensors(folder: str) -> Dict[str, torch.Tensor]:
    files = sorted(f for f in os.listdir(folder)
                   if f.endswith(".safetensors"))
    if not files:
        raise FileNotFoundError(f"no *.safetensors in {folder}")
    out: Dict[str, torch.Tensor] = {}
    for f in files:
        out.update(load_safetensors(os.path.join(folder, f)))
    return out


def build_model(name: str, config, dtype=torch.bfloat16, device="cpu"):
    """An instance with random weights on ``device``."""
    prev = torch.get_default_dtype()
    fast = os.environ.get("NXDA_FAST_INIT")
    torch.set_default_dtype(dtype)
    os.environ["NXDA_FAST_INIT"] = "1"   # initialise in place, once
    try:
        with torch.device(device):
            model = _REGISTRY[name].build(config)
    finally:
        torch.set_default_dtype(prev)
        if fast is None:
            del os.environ["NXDA_FAST_INIT"]
        else:
            os.environ["NXDA_FAST_INIT"] = fast
    return model.eval()


def load_pretrained(folder: str, dtype=torch.bfloat16, device="cpu"):
    config = read_config(folder)
    name = architecture_of(config)
    entry = _REGISTRY[name]
    model = build_model(name, entry.config_from_dict(config), dtype, device)
    entry.load_weights(model, read_tensors(folder))
    return model


# -- built-in entries -------------------------------------------------------

def _llama_config(d: dict):
    from .llama import LlamaConfig

    keys = ("hidden_size", "intermediate_size", "num_hidden_layers",
            "num_attention_heads", "num_key_value_heads", "vocab_size",
            "max_position_embeddings", "rope_theta", "rms_norm_eps",
            "tie_word_embeddings", "rope_scaling")
    kw = {k: d[k] for k in keys if d.get(k) is not None}
    kw.setdefault("num_key_value_heads", d["num_attention_heads"])
    kw["head_dim_override"] = d.get("head_dim")
    kw["sliding_window"] = d.get("sliding_window") \
        if d.get("use_sliding_window", True) else None
    kw["attention_bias"] = d.get("attention_bias",
                                 d.get("model_type") == "qwen2")
    return LlamaConfig(**kw)


def _llama_build(config):
    from .llama import LlamaForCausalLM

    return LlamaForCausalLM(config)


def _llama_load(model, tensors):
    from ..overrides import convert_hf_llama_state_dict

    missing, extra = model.load_state_dict(
        convert_hf_llama_state_dict(tensors), strict=False)
    if model.config.tie_word_embeddings:
        missing = [m for m in missing if m != "lm_head.weight"]
    if missing or extra:
        raise KeyError(f"checkpoint does not fit: missing {missing[:5]}, "
                       f"extra {extra[:5]}")


for _name in ("LlamaForCausalLM", "MistralForCausalLM", "Qwen2ForCausalLM"):
    register_model(_name, ModelEntry(_llama_config, _llama_build,
                                     _llama_load))


def _voletar_config(d: dict):
    from .voletar import VoletarConfig

    return VoletarConfig.from_dict(d)


def _voletar_build(config):
    from .voletar import VoletarForCausalLM

    return VoletarForCausalLM(config)


register_model("Voletar", ModelEntry(
    _voletar_config, _voletar_build,
    lambda model, tensors: model.load_checkpoint(tensors)))


def _nesilorn_config(d: dict):
    from .nesilorn import NesilornConfig

    return NesilornConfig.from_dict(d)


def _nesilorn_build(config):
    from .nesilorn import NesilornForCausalLM

    return NesilornForCausalLM(config)


register_model("Nesilorn", ModelEntry(
    _nesilorn_config, _nesilorn_build,
    lambda model, tensors: model.load_checkpoint(tensors)))


def _sutuvik_config(d: dict):
    from .sutuvik import SutuvikConfig

    return SutuvikConfig.from_dict(d)


def _sutuvik_build(config):
    from .sutuvik import SutuvikForCausalLM

    return SutuvikForCausalLM(config)


register_model("Sutuvik", ModelEntry(
    _sutuvik_config, _sutuvik_build,
    lambda model, tensors: model.load_checkpoint(tensors)))


def _pokepel_config(d: dict):
    from .pokepel import PokepelConfig

    return PokepelConfig.from_dict(d)


def _pokepel_build(config):
    from .pokepel import PokepelForCausalLM

    return PokepelForCausalLM(config)


register_model("Pokepel", ModelEntry(
    _pokepel_config, _pokepel_build,
    lambda model, tensors: model.load_checkpoint(tensors)))
