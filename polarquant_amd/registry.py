"""Which configuration and model class a checkpoint's config.json asks for.

A family is registered under the names its config.json gives itself: `architecture`, or Hugging Face's `model_type`.
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import Callable, Dict, Tuple


@dataclass(frozen=True)
class Family:
    name: str
    config: Callable                    # (dict of config.json, **options) -> configuration
    model_class: Callable               # () -> class, imported on demand
    libraries: Tuple[str, ...]          # HIP libraries its forward runs, of build.LIBRARIES
    polar_cache: bool                   # takes the polar-key cache options (rbits, tbits, vbits, ...)


_FAMILIES: Dict[str, Family] = {}


def register(family: Family, *names: str) -> None:
    for n in names:
        _FAMILIES[n.lower()] = family


def family_of(config_json: Dict) -> Family:
    name = str(config_json.get("architecture") or config_json.get("model_type", "llama"))
    fam = _FAMILIES.get(name.lower())
    if fam is None:
        raise ValueError("polarquant_amd: model_type %r is not one of %s" % (name, ", ".join(sorted(_FAMILIES))))
    return fam


def _polar_config(d, **options):
    from .checkpoint import config_from_hf
    return config_from_hf(d, **options)


def _llama():
    from .modeling_llama_polar import LlamaPolarForCausalLM
    return LlamaPolarForCausalLM


def _qwen2():
    from .modeling_qwen_polar import Qwen2PolarForCausalLM
    return Qwen2PolarForCausalLM


def _dekipel_config(d, **options):
    from .modeling_dekipel import DekipelConfig
    return DekipelConfig.from_dict(d, **options)


def _dekipel():
    from .modeling_dekipel import DekipelForCausalLM
    return DekipelForCausalLM


def _kapudra_config(d, **options):
    from .modeling_kapudra import KapudraConfig
    return KapudraConfig.from_dict(d, **options)


def _kapudra():
    from .modeling_kapudra import KapudraForCausalLM
    return KapudraForCausalLM


register(Family("llama", _polar_config, _llama, ("hip",), True), "llama", "mistral")      # (Mistral's layers are Llama's)
register(Family("qwen2", _polar_config, _qwen2, ("hip",), True), "qwen2")
register(Family("dekipel", _dekipel_config, _dekipel, ("steps", "latent"), False), "dekipel")
register(Family("kapudra", _kapudra_config, _kapudra, ("steps", "recurrent"), False), "kapudra")
