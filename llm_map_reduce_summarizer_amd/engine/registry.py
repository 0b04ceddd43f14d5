"""Model designs the engine serves: how a checkpoint folder's config.json becomes a configuration, and which model
class runs that configuration."""

from __future__ import annotations

import json
import os
from typing import Any, Callable, Dict, Tuple

from .config import HybridConfig, ModelConfig


def _llama():
    from .model import LlamaModel
    from .weights import config_from_hf
    return config_from_hf, LlamaModel


def _merulorn():
    from .hybrid import HybridModel
    from .weights import config_from_merulorn
    return config_from_merulorn, HybridModel


def _muzozen():
    from .hybrid import HybridModel
    from .weights import config_from_muzozen
    return config_from_muzozen, HybridModel


# architecture name in config.json -> (config reader, model class), imported on use
ARCHITECTURES: Dict[str, Callable[[], Tuple[Callable, type]]] = {
    "LlamaForCausalLM": _llama,
    "Merulorn": _merulorn,
    "Muzozen": _muzozen,
}


def architecture(path: str) -> str:
    """The design named by a config.json (directory or file); files without a name are Llama configs."""
    f = os.path.join(path, "config.json") if os.path.isdir(path) else path
    with open(f) as fh:
        c = json.load(fh)
    name = c.get("architecture") or (c.get("architectures") or ["LlamaForCausalLM"])[0]
    if name not in ARCHITECTURES:
        raise ValueError("%s: unknown architecture %r (known: %s)" % (f, name, ", ".join(sorted(ARCHITECTURES))))
    return name


def load_config(path: str, name: str = "hf"):
    """Model configuration of a checkpoint folder (or config.json)."""
    return ARCHITECTURES[architecture(path)]()[0](path, name)


def model_class(cfg: Any) -> type:
    if isinstance(cfg, HybridConfig):
        from .hybrid import HybridModel
        return HybridModel
    if isinstance(cfg, ModelConfig):
        from .model import LlamaModel
        return LlamaModel
    raise TypeError("no model class for %r" % type(cfg).__name__)
