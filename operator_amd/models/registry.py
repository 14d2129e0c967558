"""Model registry: configuration -> model class.

``build_model`` is how the engine factory, the trace replay and the benchmarks make a model;
a new architecture adds its ``arch`` name here and its configuration to ``config.py``.
"""
from __future__ import annotations

from .config import ARCHS, config_from_dir, get_config
from .llama import LlamaModel
from .relurax import ReluraxModel
from .sufolix import SufolixModel

MODELS = {**{a: LlamaModel for a in ARCHS}, "sufolix": SufolixModel, "relurax": ReluraxModel}


def load_config(name: str, model_path: str | None = None):
    """A preset by name, or the configuration of the checkpoint directory ``model_path``."""
    import os

    if model_path and os.path.exists(os.path.join(model_path, "config.json")):
        return config_from_dir(model_path, name=name)
    return get_config(name)


def model_class(cfg):
    return MODELS[cfg.arch]


def build_model(cfg, **kw):
    """An empty model of ``cfg``'s class (weights: ``init_random`` / ``load_checkpoint``)."""
    return model_class(cfg)(cfg, **kw)
