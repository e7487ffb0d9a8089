"""Model registry: an architecture name in config.json, or a configuration object, leads to a model class.

A model class offers
  config_class            parses config.json (from_dict) and says what it needs
  __init__(config, weights, ops, cache settings)
  forward(ids, positions, ctx)   logits, or the final hidden rows with ctx["hidden_only"]
and registers itself with @register_model(names of the architecture in config.json).
"""
from __future__ import annotations

import json
from pathlib import Path

_BY_ARCHITECTURE: dict = {}
_BY_CONFIG: dict = {}


def register_model(*architectures):
    def decorator(cls):
        for name in architectures:
            if name in _BY_ARCHITECTURE:
                raise RuntimeError(f"architecture {name} is registered twice")
            _BY_ARCHITECTURE[name] = cls
        _BY_CONFIG[cls.config_class] = cls
        return cls

    return decorator


def architectures() -> list:
    return sorted(_BY_ARCHITECTURE)


def model_class(config):
    """The model class of a configuration object."""
    cls = _BY_CONFIG.get(type(config))
    if cls is None:
        raise ValueError(f"no model is registered for {type(config).__name__}")
    return cls


def load_config(path):
    """The configuration object of a folder's config.json ("architecture", or the first of "architectures")."""
    p = Path(path)
    return parse_config(json.loads((p / "config.json" if p.is_dir() else p).read_text()))


def parse_config(raw: dict):
    """The same from what config.json holds."""
    name = raw.get("architecture") or (raw.get("architectures") or [None])[0]
    cls = _BY_ARCHITECTURE.get(name)
    if cls is None:
        raise ValueError(f"unknown architecture {name!r}; registered: {', '.join(architectures())}")
    return cls.config_class.from_dict(raw)


from . import fedovik, lulizen, nepulix, qwen3, sozarax  # noqa: E402,F401  (register themselves)
