"""Model registry: architecture name (config.json's "architecture") -> how such a model is loaded.

A family is a function ``load(config, model_dir, **options) -> runner``.  The runner is what
llaminar_amd.engine steps: ``vocab``, ``slots``, ``cap``, ``max_rows``, ``forward(entries, want,
best)``, ``decode(slots, pos, ids, steps)``, ``max_decode_steps(n)`` and ``close()``.
Options every family takes: slots, cap, max_rows, dtype, device_id.
"""
from __future__ import annotations

import json
from pathlib import Path

_FAMILIES = {}
_SEQUENCE = set()   # families served by the sequence-model library alone


class ConfigError(ValueError):
    """config.json does not describe a model of the family it names."""


def register(name: str, sequence: bool = False):
    def add(load):
        _FAMILIES[name] = load
        if sequence:
            _SEQUENCE.add(name)
        return load
    return add


def needs_sequence_library(config: dict) -> bool:
    return config["architecture"] in _SEQUENCE


def families() -> list[str]:
    return sorted(_FAMILIES)


def read_config(model_dir) -> dict:
    config = json.loads((Path(model_dir) / "config.json").read_text())
    if not isinstance(config, dict) or not isinstance(config.get("architecture"), str):
        raise ConfigError(f"{model_dir}/config.json names no architecture")
    return config


def load_model(model_dir, **options):
    """The runner of the model in a folder, by the architecture its config.json names."""
    config = read_config(model_dir)
    name = config["architecture"]
    if name not in _FAMILIES:
        raise ConfigError(f"architecture {name!r} is not one of {', '.join(families())}")
    return _FAMILIES[name](config, Path(model_dir), **options)


def integer(where: dict, key: str, least: int = 1) -> int:
    v = where.get(key) if isinstance(where, dict) else None
    if not isinstance(v, int) or isinstance(v, bool) or v < least:
        raise ConfigError(f"config: {key!r} must be an integer of at least {least}, not {v!r}")
    return v


def number(where: dict, key: str) -> float:
    v = where.get(key) if isinstance(where, dict) else None
    if not isinstance(v, (int, float)) or isinstance(v, bool):
        raise ConfigError(f"config: {key!r} must be a number, not {v!r}")
    return float(v)


from . import bosirax, dense, kogilix  # noqa: E402,F401  (each registers itself)
