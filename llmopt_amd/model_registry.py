"""Which class serves a model directory: config.json's "architecture" names it.

A served model offers
    vocabulary                              number of tokens
    state.free_slots                        sequences that can still be opened
    open() / close(sequence)                a sequence and what it holds in device memory
    step(sequence, tokens, want) -> logits  the next tokens; float32 [len(want), vocabulary]
    decode(sequence, token) -> token        one token, greedy
    logits_row()                            the logits behind the last decode
and `load(runtime, directory, config, **options)`, which builds one.  The engine, the trace replay and the
command line use nothing else.
"""
from __future__ import annotations

import json
import os

from .layered_model import DESIGNS, LayeredModel
from .native import Runtime
from .w4a16_model import W4a16Model

_ARCHITECTURES = {}


class UnknownArchitecture(ValueError):
    pass


def register(name: str, model_class) -> None:
    _ARCHITECTURES[name] = model_class


def architectures() -> list[str]:
    return sorted(_ARCHITECTURES)


def read_config(directory: str) -> dict:
    with open(os.path.join(directory, "config.json")) as handle:
        return json.load(handle)


def model_class(config: dict):
    name = config.get("architecture")
    if name not in _ARCHITECTURES:
        raise UnknownArchitecture(f"no model for architecture {name!r}; known: {', '.join(architectures())}")
    return _ARCHITECTURES[name]


def load_model(directory: str, runtime: Runtime | None = None, **options):
    config = read_config(directory)
    return model_class(config).load(runtime or Runtime(), directory, config, **options)


for _design in DESIGNS:
    register(_design, LayeredModel)
register("W4A16Transformer", W4a16Model)
