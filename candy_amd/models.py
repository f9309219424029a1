"""The decoders of the library by architecture name, and loading one from disk.

A GGUF file names its architecture in `general.architecture`; a model folder in the `architecture` of its config.json.
"""
from __future__ import annotations

import json
import os

from . import gguf, gulisun, hip, suvazen

DEFAULT_MAX_POS = 4096


class UnsupportedFormat(ValueError):
    """The model has no mode with activations in the format asked for."""


def _llama(dev, path, max_pos, act):
    if act == hip.ACT_F32:
        raise UnsupportedFormat("the Llama decoder quantizes its activations: it has no 32-bit mode")
    return gguf.load_llama(dev, path, max_pos)[0]


# architecture -> loader(dev, path, max_pos or None, activation format) -> hip.Decoder
ARCHITECTURES = {
    "llama": _llama,
    "Gulisun": lambda dev, path, max_pos, act: gulisun.load(dev, path, max_pos or DEFAULT_MAX_POS, act),
    "Suvazen": lambda dev, path, max_pos, act: suvazen.load(dev, path, max_pos or DEFAULT_MAX_POS, act),
}


def architecture_of(path: str) -> str:
    if os.path.isdir(path):
        with open(os.path.join(path, "config.json")) as f:
            name = json.load(f).get("architecture")
    else:
        name = gguf.GGUFFile(path).metadata.get("general.architecture", "llama")
    if name not in ARCHITECTURES:
        raise ValueError(f"{path}: unknown architecture {name!r} (known: {', '.join(sorted(ARCHITECTURES))})")
    return name


def load(dev, path: str, max_pos: int | None = None, act: int = hip.ACT_BF16) -> hip.Decoder:
    """The decoder a GGUF file or a model folder describes, its weights on the device.  max_pos: positions the cache has
    room for."""
    return ARCHITECTURES[architecture_of(path)](dev, path, max_pos, act)
