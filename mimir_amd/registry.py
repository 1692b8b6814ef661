"""The models this package runs, by architecture, and how a model on disk is
opened: a .mim file names its architecture in its metadata (general.architecture),
a folder in its config.json (architecture)."""
from __future__ import annotations

import json
import os

from . import build, capi
from .decoder import Decoder
from .mimfile import MimFile


def _llama(path: str, dtype: str | None = None, **kw) -> Decoder:
    from .llama import load_mim
    if dtype is not None:
        raise ValueError(f"{path}: dtype {dtype}: a .mim model multiplies in the block dtypes of its file")
    return load_mim(path, **kw)


def _stack(path: str, **kw) -> Decoder:
    from .stack import load_stack
    return load_stack(path, **kw)


# architecture -> (loader, the part of the library that it needs: a name of build.PARTS, None: the whole library)
ARCHITECTURES = {"llama": (_llama, None), "qwen2": (_llama, None), "Fuvolix": (_stack, "stack"), "Genetar": (_stack, "stack")}


def architecture(path: str) -> str:
    if os.path.isdir(path):
        with open(os.path.join(path, "config.json")) as f:
            arch = json.load(f).get("architecture")
    else:
        arch = MimFile(path).metadata.get("general.architecture")
    if arch not in ARCHITECTURES:
        raise ValueError(f"{path}: architecture {arch!r}, want one of {', '.join(ARCHITECTURES)}")
    return arch


def load(path: str, device: int = 0, build_missing: bool = False, **kw) -> Decoder:
    """Opens the model at path on a device. kw goes to the architecture's loader (context, max_tokens, batch, ...).
    build_missing compiles the part of the library that the model needs if it is not built."""
    loader, part = ARCHITECTURES[architecture(path)]
    if build_missing:
        build.ensure(part)
    capi.check(capi.load(part).mi355x_init(device))
    return loader(path, **kw)
