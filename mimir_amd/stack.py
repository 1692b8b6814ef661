"""A handle on a mixer stack (mi355x_stack_create), and the Fuvolix design's
configuration for it: latent attention, mLSTM and lightning layers in any order,
each with sizes of its own (config.json beside model.safetensors)."""
from __future__ import annotations

import ctypes as C
import json
import os

import numpy as np

from . import capi
from .decoder import Decoder
from .safetensors import SafetensorsFile

DTYPES = {"bfloat16": capi.BF16, "float32": capi.F32}
_TO_ABI = {"BF16": capi.BF16, "F32": capi.F32}


class Stack(Decoder):
    """layers: capi.StackLayer each."""

    def __init__(self, config: capi.StackConfig, layers):
        self.lib = capi.load("stack")
        self.config = config
        self._layers = (capi.StackLayer * len(layers))(*layers)
        self._h = C.c_void_p()
        capi.check(self.lib.mi355x_stack_create(C.byref(config), self._layers, C.byref(self._h)))

    def tensors(self):
        """(name, rows, columns) of every tensor that the model takes (vectors: one row)."""
        out, i = [], 0
        name, n, k = C.create_string_buffer(64), C.c_int64(), C.c_int64()
        while self.lib.mi355x_stack_tensor(self._h, i, name, 64, C.byref(n), C.byref(k)) == capi.OK:
            out.append((name.value.decode(), n.value, k.value))
            i += 1
        return out


def _latent_layer(mx: dict) -> dict:
    rot = mx["rot"]
    if rot["dims"] != mx["rot_dim"]:
        raise ValueError(f"latent_attention: {rot['dims']} rotated features of {mx['rot_dim']}")
    return dict(mixer=capi.MIXER_LATENT, rot_dim=mx["rot_dim"], kv_rank=mx["kv_rank"], scale=mx["scale"], rot_base=rot["base"])


def _mlstm_layer(mx: dict) -> dict:
    return dict(mixer=capi.MIXER_MLSTM, gate_cap=mx["gate_cap"])


def _lightning_layer(mx: dict) -> dict:
    if len(mx["decay"]) != mx["heads"]:
        raise ValueError(f"lightning: {len(mx['decay'])} decays for {mx['heads']} heads")
    return dict(mixer=capi.MIXER_LIGHTNING, decay=(C.c_double * mx["heads"])(*mx["decay"]))


# a layer's 'type' in config.json -> the fields of capi.StackLayer that only this mixer has
MIXERS = {"latent_attention": _latent_layer, "mlstm": _mlstm_layer, "lightning": _lightning_layer}


def fuvolix_config(cfg: dict, context: int, batch: int = 1, dtype: str = "bfloat16"):
    """config.json -> (capi.StackConfig, [capi.StackLayer])."""
    layers = []
    for i, entry in enumerate(cfg["layers"]):
        mx, mlp = entry["mixer"], entry["mlp"]
        if entry["type"] not in MIXERS:
            raise ValueError(f"layer {i}: mixer {entry['type']!r}, want one of {', '.join(MIXERS)}")
        if mlp is not None and mlp["kind"] != "dense":
            raise ValueError(f"layer {i}: feed-forward {mlp['kind']!r}, want dense")
        layers.append(capi.StackLayer(heads=mx["heads"], dim=mx["dim"], vdim=mx["vdim"], ff=0 if mlp is None else mlp["ff"], **MIXERS[entry["type"]](mx)))
    c = capi.StackConfig(width=cfg["width"], vocab=cfg["vocab"], layers=len(layers), context=context, batch=batch, taps=cfg["canon"]["taps"],
                         norm_groups=cfg["norm"]["groups"], dtype=DTYPES[dtype], eps=cfg["norm"]["eps"])
    return c, layers


def load_fuvolix(path: str, context: int = 2048, max_tokens: int | None = None, batch: int = 1, dtype: str = "bfloat16") -> Stack:
    """path: a folder with config.json and model.safetensors. context: positions a sequence may hold; max_tokens: of
    them in one call (longer calls are cut; default: context)."""
    with open(os.path.join(path, "config.json")) as f:
        cfg = json.load(f)
    m = Stack(*fuvolix_config(cfg, context, batch, dtype))
    for name, (dt, data) in SafetensorsFile(os.path.join(path, "model.safetensors")).tensors.items():
        if dt not in _TO_ABI:
            raise ValueError(f"{name}: dtype {dt}")
        m.set_tensor(name, _TO_ABI[dt], data, int(np.prod(data.shape)))
    m.finalize(max_tokens or context)
    return m
