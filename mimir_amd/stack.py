"""A handle on a mixer stack (mi355x_stack_create), and the configurations of the
designs that are one: Fuvolix (latent attention, mLSTM and lightning layers
between norms) and Genetar (two kinds of attention beside their feed-forwards),
in any order, each layer with sizes of its own (config.json beside
model.safetensors)."""
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


def _attention_layer(mx: dict) -> dict:
    return dict(mixer=capi.MIXER_ATTENTION, kv_heads=mx["kv_heads"], scale=mx["scale"], softcap=mx.get("softcap") or 0.0, value_mix=bool(mx.get("v_mix")))


def _unit_attention_layer(mx: dict) -> dict:
    return dict(_attention_layer(mx), unit_qk=1)


def _rotary_attention_layer(mx: dict) -> dict:
    rot, scaling = mx["rot"], mx["rot"].get("scaling")
    out = dict(_attention_layer(mx), head_gate=1, rot_dim=rot["dims"], rot_base=rot["base"])
    if scaling:
        out |= dict(rot_factor=scaling["factor"], rot_low=scaling["low"], rot_high=scaling["high"], rot_original=scaling["original"])
    return out


# a design's layer 'type' in config.json -> the fields of capi.StackLayer that only this mixer has
FUVOLIX_MIXERS = {"latent_attention": _latent_layer, "mlstm": _mlstm_layer, "lightning": _lightning_layer}
GENETAR_MIXERS = {"attention": _unit_attention_layer, "attention_2": _rotary_attention_layer}


def _layers(cfg: dict, mixers: dict, mlp_kind: int):
    out = []
    for i, entry in enumerate(cfg["layers"]):
        mx, mlp = entry["mixer"], entry.get("mlp")
        if entry["type"] not in mixers:
            raise ValueError(f"layer {i}: mixer {entry['type']!r}, want one of {', '.join(mixers)}")
        if mlp is not None and mlp["kind"] != "dense":
            raise ValueError(f"layer {i}: feed-forward {mlp['kind']!r}, want dense")
        out.append(capi.StackLayer(heads=mx["heads"], dim=mx["dim"], vdim=mx["vdim"], ff=0 if mlp is None else mlp["ff"], mlp=mlp_kind, **mixers[entry["type"]](mx)))
    return out


def fuvolix_config(cfg: dict, context: int, batch: int = 1, dtype: str = "bfloat16"):
    """config.json -> (capi.StackConfig, [capi.StackLayer])."""
    layers = _layers(cfg, FUVOLIX_MIXERS, capi.MLP_RELU2)
    c = capi.StackConfig(width=cfg["width"], vocab=cfg["vocab"], layers=len(layers), context=context, batch=batch, taps=cfg["canon"]["taps"],
                         norm_groups=cfg["norm"]["groups"], dtype=DTYPES[dtype], eps=cfg["norm"]["eps"], logit_scale=1.0,
                         flags=capi.STACK_EMBED_NORM | capi.STACK_POST_NORMS | capi.STACK_DEPTH_AVERAGE)
    return c, layers


def genetar_config(cfg: dict, context: int, batch: int = 1, dtype: str = "bfloat16"):
    """config.json -> (capi.StackConfig, [capi.StackLayer])."""
    layers = _layers(cfg, GENETAR_MIXERS, capi.MLP_SWIGLU)
    pairs = cfg["embedding"]["bigram"]
    c = capi.StackConfig(width=cfg["width"], vocab=cfg["vocab"], layers=len(layers), context=context, batch=batch, taps=0, norm_groups=1, dtype=DTYPES[dtype],
                         eps=cfg["norm"]["eps"], logit_scale=cfg["logit_scale"], pair_buckets=pairs["buckets"], pair_mul_prev=pairs["mul_prev"],
                         pair_mul_cur=pairs["mul_cur"], flags=capi.STACK_PARALLEL | capi.STACK_LAYER_SCALE | capi.STACK_OUTPUT_MATRIX)
    return c, layers


# architecture in config.json -> its reader
CONFIGS = {"Fuvolix": fuvolix_config, "Genetar": genetar_config}


def load_stack(path: str, context: int = 2048, max_tokens: int | None = None, batch: int = 1, dtype: str = "bfloat16") -> Stack:
    """path: a folder with config.json and model.safetensors. context: positions a sequence may hold; max_tokens: of
    them in one call (longer calls are cut; default: context)."""
    with open(os.path.join(path, "config.json")) as f:
        cfg = json.load(f)
    m = Stack(*CONFIGS[cfg["architecture"]](cfg, context, batch, dtype))
    for name, (dt, data) in SafetensorsFile(os.path.join(path, "model.safetensors")).tensors.items():
        if dt not in _TO_ABI:
            raise ValueError(f"{name}: dtype {dt}")
        m.set_tensor(name, _TO_ABI[dt], data, int(np.prod(data.shape)))
    m.finalize(max_tokens or context)
    return m
