"""Temetar model handle: sliding-window attention with kept first tokens and a sink, a delta rule with a decay per channel,
several residual streams (hyper-connections), layers that run more than once (``config["architecture"] = "Temetar"``).

A sublayer reads a weighted sum of the streams through a norm and is written back to all of them.  The configuration lists the
layers with their own sizes, so the engine gets one ``mi_layer_desc`` per layer (``layer_list``); the handle around it is the
one of the llama family.  The inner sizes of the low-rank maps stand in the tensors' shapes only (``complete_config``).
"""
from __future__ import annotations

import copy
from dataclasses import dataclass, field
from typing import Any, Dict, List, Optional, Tuple

from .base import BaseModelArgs, BatchedKVCache, make_cache_list
from .llama import Model as _LlamaModel

UNIT_EPS = 1e-6                      # x / sqrt(sum x^2 + eps) of the delta rule's queries and keys
MIXERS = ("attention", "channel_delta")


@dataclass
class ModelArgs(BaseModelArgs):
    vocab: int
    width: int
    layers: List[Dict[str, Any]]
    norm: Dict[str, float]
    embedding: Dict[str, Any] = field(default_factory=dict)
    loop: Optional[Dict[str, int]] = None
    residual_mult: float = 1.0
    streams: int = 0
    model_type: str = "temetar"

    def __post_init__(self):
        for i, layer in enumerate(self.layers):
            if layer["type"] not in MIXERS:
                raise ValueError(f"layer {i}: mixer type {layer['type']!r} not supported")
            mlp = layer.get("mlp")
            if mlp and mlp.get("kind", "dense") != "dense":
                raise ValueError(f"layer {i}: feed-forward kind {mlp['kind']!r} not supported")

    @property
    def num_hidden_layers(self) -> int:
        return len(self.layers)


def layer_list(config: dict):
    """``config.json`` -> (fields of ``mi_model_desc``, fields of one ``mi_layer_desc`` per layer)."""
    from .. import _lib as L

    a = ModelArgs.from_dict(config)
    model = dict(hidden_size=int(a.width), num_layers=len(a.layers), vocab_size=int(a.vocab), rms_norm_eps=float(a.norm["eps"]),
                 position=L.MI_POS_NONE, block_form=L.MI_BLOCK_PRE_NORM, norm_kind=L.MI_NORM_VECTOR, norm_offset=1,
                 embed_scale=float(a.embedding.get("scale", 1.0)), residual_mult=float(a.residual_mult), streams=int(a.streams or 0))
    pair = a.embedding.get("bigram")
    if pair:
        n = int(pair["buckets"])
        model.update(pair_buckets=n, pair_mul_prev=int(pair["mul_prev"]) % n, pair_mul_cur=int(pair["mul_cur"]) % n)
    if a.loop:
        start, stop, times = (int(a.loop[k]) for k in ("start", "stop", "times"))
        if not 0 <= start <= stop <= len(a.layers) or times < 0:
            raise ValueError(f"loop {a.loop}: not a range of the {len(a.layers)} layers")
        if stop > start:
            model.update(loop_start=start, loop_stop=stop, loop_times=times)
    layers = []
    for i, layer in enumerate(a.layers):
        m, mlp = layer["mixer"], layer.get("mlp")
        d = dict(heads=int(m["heads"]), kv_heads=int(m["kv_heads"]), dim=int(m["dim"]), vdim=int(m["vdim"]), kv_from=-1,
                 ff=int(mlp["ff"]) if mlp else 0, ff_kind=L.MI_FF_DENSE, act=L.MI_ACT_SWIGLU)
        if layer["type"] == "channel_delta":
            if "decay_rank" not in m or "gate_rank" not in m:
                raise ValueError(f"layer {i}: the inner sizes of the decay and gate maps are missing (complete_config)")
            d.update(mixer=L.MI_MIXER_DELTA, conv=int(m["conv"]), scale=float(m["dim"]) ** -0.5, unit_eps=UNIT_EPS,
                     decay_rank=int(m["decay_rank"]), gate_rank=int(m["gate_rank"]), out_gate=L.MI_GATE_SIGMOID)
        else:
            rot, mask = m.get("rot") or {}, m.get("mask") or {}
            d.update(mixer=L.MI_MIXER_GQA, scale=float(m["scale"]), rot_dims=int(rot.get("dims", 0)), rot_base=float(rot.get("base", 1.0)),
                     window=int(mask.get("size") or 0), keep_first=int(mask.get("keep_first") or 0), sink=1, out_gate=L.MI_GATE_NONE)
        layers.append(d)
    return model, layers


class Model(_LlamaModel):
    _ARCH = "temetar"
    ragged_prompts = True            # prompts of one batch run at their own lengths, never padded (a pad would enter the state)

    @classmethod
    def complete_config(cls, config: dict, shapes: Dict[str, Tuple[int, ...]]) -> dict:
        out = copy.deepcopy(config)
        for i, layer in enumerate(out["layers"]):
            if layer["type"] == "channel_delta":
                for key, name in (("decay_rank", "a1"), ("gate_rank", "g1")):
                    if f"l{i}.mix.{name}" not in shapes:
                        raise ValueError(f"l{i}.mix.{name} is missing")
                    layer["mixer"][key] = int(shapes[f"l{i}.mix.{name}"][0])
        return out

    def sanitize(self, weights):
        return weights

    def make_cache(self, batch_size: int, paged: bool = True, step: Optional[int] = None):
        return make_cache_list(BatchedKVCache, self.head_dim, [self.n_kv_heads] * len(self.layers), batch_size, step)

    @property
    def head_dim(self):              # (cache-pool key)
        return max(max(int(layer["mixer"]["dim"]), int(layer["mixer"]["vdim"])) for layer in self.args.layers)

    @property
    def n_kv_heads(self):
        return max(int(layer["mixer"]["kv_heads"]) for layer in self.args.layers)
