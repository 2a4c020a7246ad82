"""Beronex model handle: latent attention with a rotated part, windowed attention with shared keys and values, lightning attention;
dense and expert feed-forwards; a norm in front of and behind every sublayer (``config["architecture"] = "Beronex"``).

A layer is ``x += norm1b(mixer(norm1(x)))``, then ``x += norm2b(ff(norm2(x)))``.  The configuration lists the layers with their own
sizes, so the engine gets one ``mi_layer_desc`` per layer (``layer_list``); the handle around it is the one of the llama family.
"""
from __future__ import annotations

from dataclasses import dataclass, field
from typing import Any, Dict, List, Optional

from .base import BaseModelArgs, BatchedKVCache, make_cache_list
from .llama import Model as _LlamaModel

MIXERS = ("latent_attention", "attention", "lightning")


@dataclass
class ModelArgs(BaseModelArgs):
    vocab: int
    width: int
    layers: List[Dict[str, Any]]
    norm: Dict[str, float]
    embedding: Dict[str, Any] = field(default_factory=dict)
    model_type: str = "beronex"

    def __post_init__(self):
        for i, layer in enumerate(self.layers):
            kind, m, mlp = layer["type"], layer["mixer"], layer.get("mlp")
            if kind not in MIXERS:
                raise ValueError(f"layer {i}: mixer type {kind!r} not supported")
            if mlp and mlp.get("kind", "dense") not in ("dense", "moe"):
                raise ValueError(f"layer {i}: feed-forward kind {mlp['kind']!r} not supported")
            if kind == "lightning" and len(m["decay"]) != m["heads"]:
                raise ValueError(f"layer {i}: {len(m['decay'])} decays for {m['heads']} heads")
            if kind == "latent_attention" and (m.get("rot") or {"dims": 0})["dims"] != (m.get("rot_dim") or 0):
                raise ValueError(f"layer {i}: the whole rotated part turns (rot.dims = rot_dim)")

    @property
    def num_hidden_layers(self) -> int:
        return len(self.layers)


def _rotation(rot: Optional[dict]) -> dict:
    if not rot:
        return {}
    d, s = dict(rot_dims=int(rot["dims"]), rot_base=float(rot["base"])), rot.get("scaling")
    if s:
        d.update(rot_factor=float(s["factor"]), rot_original=float(s["original"]), rot_fast=float(s["fast"]), rot_slow=float(s["slow"]))
    return d


def layer_list(config: dict):
    """``config.json`` -> (fields of ``mi_model_desc``, fields of one ``mi_layer_desc`` per layer)."""
    from .. import _lib as L

    a = ModelArgs.from_dict(config)
    scale = a.embedding.get("scale")
    model = dict(hidden_size=int(a.width), num_layers=len(a.layers), vocab_size=int(a.vocab), rms_norm_eps=float(a.norm["eps"]),
                 position=L.MI_POS_NONE, block_form=L.MI_BLOCK_SANDWICH, norm_kind=L.MI_NORM_VECTOR,
                 embed_scale=float(1.0 if scale is None else scale))
    layers = []
    for layer in a.layers:
        m, mlp = layer["mixer"], layer.get("mlp")
        d = dict(heads=int(m["heads"]), dim=int(m["dim"]), vdim=int(m["vdim"]), kv_from=-1, **_rotation(m.get("rot")))
        if layer["type"] == "latent_attention":
            d.update(mixer=L.MI_MIXER_LATENT, q_rank=int(m["q_rank"]), kv_rank=int(m["kv_rank"]), scale=float(m["scale"]), rot_pairs=L.MI_ROT_HALVES,
                     out_gate=L.MI_GATE_NONE)
        elif layer["type"] == "attention":
            d.update(mixer=L.MI_MIXER_GQA, kv_heads=int(m["kv_heads"]), scale=float(m["scale"]), window=int((m.get("mask") or {}).get("size") or 0),
                     rot_pairs=L.MI_ROT_PAIRS, qk_norm=L.MI_QK_NORM_LAST, out_gate=L.MI_GATE_SIGMOID_HEAD)
            if m.get("kv_from") is not None:
                d["kv_from"] = int(m["kv_from"])
        else:
            d.update(mixer=L.MI_MIXER_LIGHTNING, decay=[float(x) for x in m["decay"]], out_gate=L.MI_GATE_SIGMOID)
        if mlp and mlp.get("kind", "dense") == "moe":
            d.update(ff_kind=L.MI_FF_MOE, ff=int(mlp["expert"]["ff"]), act=L.MI_ACT_CLAMPED, act_limit=float(mlp["expert"]["limit"]),
                     experts=int(mlp["router"]["experts"]), top=int(mlp["router"]["top"]), groups=1, keep=1, router_bias=1)
        elif mlp:
            d.update(ff_kind=L.MI_FF_DENSE, ff=int(mlp["ff"]), act=L.MI_ACT_GEGLU)
        layers.append(d)
    return model, layers


class Model(_LlamaModel):
    _ARCH = "beronex"
    ragged_prompts = True            # prompts of one batch run at their own lengths, never padded (a pad would enter the state)

    def sanitize(self, weights):
        return weights

    def make_cache(self, batch_size: int, paged: bool = True, step: Optional[int] = None):
        return make_cache_list(BatchedKVCache, self.head_dim, [self.n_kv_heads] * len(self.layers), batch_size, step)

    @property
    def head_dim(self):              # (cache-pool key)
        return max(max(int(layer["mixer"]["dim"]), int(layer["mixer"]["vdim"]), int(layer["mixer"].get("kv_rank", 0))) for layer in self.args.layers)

    @property
    def n_kv_heads(self):
        return max(int(layer["mixer"].get("kv_heads", 1)) for layer in self.args.layers)
