"""Runevik model handle: gated-delta-rule and latent-attention layers in any order (``config["architecture"] = "Runevik"``).

A layer is ``x += mixer(h) + ff(h)`` with ``h = norm(x)``; the norm has one weight for all coordinates; every layer ends with a
per-layer token input.  The configuration lists the layers with their own sizes, so the engine gets one ``mi_layer_desc`` per
layer (``layer_list``) instead of the uniform description of the llama family; the handle around it is the llama one.
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import Any, Dict, List, Optional

from .base import BaseModelArgs, BatchedKVCache, make_cache_list
from .llama import Model as _LlamaModel

UNIT_EPS = 1e-6                      # x / sqrt(sum x^2 + eps) of the delta rule's queries and keys
MIXERS = ("delta", "latent_attention")


@dataclass
class ModelArgs(BaseModelArgs):
    vocab: int
    width: int
    layers: List[Dict[str, Any]]
    norm: Dict[str, float]
    token_side: Optional[Dict[str, int]] = None
    model_type: str = "runevik"

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

    @property
    def side_dim(self) -> int:
        return int(self.token_side["dim"]) if self.token_side else 0


def layer_list(config: dict):
    """``config.json`` -> (fields of ``mi_model_desc``, fields of one ``mi_layer_desc`` per layer)."""
    from .. import _lib as L

    a = ModelArgs.from_dict(config)
    model = dict(hidden_size=int(a.width), num_layers=len(a.layers), vocab_size=int(a.vocab), rms_norm_eps=float(a.norm["eps"]),
                 position=L.MI_POS_SINUSOIDAL, block_form=L.MI_BLOCK_PARALLEL, norm_kind=L.MI_NORM_SCALAR, side_dim=a.side_dim)
    layers = []
    for layer in a.layers:
        m, mlp = layer["mixer"], layer.get("mlp")
        d = dict(heads=int(m["heads"]), dim=int(m["dim"]), vdim=int(m["vdim"]), kv_from=-1,
                 ff=int(mlp["ff"]) if mlp else 0, act=L.MI_ACT_POLYNORM)
        if layer["type"] == "delta":
            d.update(mixer=L.MI_MIXER_DELTA, kv_heads=int(m["kv_heads"]), conv=int(m["conv"]), scale=float(m["dim"]) ** -0.5,
                     unit_eps=UNIT_EPS, out_gate=L.MI_GATE_SILU)
        else:
            d.update(mixer=L.MI_MIXER_LATENT, kv_rank=int(m["kv_rank"]), scale=float(m["scale"]), out_gate=L.MI_GATE_SIGMOID_HEAD)
            if m.get("kv_from") is not None:
                d["kv_from"] = int(m["kv_from"])
        layers.append(d)
    return model, layers


class Model(_LlamaModel):
    _ARCH = "runevik"
    ragged_prompts = True            # prompts of one batch run at their own lengths, never padded (a pad would enter the state)

    def sanitize(self, weights):
        return weights

    def make_cache(self, batch_size: int, paged: bool = True, step: Optional[int] = None):
        return make_cache_list(BatchedKVCache, self.head_dim, [self.n_kv_heads] * len(self.layers), batch_size, step)

    @property
    def head_dim(self):              # (cache-pool key: elements a token adds to one layer's cache at most)
        return max([int(layer["mixer"].get("kv_rank", 0)) for layer in self.args.layers] + [1])

    @property
    def n_kv_heads(self):
        return 1
