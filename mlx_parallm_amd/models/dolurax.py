"""Dolurax model handle: chunked grouped-query attention and a mixture of experts, layer norms behind the sublayers
(``config["architecture"] = "Dolurax"``).

A layer is ``x += norm1(attention(x))``, then ``x += norm2(experts(x))``, without a norm in front of either.  The
configuration lists the layers with their own sizes, so the engine gets one ``mi_layer_desc`` per layer (``layer_list``); the
handle around it is the one of the llama family.
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import Any, Dict, List, Optional

from .base import BaseModelArgs, BatchedKVCache, make_cache_list
from .llama import Model as _LlamaModel

SLOPE_EXP = 8.0                      # head h of H takes 2^(-8 (h + 1) / H) off a score per token of distance
MIXERS = ("attention",)


@dataclass
class ModelArgs(BaseModelArgs):
    vocab: int
    width: int
    layers: List[Dict[str, Any]]
    norm: Dict[str, float]
    logit_scale: float = 1.0
    logit_softcap: Optional[float] = None
    model_type: str = "dolurax"

    def __post_init__(self):
        for i, layer in enumerate(self.layers):
            if layer["type"] not in MIXERS:
                raise ValueError(f"layer {i}: mixer type {layer['type']!r} not supported")
            mlp = layer.get("mlp")
            if mlp and mlp.get("kind", "moe") != "moe":
                raise ValueError(f"layer {i}: feed-forward kind {mlp['kind']!r} not supported")

    @property
    def num_hidden_layers(self) -> int:
        return len(self.layers)


def layer_list(config: dict):
    """``config.json`` -> (fields of ``mi_model_desc``, fields of one ``mi_layer_desc`` per layer)."""
    from .. import _lib as L

    a = ModelArgs.from_dict(config)
    model = dict(hidden_size=int(a.width), num_layers=len(a.layers), vocab_size=int(a.vocab), rms_norm_eps=float(a.norm["eps"]),
                 position=L.MI_POS_NONE, block_form=L.MI_BLOCK_POST_NORM, norm_kind=L.MI_NORM_LAYER,
                 logit_scale=float(a.logit_scale if a.logit_scale is not None else 1.0), logit_softcap=float(a.logit_softcap or 0.0))
    layers = []
    for layer in a.layers:
        m, mlp = layer["mixer"], layer.get("mlp")
        d = dict(mixer=L.MI_MIXER_GQA, heads=int(m["heads"]), kv_heads=int(m["kv_heads"]), dim=int(m["dim"]), vdim=int(m["vdim"]),
                 kv_from=-1, scale=float(m["scale"]), softcap=float(m.get("softcap") or 0.0), slope_exp=SLOPE_EXP,
                 chunk=int((m.get("mask") or {}).get("size") or 0), v_mix=int(bool(m.get("v_mix"))), out_gate=L.MI_GATE_SIGMOID, act=L.MI_ACT_SWIGLU)
        if mlp:
            r = mlp["router"]
            g = r.get("groups") or {"count": 1, "keep": 1}
            d.update(ff_kind=L.MI_FF_MOE, ff=int(mlp["expert"]["ff"]), experts=int(r["experts"]), top=int(r["top"]),
                     groups=int(g["count"]), keep=int(g["keep"]), shared_ff=int((mlp.get("shared") or {}).get("ff") or 0))
        layers.append(d)
    return model, layers


class Model(_LlamaModel):
    _ARCH = "dolurax"
    ragged_prompts = True            # prompts of one batch run at their own lengths, never padded (a pad would move the chunks)

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
