"""Small Dolurax configurations for the tests: sizes with awkward remainders, every branch of the design, values that are 1."""
from __future__ import annotations


def attn(heads, kv_heads, dim, vdim, chunk, scale=0.4, softcap=20.0, v_mix=True):
    return {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "mask": {"size": chunk} if chunk else None, "scale": scale,
            "softcap": softcap, "v_mix": v_mix}


def moe(experts, top, ff, groups=1, keep=1, shared=0):
    m = {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top, "groups": {"count": groups, "keep": keep}}}
    if shared:
        m["shared"] = {"ff": shared}
    return m


def layer(mixer, mlp=None):
    return {"type": "attention", "mixer": mixer, "mlp": mlp}


def config(width, vocab, layers, eps=1e-5, logit_scale=0.5, logit_softcap=25.0):
    return {"architecture": "Dolurax", "width": width, "vocab": vocab, "layers": layers, "norm": {"eps": eps}, "logit_scale": logit_scale,
            "logit_softcap": logit_softcap}


CONFIGS = {
    # nothing divides anything: padded matrices, scalar loads, an odd vocabulary; the first layer does not mix
    "odd": config(100, 333, [layer(attn(6, 2, 20, 36, 37, v_mix=False), moe(6, 3, 40, 3, 2, 72)),
                             layer(attn(5, 5, 24, 12, 64), moe(8, 2, 24, 4, 3, 16)),
                             layer(attn(4, 2, 33, 30, 0, 0.3, None)),
                             layer(attn(3, 3, 16, 20, 10), moe(5, 5, 33)),
                             layer(attn(6, 1, 40, 60, 50, 0.2), moe(9, 4, 48, 3, 3, 130))], 3e-6),
    # two head tiles, head sizes of the matrix-core kernels, many experts in groups
    "wide": config(256, 512, [layer(attn(34, 2, 128, 64, 96, 0.09), moe(40, 5, 64, 8, 3, 192)),
                              layer(attn(8, 4, 64, 128, 130, 0.125, v_mix=False), moe(16, 4, 128, 2, 1)),
                              layer(attn(4, 1, 32, 128, 70, 0.2), moe(24, 3, 96, 6, 6, 64))]),
    # everything is one
    "ones": config(64, 96, [layer(attn(1, 1, 1, 1, 1, 1.0, 1.0), moe(1, 1, 1, 1, 1, 1)), layer(attn(1, 1, 1, 1, 1, 1.0, 1.0), moe(1, 1, 1)),
                            layer(attn(2, 1, 1, 1, 3, 1.0, 1.0), moe(2, 1, 1, 2, 1, 1))], 1e-5, 1.0, 1.0),
    # head sizes beyond the matrix-core kernels, more experts than the matrix-core router takes, no logit transformation
    "generic": config(128, 160, [layer(attn(2, 1, 144, 200, 45, 0.08), moe(300, 2, 8)), layer(attn(2, 2, 136, 100, 33, 0.1), moe(3, 1, 700))],
                      1e-5, 1.0, None),
    # matrix-core and generic attention in one stack, mixed values between them
    "both_forms": config(80, 120, [layer(attn(2, 1, 144, 64, 30, 0.08), moe(4, 2, 24)), layer(attn(4, 2, 48, 32, 41, 0.15)),
                                   layer(attn(1, 1, 200, 64, 0, 0.07, None), moe(4, 1, 16, 4, 2, 8)), layer(attn(2, 1, 96, 64, 25, 0.1))]),
    # a wide row (several pieces per thread in the row kernels)
    "wide_row": config(2304, 96, [layer(attn(3, 1, 48, 64, 40), moe(4, 2, 64, 2, 2, 96)), layer(attn(2, 2, 64, 32, 25))]),
}
