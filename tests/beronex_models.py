"""Small Beronex configurations for the tests: sizes with awkward remainders, every branch of the design, values that are 1."""
from __future__ import annotations


def dense(ff):
    return {"kind": "dense", "ff": ff}


def moe(experts, top, ff, limit=1.5):
    return {"kind": "moe", "router": {"experts": experts, "top": top}, "expert": {"ff": ff, "limit": limit}}


def yarn(factor, original=64, fast=32.0, slow=1.0):
    return {"factor": factor, "original": original, "fast": fast, "slow": slow}


def rotation(dims, base, scaling):
    r = {"base": base, "dims": dims}
    return {**r, "scaling": scaling} if scaling else r


def latent(heads, dim, rot, vdim, q_rank, kv_rank, mlp=None, scale=0.3, base=10000.0, scaling=yarn(4.0)):
    return {"type": "latent_attention", "mlp": mlp,
            "mixer": {"heads": heads, "dim": dim, "rot_dim": rot, "vdim": vdim, "q_rank": q_rank, "kv_rank": kv_rank, "scale": scale,
                      "rot": rotation(rot, base, scaling)}}


def attn(heads, kv_heads, dim, vdim, window, rot=None, mlp=None, scale=0.3, base=10000.0, scaling=yarn(8.0), kv_from=None):
    """rot: rotated coordinates (None: all of the head); window 0: no mask besides the causal one."""
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale, "mask": {"size": window} if window else None,
         "rot": rotation(dim if rot is None else rot, base, scaling) if rot != 0 else None}
    if kv_from is not None:
        m["kv_from"] = kv_from
    return {"type": "attention", "mixer": m, "mlp": mlp}


def light(heads, dim, vdim, decay=None, mlp=None):
    if decay is None:
        decay = [1.0 - 0.6 * 0.3 ** h for h in range(heads)]
    return {"type": "lightning", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "decay": list(decay)}, "mlp": mlp}


def config(width, vocab, layers, scale=2.5, eps=1e-5):
    return {"architecture": "Beronex", "width": width, "vocab": vocab, "layers": layers, "norm": {"eps": eps}, "embedding": {"scale": scale}}


CONFIGS = {
    # nothing divides anything: padded matrices, scalar loads, an odd vocabulary, parts of a head that begin anywhere
    "odd": config(100, 333, [latent(5, 20, 6, 28, 37, 45, dense(72)), attn(6, 2, 20, 36, 37, 12, moe(7, 3, 40)), light(3, 18, 23),
                             attn(6, 2, 20, 36, 64, 12, dense(50), 0.4, kv_from=1), light(2, 33, 30, None, moe(5, 2, 24, 0.8)),
                             latent(3, 33, 10, 12, 50, 30, moe(6, 6, 70)), attn(5, 5, 22, 10, 0, 22, None, 0.5, 300.0, None)], 1.7, 3e-6),
    # head sizes of the matrix-core kernels, two head tiles, more keys than a block; a wider mask on another layer's keys than on its own
    "wide": config(256, 512, [latent(18, 64, 64, 64, 192, 128, dense(320), 0.09, 500000.0), attn(34, 2, 128, 64, 90, 64, moe(20, 4, 96), 0.2),
                              light(4, 128, 128, [0.2, 0.9, 0.99, 0.9995], dense(192)), attn(34, 2, 128, 64, 130, 64, None, 0.1, kv_from=1),
                              latent(4, 128, 64, 128, 320, 512, moe(9, 2, 128), 0.07), light(3, 64, 32), attn(34, 2, 128, 64, 33, 64, dense(64), 0.3, kv_from=1)], 3.0),
    # everything is one (a latent of one number would be a sign)
    "ones": config(64, 96, [latent(1, 1, 2, 1, 2, 2, dense(1), 1.0, 2.0, yarn(1.0, 1, 1.0, 1.0)), attn(1, 1, 2, 1, 1, 2, moe(1, 1, 1, 1.0), 1.0),
                            light(1, 1, 2, [1.0], dense(1)), attn(1, 1, 2, 1, 1, 2, None, 1.0, kv_from=1), attn(2, 1, 2, 1, 3, 2, moe(2, 1, 1, 1.0), 1.0),
                            light(2, 1, 1, [0.0, 1.0])], 1.0),
    # head sizes beyond the matrix-core and chunk kernels
    "generic": config(128, 160, [latent(2, 100, 100, 72, 70, 600, dense(400), 0.1), attn(2, 1, 144, 200, 45, 100, moe(4, 2, 64), 0.1), light(2, 136, 72),
                                 attn(2, 1, 144, 200, 0, 100, None, 0.1, kv_from=1), light(1, 24, 300, [0.95], dense(40)),
                                 latent(3, 40, 12, 136, 36, 80, None, 0.2)]),
    # a wide row (several pieces per thread in the row kernels)
    "wide_row": config(2304, 96, [attn(3, 1, 48, 64, 40, 16, moe(3, 2, 48)), light(2, 32, 48, None, dense(96)), latent(2, 32, 16, 32, 48, 48)]),
}
