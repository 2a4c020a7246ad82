"""Small Temetar configurations for the tests: sizes with awkward remainders, every branch of the design, values that are 1."""
from __future__ import annotations


def attn(heads, kv_heads, dim, vdim, window, keep=0, rot=None, scale=0.3, ff=0, base=10000.0):
    """rot: rotated coordinates (None: all of the head); window 0: no mask besides the causal one."""
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale, "mask": {"size": window, "keep_first": keep} if window else None,
         "rot": {"base": base, "dims": dim if rot is None else rot} if rot != 0 else None}
    return {"type": "attention", "mixer": m, "mlp": {"ff": ff, "kind": "dense"} if ff else None}


def delta(heads, kv_heads, dim, vdim, conv, ff=0):
    return {"type": "channel_delta", "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": conv},
            "mlp": {"ff": ff, "kind": "dense"} if ff else None}


def config(width, vocab, layers, streams=3, loop=None, pair=(97, 31, 11), scale=3.0, mult=0.7, eps=1e-5):
    e = {"scale": scale}
    if pair:
        e["bigram"] = dict(zip(("buckets", "mul_prev", "mul_cur"), pair))
    return {"architecture": "Temetar", "width": width, "vocab": vocab, "layers": layers, "norm": {"eps": eps}, "streams": streams,
            "residual_mult": mult, "embedding": e, "loop": dict(zip(("start", "stop", "times"), loop)) if loop else None}


CONFIGS = {
    # nothing divides anything: padded matrices, scalar loads, an odd vocabulary, halves of a rotation that are no multiple of a load
    "odd": config(100, 333, [attn(6, 2, 20, 36, 37, 3, 12, ff=72), delta(6, 3, 20, 24, 3), attn(5, 5, 24, 12, 64, 0, 10),
                             delta(5, 5, 18, 9, 2, 50), attn(3, 1, 33, 30, 25, 7, 22, ff=130)], 3, (1, 4, 2), (61, 1000, 77), 2.5, 0.6, 3e-6),
    # head sizes of the matrix-core kernels, two head tiles, more key channels than a chunk has tokens
    "wide": config(256, 512, [attn(34, 2, 128, 64, 90, 5, 64, 0.09, 320), delta(4, 2, 128, 64, 4, 192), attn(8, 4, 64, 128, 130, 1, 32, 0.125),
                              delta(3, 3, 64, 128, 5), attn(4, 1, 32, 128, 70, 65, 8, 0.2, 64)], 4, (0, 2, 3)),
    # everything is one
    "ones": config(64, 96, [attn(1, 1, 2, 1, 1, 1, 2, 1.0, 1), delta(1, 1, 1, 1, 1, 1), attn(1, 1, 2, 1, 1, 0, 2, 1.0), attn(2, 1, 2, 1, 3, 1, 2, 1.0)],
                   1, (1, 2, 1), (1, 1, 1), 1.0, 1.0),
    # head sizes beyond the matrix-core and chunk kernels, no pairs, no loop, more streams than the kernels have cases for
    "generic": config(128, 160, [attn(2, 1, 144, 200, 45, 2, 100, 0.08, 700), delta(2, 1, 136, 72, 6, 64), attn(2, 2, 136, 100, 0, 0, 136, 0.1)],
                      7, None, None),
    # value heads wider than a thread row, no rotation, a loop over everything
    "wide_values": config(72, 112, [delta(2, 2, 24, 520, 3), attn(2, 1, 16, 24, 33, 5, 0), delta(1, 1, 512, 12, 2)], 2, (0, 3, 2)),
    # a wide row (several pieces per thread in the row kernels)
    "wide_row": config(2304, 96, [attn(3, 1, 48, 64, 40, 4, 16, ff=96), delta(2, 1, 32, 48, 3)], 5, (0, 1, 2)),
}
