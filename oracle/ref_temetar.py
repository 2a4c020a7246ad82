"""Plain, slow NumPy restatement of the Temetar decoder: one function per mechanism, float64 throughout.

What ``tests/test_temetar_oracle.py`` and ``tests/test_gpu_temetar.py`` compare with (never imported by the product).
A model is ``(cfg, w)``: the parsed ``config.json`` and a dict of float arrays under their checkpoint names.  Every
sequence is evaluated whole, without a cache: what portions, batches and caches must reproduce.
"""
from __future__ import annotations

from typing import Dict, List, Optional

import numpy as np

F = np.float64


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def silu(z):
    return z * sigmoid(z)


def softplus(z):
    return np.logaddexp(0.0, z)


def rms(x, eps):
    """x / sqrt(mean(x^2) + eps) over the last axis."""
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps)


def norm(x, w, eps):
    """RMS norm whose stored weight is the distance from one."""
    return rms(x, eps) * (1.0 + w)


# ---- embedding ---------------------------------------------------------------------------------------------------------
def bigram_rows(tokens, buckets, mul_prev, mul_cur):
    """Row of the pair table for every token; the first token of a sequence has a row of its own behind the buckets."""
    t = [int(x) for x in tokens]
    return [buckets if i == 0 else (t[i - 1] * mul_prev + t[i] * mul_cur) % buckets for i in range(len(t))]


def embedding(cfg: dict, w, tokens):
    e = cfg["embedding"]
    x = w["embed"][np.asarray(tokens, int)] * e.get("scale", 1.0)
    b = e.get("bigram")
    return x + w["bigram"][bigram_rows(tokens, b["buckets"], b["mul_prev"], b["mul_cur"])] if b else x


# ---- attention ---------------------------------------------------------------------------------------------------------
def rotate(x, positions, base, dims):
    """x [n][heads][dim]: coordinate i < dims / 2 and coordinate i + dims / 2 turned by position * base^(-2i/dims)."""
    half, y = dims // 2, x.copy()
    for i in range(half):
        a = np.asarray(positions, F)[:, None] * base ** (-2.0 * i / dims)
        u, v = x[:, :, i], x[:, :, i + half]
        y[:, :, i], y[:, :, i + half] = u * np.cos(a) - v * np.sin(a), v * np.cos(a) + u * np.sin(a)
    return y


def visible(n, mask):
    """[query][key]: causal, the last `size` tokens (itself included) and the first `keep_first` of the sequence."""
    i, j = np.arange(n)[:, None], np.arange(n)[None, :]
    m = j <= i
    if mask and mask.get("size"):
        m = m & ((i - j < mask["size"]) | (j < mask.get("keep_first", 0)))
    return m


def softmax_sink(s, mask, sink):
    """Rows of weights; the denominator has one more term, exp(sink)."""
    s = np.where(mask, s, -np.inf)
    top = np.maximum(s.max(axis=-1, keepdims=True), sink)
    e = np.exp(s - top)
    return e / (e.sum(axis=-1, keepdims=True) + np.exp(sink - top))


def attention(h, w: Dict[str, np.ndarray], p: str, m: dict, eps: float):
    """h [n][width] -> [n][width]."""
    n, H, G, d, e = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = rms((h @ w[p + "q"].T).reshape(n, H, d), eps) * w[p + "q.norm"]
    k = rms((h @ w[p + "k"].T).reshape(n, G, d), eps) * w[p + "k.norm"]
    v = (h @ w[p + "v"].T).reshape(n, G, e)
    r = m.get("rot")
    if r:
        q, k = (rotate(x, np.arange(n), r["base"], r["dims"]) for x in (q, k))
    mask, o = visible(n, m.get("mask")), np.zeros((n, H, e), F)
    for j in range(H):
        g = j // (H // G)
        o[:, j] = softmax_sink(q[:, j] @ k[:, g].T * m["scale"], mask, w[p + "sink"][j]) @ v[:, g]
    return o.reshape(n, H * e) @ w[p + "o"].T


# ---- delta rule with a decay per channel ---------------------------------------------------------------------------------
def short_conv(x, taps):
    """x [n][C], taps [C][K]: y[t] = sum_j taps[:, K-1-j] x[t-j], zeros before the start."""
    n, k = x.shape[0], taps.shape[1]
    y = np.zeros_like(x)
    for j in range(min(k, n)):
        y[j:] += x[: n - j] * taps[:, k - 1 - j]
    return y


def unit(x):
    return x / np.sqrt(np.sum(x * x, axis=-1, keepdims=True) + 1e-6)


def channel_delta_rule(q, k, v, beta, log_g, state: Optional[np.ndarray] = None):
    """q, k, log_g [n][H][d] (per value head), v [n][H][e], beta [n][H] -> (o [n][H][e], S [H][d][e])."""
    n, H, d = q.shape
    S = np.zeros((H, d, v.shape[2]), F) if state is None else state.copy()
    o = np.zeros_like(v)
    for t in range(n):
        for h in range(H):
            S[h] *= np.exp(log_g[t, h])[:, None]
            u = beta[t, h] * (v[t, h] - S[h].T @ k[t, h])
            S[h] += np.outer(k[t, h], u)
            o[t, h] = S[h].T @ q[t, h]
    return o, S


def channel_delta(h, w: Dict[str, np.ndarray], p: str, m: dict, eps: float):
    """h [n][width] (normed) -> [n][width]."""
    n, H, G, d, e = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = silu(short_conv(h @ w[p + "q"].T, w[p + "q.conv"])).reshape(n, G, d)
    k = silu(short_conv(h @ w[p + "k"].T, w[p + "k.conv"])).reshape(n, G, d)
    v = silu(short_conv(h @ w[p + "v"].T, w[p + "v.conv"])).reshape(n, H, e)
    q, k = unit(q) * d ** -0.5, unit(k)
    src = [j // (H // G) for j in range(H)]
    beta = sigmoid(h @ w[p + "b"].T)
    step = softplus(h @ w[p + "a1"].T @ w[p + "a2"].T + w[p + "dt_bias"]).reshape(n, H, d)
    log_g = -np.exp(w[p + "A_log"])[None, :, None] * step
    o, _ = channel_delta_rule(q[:, src], k[:, src], v, beta, log_g)
    gate = sigmoid(h @ w[p + "g1"].T @ w[p + "g2"].T).reshape(n, H, e)
    o = rms(o, eps) * w[p + "norm"] * gate
    return o.reshape(n, H * e) @ w[p + "o"].T


# ---- the stack ---------------------------------------------------------------------------------------------------------
def feed_forward(h, w, p: str):
    return (silu(h @ w[p + "gate"].T) * (h @ w[p + "up"].T)) @ w[p + "down"].T


def hyper_read(xs, w_in):
    """xs [streams][n][width] -> what the sublayer reads."""
    return sum(w_in[s] * xs[s] for s in range(len(xs)))


def hyper_write(xs, y, mix, w_out, mult):
    """Every stream from all the old ones (mix [from][to]) and the sublayer's output."""
    return np.stack([sum(mix[s, t] * xs[s] for s in range(len(xs))) + mult * w_out[t] * y for t in range(len(xs))])


def layer_runs(cfg: dict) -> List[int]:
    """Layer numbers in the order in which they run."""
    n, loop = len(cfg["layers"]), cfg.get("loop")
    if not loop:
        return list(range(n))
    a, b = loop["start"], loop["stop"]
    return list(range(a)) + list(range(a, b)) * loop["times"] + list(range(b, n))


def forward(cfg: dict, w: Dict[str, np.ndarray], tokens, layers_out: Optional[List[np.ndarray]] = None):
    """[n] ids -> logits [n][vocab]."""
    w = {k: np.asarray(v, F) for k, v in w.items()} if not isinstance(w, _F64) else w
    eps, mult = cfg["norm"]["eps"], cfg.get("residual_mult", 1.0)
    xs = np.stack([embedding(cfg, w, tokens)] * cfg["streams"])
    for i in layer_runs(cfg):
        layer, p = cfg["layers"][i], f"l{i}."
        for sub in (1, 2) if layer.get("mlp") else (1,):
            hc = p + f"hc{sub}."
            h = norm(hyper_read(xs, w[hc + "in"]), w[p + f"norm{sub}"], eps)
            if sub == 2:
                y = feed_forward(h, w, p + "mlp.")
            else:
                y = {"attention": attention, "channel_delta": channel_delta}[layer["type"]](h, w, p + "mix.", layer["mixer"], eps)
            xs = hyper_write(xs, y, w[hc + "mix"], w[hc + "out"], mult)
        if layers_out is not None:
            layers_out.append(xs.sum(axis=0))
    return norm(xs.sum(axis=0), w["final.norm"], eps) @ w["head"].T


class _F64(dict):
    """Marks weights that are float64 already (``as_f64``), so that repeated calls do not convert again."""


def as_f64(w) -> _F64:
    return _F64({k: np.asarray(getattr(v, "float", lambda: v)(), F) for k, v in w.items()})


def random_model(cfg: dict, seed: int = 0, decay_rank: int = 5, gate_rank: int = 7) -> Dict[str, np.ndarray]:
    """Random float32 weights (exactly representable in bfloat16) of the shapes ``cfg`` implies; the inner sizes of the low-rank
    maps, which no configuration names, are arguments."""
    rng = np.random.default_rng(seed)
    w: Dict[str, np.ndarray] = {}
    W, V, S = cfg["width"], cfg["vocab"], cfg["streams"]

    def bf(a):
        u = np.ascontiguousarray(a, np.float32).view(np.uint32)
        return ((u + 0x8000) & np.uint32(0xFFFF0000)).view(np.float32)

    def lin(name, n, k, s=1.0):
        w[name] = bf(rng.standard_normal((n, k)) * (s / np.sqrt(k)))

    scale = cfg["embedding"].get("scale", 1.0)
    w["embed"] = bf(rng.standard_normal((V, W)) / scale)
    pair = cfg["embedding"].get("bigram")
    if pair:
        w["bigram"] = bf(0.7 * rng.standard_normal((pair["buckets"] + 1, W)))
    for i, layer in enumerate(cfg["layers"]):
        p, m, mlp = f"l{i}.", layer["mixer"], layer.get("mlp")
        for sub in (1, 2) if mlp else (1,):
            w[p + f"norm{sub}"] = bf(0.2 * rng.standard_normal(W))
            w[p + f"hc{sub}.in"] = bf((1.0 + 0.3 * rng.standard_normal(S)) / S)
            w[p + f"hc{sub}.out"] = bf(0.6 + 0.3 * rng.standard_normal(S))
            w[p + f"hc{sub}.mix"] = bf(0.9 * np.eye(S) + 0.1 * rng.standard_normal((S, S)))
        if layer["type"] == "channel_delta":
            H, d, qk, vv = m["heads"], m["dim"], m["kv_heads"] * m["dim"], m["heads"] * m["vdim"]
            for t, c in (("q", qk), ("k", qk), ("v", vv)):
                lin(p + "mix." + t, c, W)
                w[p + f"mix.{t}.conv"] = bf(rng.standard_normal((c, m["conv"])) * 0.7 / np.sqrt(m["conv"]) + 0.7 * (np.arange(m["conv"]) == m["conv"] - 1))
            lin(p + "mix.b", H, W)
            w[p + "mix.A_log"] = bf(np.log(rng.uniform(0.05, 1.5, H)))
            w[p + "mix.dt_bias"] = bf(rng.uniform(-4.0, 0.5, H * d))
            w[p + "mix.norm"] = bf(1.0 + 0.2 * rng.standard_normal(m["vdim"]))
            lin(p + "mix.a1", decay_rank, W)
            lin(p + "mix.a2", H * d, decay_rank)
            lin(p + "mix.g1", gate_rank, W)
            lin(p + "mix.g2", vv, gate_rank, 2.0)
            lin(p + "mix.o", W, vv, 0.7)
        else:
            for t, c in (("q", m["heads"] * m["dim"]), ("k", m["kv_heads"] * m["dim"]), ("v", m["kv_heads"] * m["vdim"])):
                lin(p + "mix." + t, c, W)
            w[p + "mix.q.norm"] = bf(1.0 + 0.2 * rng.standard_normal(m["dim"]))
            w[p + "mix.k.norm"] = bf(1.0 + 0.2 * rng.standard_normal(m["dim"]))
            w[p + "mix.sink"] = bf(1.0 + rng.standard_normal(m["heads"]))
            lin(p + "mix.o", W, m["heads"] * m["vdim"])
        if mlp:
            lin(p + "mlp.gate", mlp["ff"], W)
            lin(p + "mlp.up", mlp["ff"], W)
            lin(p + "mlp.down", W, mlp["ff"])
    w["final.norm"] = bf(0.2 * rng.standard_normal(W))
    lin("head", V, W, 2.0)
    return w


def save_model(path, cfg: dict, w: Dict[str, np.ndarray], dtype: str = "bfloat16") -> None:
    """config.json + model.safetensors."""
    import json
    from pathlib import Path

    import torch
    from safetensors.torch import save_file

    path = Path(path)
    path.mkdir(parents=True, exist_ok=True)
    (path / "config.json").write_text(json.dumps(cfg))
    save_file({k: torch.from_numpy(np.asarray(v, np.float32).copy()).to(getattr(torch, dtype)) for k, v in w.items()},
              str(path / "model.safetensors"))
