"""Plain, slow NumPy restatement of the Beronex decoder: one function per mechanism, float64 throughout.

What ``tests/test_beronex_oracle.py`` and ``tests/test_gpu_beronex.py`` compare with (never imported by the product).
A model is ``(cfg, w)``: the parsed ``config.json`` and a dict of float arrays under their checkpoint names.  Every
sequence is evaluated whole, without a cache: what portions, batches and caches must reproduce.
"""
from __future__ import annotations

import math
from typing import Dict, List, Optional

import numpy as np

F = np.float64


def sigmoid(z):
    return 0.5 * (1.0 + np.tanh(0.5 * z))


def silu(z):
    return z * sigmoid(z)


def gelu_tanh(z):
    return 0.5 * z * (1.0 + np.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def rms(x, eps):
    """x / sqrt(mean(x^2) + eps) over the last axis."""
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps)


def norm(x, w, eps):
    return rms(x, eps) * w


# ---- rotation ----------------------------------------------------------------------------------------------------------
def frequencies(rot: dict):
    """Angle per token of every pair, and the factor on cosines and sines."""
    n, base = rot["dims"], rot["base"]
    f = np.asarray([base ** (-2.0 * i / n) for i in range(n // 2)], F)
    s = rot.get("scaling")
    if not s:
        return f, 1.0

    def dim_of(turns):
        return n * math.log(s["original"] / (2.0 * math.pi * turns)) / (2.0 * math.log(base))
    lo, hi = max(math.floor(dim_of(s["fast"])), 0), min(math.ceil(dim_of(s["slow"])), n - 1)
    ramp = np.asarray([min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0) for i in range(n // 2)], F)
    return f / s["factor"] * ramp + f * (1.0 - ramp), 0.1 * math.log(s["factor"]) + 1.0


def rotate(x, positions, rot: dict, interleaved: bool):
    """x [n][..][dim]: the first ``dims`` coordinates turned in pairs, (2i, 2i + 1) or (i, i + dims / 2)."""
    n, y = rot["dims"], x.copy()
    f, gain = frequencies(rot)
    a = np.asarray(positions, F)[:, None] * f[None, :]
    a = a.reshape(a.shape[0], *([1] * (x.ndim - 2)), n // 2)
    first, second = (np.arange(0, n, 2), np.arange(1, n, 2)) if interleaved else (np.arange(n // 2), np.arange(n // 2, n))
    u, v, c, s = x[..., first], x[..., second], gain * np.cos(a), gain * np.sin(a)
    y[..., first], y[..., second] = u * c - v * s, v * c + u * s
    return y


# ---- attention ---------------------------------------------------------------------------------------------------------
def visible(n, size: Optional[int] = None):
    """[query][key]: causal, at most the last `size` tokens (itself included)."""
    i, j = np.arange(n)[:, None], np.arange(n)[None, :]
    return (j <= i) & (i - j < size) if size else j <= i


def softmax_rows(s, mask):
    s = np.where(mask, s, -np.inf)
    e = np.exp(s - s.max(axis=-1, keepdims=True))
    return e / e.sum(axis=-1, keepdims=True)


def rotated_rms(x, rot, eps):
    """Rotation, then the division by the root mean square over the head, without a weight."""
    if rot:
        x = rotate(x, np.arange(x.shape[0]), rot, True)
    return rms(x, eps)


def attention(h, w: Dict[str, np.ndarray], p: str, m: dict, eps: float, kv=None):
    """h [n][width] -> ([n][width], (keys, values)); ``kv``: another layer's keys and values."""
    n, H, G, d, e = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = rotated_rms((h @ w[p + "q"].T).reshape(n, H, d), m.get("rot"), eps)
    if kv is None:
        kv = rotated_rms((h @ w[p + "k"].T).reshape(n, G, d), m.get("rot"), eps), (h @ w[p + "v"].T).reshape(n, G, e)
    k, v = kv
    mask, o = visible(n, (m.get("mask") or {}).get("size")), np.zeros((n, H, e), F)
    for j in range(H):
        g = j // (H // G)
        o[:, j] = softmax_rows(q[:, j] @ k[:, g].T * m["scale"], mask) @ v[:, g]
    o = o * sigmoid(h @ w[p + "g"].T)[:, :, None]
    return o.reshape(n, H * e) @ w[p + "o"].T, kv


def latent_attention(h, w: Dict[str, np.ndarray], p: str, m: dict, eps: float):
    """h [n][width] -> [n][width]."""
    n, H, d, r, e, rank = h.shape[0], m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    q = (norm(h @ w[p + "dq"].T, w[p + "dq.norm"], eps) @ w[p + "uq"].T).reshape(n, H, d + r)
    z = h @ w[p + "dkv"].T
    c, kr = norm(z[:, :rank], w[p + "dkv.norm"], eps), z[:, rank:]
    qr, kr = rotate(q[:, :, d:], np.arange(n), m["rot"], False), rotate(kr, np.arange(n), m["rot"], False)
    k, v = (c @ w[p + "uk"].T).reshape(n, H, d), (c @ w[p + "uv"].T).reshape(n, H, e)
    mask, o = visible(n), np.zeros((n, H, e), F)
    for j in range(H):
        o[:, j] = softmax_rows((q[:, j, :d] @ k[:, j].T + qr[:, j] @ kr.T) * m["scale"], mask) @ v[:, j]
    return o.reshape(n, H * e) @ w[p + "o"].T


# ---- linear attention with a fixed decay ---------------------------------------------------------------------------------
def decayed_sums(q, k, v, decay, state=None):
    """q, k [n][H][d], v [n][H][e] -> (o [n][H][e], S [H][d][e])."""
    n, H, d = q.shape
    S = np.zeros((H, d, v.shape[2]), F) if state is None else state.copy()
    o, g = np.zeros_like(v), np.asarray(decay, F)[:, None, None]
    for t in range(n):
        S = g * S + k[t][:, :, None] * v[t][:, None, :]
        o[t] = (S * q[t][:, :, None]).sum(axis=1)
    return o, S


def lightning(h, w: Dict[str, np.ndarray], p: str, m: dict, eps: float):
    """h [n][width] -> [n][width]."""
    n, H, d, e = h.shape[0], m["heads"], m["dim"], m["vdim"]
    q, k, v = (silu(h @ w[p + t].T).reshape(n, H, x) for t, x in (("q", d), ("k", d), ("v", e)))
    o, _ = decayed_sums(q, k, v, m["decay"])
    return (norm(o.reshape(n, H * e), w[p + "norm"], eps) * sigmoid(h @ w[p + "g"].T)) @ w[p + "o"].T


# ---- feed-forward --------------------------------------------------------------------------------------------------------
def dense(h, w, p: str):
    return (gelu_tanh(h @ w[p + "gate"].T) * (h @ w[p + "up"].T)) @ w[p + "down"].T


def clamped_unit(g, u, limit):
    g, u = np.minimum(g, limit), np.clip(u, -limit, limit)
    return g * sigmoid(1.702 * g) * (u + 1.0)


def expert(h, w, p: str, limit):
    return clamped_unit(h @ w[p + "gate"].T, h @ w[p + "up"].T, limit) @ w[p + "down"].T


def route(z, top):
    """Router logits of one token -> [(expert, weight)]: the `top` largest, softmax over them."""
    chosen = np.argsort(-z, kind="stable")[:top]
    e = np.exp(z[chosen] - z[chosen].max())
    return list(zip(chosen.tolist(), e / e.sum()))


def route_margin(z, top) -> float:
    """Gap of logits between the last chosen expert and the first one left out."""
    s = np.sort(z)[::-1]
    return float(s[top - 1] - s[top]) if top < len(s) else np.inf


def moe(h, w, p: str, mlp: dict, margins=None):
    r = mlp["router"]
    z = h @ w[p + "router"].T + w[p + "router.b"]
    if margins is not None:
        margins.append([route_margin(t, r["top"]) for t in z])
    y = np.zeros_like(h)
    picks = [route(t, r["top"]) for t in z]
    for x in range(r["experts"]):
        at = [(t, g) for t, pk in enumerate(picks) for i, g in pk if i == x]
        if at:
            t, g = [a for a, _ in at], np.asarray([b for _, b in at])[:, None]
            y[t] += g * expert(h[t], w, f"{p}e{x}.", mlp["expert"]["limit"])
    return y


# ---- the stack -----------------------------------------------------------------------------------------------------------
def forward(cfg: dict, w: Dict[str, np.ndarray], tokens, layers_out: Optional[List[np.ndarray]] = None, margins: Optional[list] = None):
    """[n] ids -> logits [n][vocab].  ``margins`` receives a row of [n] router margins per expert layer."""
    w = {k: np.asarray(v, F) for k, v in w.items()} if not isinstance(w, _F64) else w
    eps, kept = cfg["norm"]["eps"], {}
    x = w["embed"][np.asarray(tokens, int)] * cfg["embedding"]["scale"]
    for i, layer in enumerate(cfg["layers"]):
        p, m, mlp = f"l{i}.", layer["mixer"], layer.get("mlp")
        h = norm(x, w[p + "norm1"], eps)
        if layer["type"] == "attention":
            y, kept[i] = attention(h, w, p + "mix.", m, eps, kept[m["kv_from"]] if m.get("kv_from") is not None else None)
        else:
            y = {"latent_attention": latent_attention, "lightning": lightning}[layer["type"]](h, w, p + "mix.", m, eps)
        x = x + norm(y, w[p + "norm1b"], eps)
        if mlp:
            h = norm(x, w[p + "norm2"], eps)
            y = moe(h, w, p + "mlp.", mlp, margins) if mlp["kind"] == "moe" else dense(h, w, p + "mlp.")
            x = x + norm(y, w[p + "norm2b"], eps)
        if layers_out is not None:
            layers_out.append(x.copy())
    return norm(x, w["final.norm"], eps) @ w["head"].T


class _F64(dict):
    """Marks weights that are float64 already (``as_f64``), so that repeated calls do not convert again."""


def as_f64(w) -> _F64:
    return _F64({k: np.asarray(getattr(v, "float", lambda: v)(), F) for k, v in w.items()})


def bf16_exact(a):
    """The nearest (half up) float32 values that bfloat16 holds."""
    u = np.ascontiguousarray(a, np.float32).view(np.uint32)
    return ((u + 0x8000) & np.uint32(0xFFFF0000)).view(np.float32)


def random_model(cfg: dict, seed: int = 0) -> Dict[str, np.ndarray]:
    """Random float32 weights (exactly representable in bfloat16) of the shapes ``cfg`` implies."""
    rng = np.random.default_rng(seed)
    w: Dict[str, np.ndarray] = {}
    W, V = cfg["width"], cfg["vocab"]

    def lin(name, n, k, s=1.0):
        w[name] = bf16_exact(rng.standard_normal((n, k)) * (s / np.sqrt(k)))

    def weight(name, n, s=1.0):
        w[name] = bf16_exact(s * (1.0 + 0.2 * rng.standard_normal(n)))

    w["embed"] = bf16_exact(rng.standard_normal((V, W)) / cfg["embedding"]["scale"])
    for i, layer in enumerate(cfg["layers"]):
        p, m, mlp = f"l{i}.", layer["mixer"], layer.get("mlp")
        vv = m["heads"] * m["vdim"]
        for sub in (1, 2) if mlp else (1,):
            weight(p + f"norm{sub}", W)
            weight(p + f"norm{sub}b", W, 0.7)
        p += "mix."
        if layer["type"] == "latent_attention":
            lin(p + "dq", m["q_rank"], W)
            weight(p + "dq.norm", m["q_rank"])
            lin(p + "uq", m["heads"] * (m["dim"] + m["rot_dim"]), m["q_rank"])
            lin(p + "dkv", m["kv_rank"] + m["rot_dim"], W)
            weight(p + "dkv.norm", m["kv_rank"])
            lin(p + "uk", m["heads"] * m["dim"], m["kv_rank"])
            lin(p + "uv", vv, m["kv_rank"])
        elif layer["type"] == "attention":
            lin(p + "q", m["heads"] * m["dim"], W)
            if m.get("kv_from") is None:
                lin(p + "k", m["kv_heads"] * m["dim"], W)
                lin(p + "v", m["kv_heads"] * m["vdim"], W)
            lin(p + "g", m["heads"], W, 2.0)
        else:
            for t, n in (("q", m["heads"] * m["dim"]), ("k", m["heads"] * m["dim"]), ("v", vv)):
                lin(p + t, n, W, 2.0)
            lin(p + "g", vv, W, 2.0)
            weight(p + "norm", vv)
        lin(p + "o", W, vv)
        p = f"l{i}.mlp."
        if mlp and mlp["kind"] == "moe":
            lin(p + "router", mlp["router"]["experts"], W, 2.0)
            w[p + "router.b"] = bf16_exact(0.5 * rng.standard_normal(mlp["router"]["experts"]))
            for x in range(mlp["router"]["experts"]):
                for t in ("gate", "up"):
                    lin(f"{p}e{x}.{t}", mlp["expert"]["ff"], W, 1.5)
                lin(f"{p}e{x}.down", W, mlp["expert"]["ff"])
        elif mlp:
            for t in ("gate", "up"):
                lin(p + t, mlp["ff"], W, 1.5)
            lin(p + "down", W, mlp["ff"])
    weight("final.norm", W)
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
