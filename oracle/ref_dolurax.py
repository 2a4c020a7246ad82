"""Plain, slow NumPy restatement of the Dolurax decoder: one function per mechanism, float64 throughout.

What ``tests/test_dolurax_oracle.py`` and ``tests/test_gpu_dolurax.py`` compare with (never imported by the product).
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


def rms(x, eps):
    """x / sqrt(mean(x^2) + eps) over the last axis."""
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps)


def layer_norm(x, w, b, eps):
    d = x - np.mean(x, axis=-1, keepdims=True)
    return d / np.sqrt(np.mean(d * d, axis=-1, keepdims=True) + eps) * w + b


def cap(s, c):
    """Soft cap: c tanh(s / c); no cap when c is None."""
    return s if not c else c * np.tanh(s / c)


def slopes(H):
    """Per-head slope of the distance bias: 2^(-8/H), 2^(-16/H), .."""
    return 2.0 ** (-8.0 * (np.arange(H) + 1) / H)


def visible(n, chunk):
    """[query][key]: causal, within the query's own chunk of positions."""
    i, j = np.arange(n)[:, None], np.arange(n)[None, :]
    m = j <= i
    return m if not chunk else m & (i // chunk == j // chunk)


def scores(q, k, scale, softcap, slope):
    """q, k [n][dim] of one head -> [query][key], before the mask."""
    n = q.shape[0]
    dist = np.arange(n)[:, None] - np.arange(n)[None, :]
    return cap(q @ k.T * scale, softcap) - slope * dist


def softmax_rows(s, mask):
    s = np.where(mask, s, -np.inf)
    e = np.exp(s - s.max(axis=-1, keepdims=True))
    return e / e.sum(axis=-1, keepdims=True)


def mix_values(v, v_first, lam):
    """lam in front of the earlier layer's values of the same token."""
    return v if v_first is None else (1.0 - lam) * v + lam * v_first


def attention(h, w: Dict[str, np.ndarray], p: str, m: dict, eps: float, v_first=None):
    """h [n][width] -> ([n][width], the layer's own values [n][G * vdim])."""
    n, H, G, d, e = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = rms((h @ w[p + "q"].T).reshape(n, H, d), eps) * w[p + "q.norm"]
    k = rms((h @ w[p + "k"].T).reshape(n, G, d), eps) * w[p + "k.norm"]
    own = h @ w[p + "v"].T
    v = mix_values(own, v_first, float(w[p + "vmix"]) if v_first is not None else 0.0).reshape(n, G, e)
    mask, sl = visible(n, (m.get("mask") or {}).get("size")), slopes(H)
    o = np.zeros((n, H, e), F)
    for j in range(H):
        g = j // (H // G)
        o[:, j] = softmax_rows(scores(q[:, j], k[:, g], m["scale"], m.get("softcap"), sl[j]), mask) @ v[:, g]
    return (o.reshape(n, H * e) * sigmoid(h @ w[p + "g"].T)) @ w[p + "o"].T, own


def expert(h, w, p: str):
    return (silu(h @ w[p + "gate"].T) * (h @ w[p + "up"].T)) @ w[p + "down"].T


def route(z, r: dict):
    """Router logits of one token -> [(expert, weight)]: the `top` largest among the best groups, weights normalised."""
    E = len(z)
    s = np.exp(z - z.max())
    s = s / s.sum()
    grp = r.get("groups") or {"count": 1, "keep": 1}
    size = E // grp["count"]
    best = np.argsort([-s[g * size:(g + 1) * size].max() for g in range(grp["count"])], kind="stable")[:grp["keep"]]
    allowed = [e for e in range(E) if e // size in set(best.tolist())]
    chosen = sorted(allowed, key=lambda e: -s[e])[:r["top"]]
    total = sum(s[e] for e in chosen) + 1e-20
    return [(e, s[e] / total) for e in chosen]


def route_margin(z, r: dict) -> float:
    """How far the choice is from another one: the smallest gap of logits, last chosen against first left out, groups and experts."""
    E, grp = len(z), r.get("groups") or {"count": 1, "keep": 1}
    size = E // grp["count"]
    best = np.asarray([z[g * size:(g + 1) * size].max() for g in range(grp["count"])])
    order = np.argsort(-best, kind="stable")
    gap = best[order[grp["keep"] - 1]] - best[order[grp["keep"]]] if grp["keep"] < grp["count"] else np.inf
    allowed = np.sort(np.concatenate([z[g * size:(g + 1) * size] for g in order[:grp["keep"]]]))[::-1]
    return float(min(gap, allowed[r["top"] - 1] - allowed[r["top"]] if r["top"] < len(allowed) else np.inf))


def moe(h, w, p: str, mlp: dict, margins=None):
    z = h @ w[p + "router"].T
    if margins is not None:
        margins.append([route_margin(t, mlp["router"]) for t in z])
    y = np.zeros_like(h)
    picks = [route(z[t], mlp["router"]) for t in range(h.shape[0])]
    for e in range(mlp["router"]["experts"]):
        at = [(t, g) for t, pk in enumerate(picks) for x, g in pk if x == e]
        if at:
            t, g = [a for a, _ in at], np.asarray([b for _, b in at])[:, None]
            y[t] += g * expert(h[t], w, f"{p}e{e}.")
    return y + expert(h, w, p + "shared.") if mlp.get("shared") else y


def forward(cfg: dict, w: Dict[str, np.ndarray], tokens, layers_out: Optional[List[np.ndarray]] = None, margins: Optional[list] = None):
    """[n] ids -> logits [n][vocab].  ``margins`` receives a row of [n] router margins per expert layer."""
    w = {k: np.asarray(v, F) for k, v in w.items()} if not isinstance(w, _F64) else w
    toks, eps = np.asarray(tokens, int), cfg["norm"]["eps"]
    x, v_first = w["embed"][toks], None
    for i, layer in enumerate(cfg["layers"]):
        p, m = f"l{i}.", layer["mixer"]
        y, own = attention(x, w, p + "mix.", m, eps, v_first if m.get("v_mix") else None)
        if m.get("v_mix") and v_first is None:
            v_first = own
        x = x + layer_norm(y, w[p + "norm1"], w[p + "norm1.b"], eps)
        if layer.get("mlp"):
            x = x + layer_norm(moe(x, w, p + "mlp.", layer["mlp"], margins), w[p + "norm2"], w[p + "norm2.b"], eps)
        if layers_out is not None:
            layers_out.append(x.copy())
    lg = layer_norm(x, w["final.norm"], w["final.norm.b"], eps) @ w["head"].T * cfg.get("logit_scale", 1.0)
    return cap(lg, cfg.get("logit_softcap"))


class _F64(dict):
    """Marks weights that are float64 already (``as_f64``), so that repeated calls do not convert again."""


def as_f64(w) -> _F64:
    return _F64({k: np.asarray(getattr(v, "float", lambda: v)(), F) for k, v in w.items()})


def random_model(cfg: dict, seed: int = 0) -> Dict[str, np.ndarray]:
    """Random float32 weights (exactly representable in bfloat16) of the shapes ``cfg`` implies."""
    rng = np.random.default_rng(seed)
    w: Dict[str, np.ndarray] = {}
    W, V = cfg["width"], cfg["vocab"]

    def bf(a):
        u = np.ascontiguousarray(a, np.float32).view(np.uint32)
        return ((u + 0x8000) & np.uint32(0xFFFF0000)).view(np.float32)

    def lin(name, n, k, s=1.0):
        w[name] = bf(rng.standard_normal((n, k)) * (s / np.sqrt(k)))

    def norm(name, s=1.0):
        w[name] = bf(s * (1.0 + 0.2 * rng.standard_normal(W)))
        w[name + ".b"] = bf(0.1 * rng.standard_normal(W))

    def ffn(name, ff):
        lin(name + "gate", ff, W)
        lin(name + "up", ff, W)
        lin(name + "down", W, ff)

    w["embed"] = bf(rng.standard_normal((V, W)))
    for i, layer in enumerate(cfg["layers"]):
        p, m, mlp = f"l{i}.", layer["mixer"], layer.get("mlp")
        norm(p + "norm1", 0.7)
        for t, c in (("q", m["heads"] * m["dim"]), ("k", m["kv_heads"] * m["dim"]), ("v", m["kv_heads"] * m["vdim"]),
                     ("g", m["heads"] * m["vdim"])):
            lin(p + "mix." + t, c, W)
        w[p + "mix.q.norm"] = bf(1.5 * (1.0 + 0.2 * rng.standard_normal(m["dim"])))
        w[p + "mix.k.norm"] = bf(1.5 * (1.0 + 0.2 * rng.standard_normal(m["dim"])))
        if m.get("v_mix"):
            w[p + "mix.vmix"] = bf(rng.uniform(0.2, 0.8, 1)).reshape(())
        lin(p + "mix.o", W, m["heads"] * m["vdim"])
        if mlp:
            norm(p + "norm2", 0.7)
            lin(p + "mlp.router", mlp["router"]["experts"], W, 2.0)
            for e in range(mlp["router"]["experts"]):
                ffn(f"{p}mlp.e{e}.", mlp["expert"]["ff"])
            if mlp.get("shared"):
                ffn(p + "mlp.shared.", mlp["shared"]["ff"])
    norm("final.norm")
    lin("head", V, W, 4.0)
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
