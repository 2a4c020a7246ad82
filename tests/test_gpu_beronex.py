"""Beronex on the GPU against the plain implementation (oracle/ref_beronex.py): whole prompts, portions, decoding, batches,
reused rows and blocks, each mechanism alone, greedy generation through the framework's own entry points."""
import json
import subprocess
from pathlib import Path

import numpy as np
import pytest

from oracle import ref_beronex as R
from tests.beronex_models import CONFIGS, attn, config, dense, latent, light, moe, yarn
from tests.gpu_helpers import serve_and_compare

pytestmark = pytest.mark.gpu
ROOT = Path(__file__).resolve().parent.parent
# error = rms over the vocabulary of the centred difference / rms of the centred logits
# (rounding the operands and results of the plain implementation's products to bfloat16 gives up to 0.041 at positions that count)
TOL = {"float32": 2e-5, "bfloat16": 0.06, "float16": 0.008}


def err(got, want, scale=None):
    """scale: the logits whose rms counts (default: these positions')"""
    d = got - want
    d = d - d.mean(-1, keepdims=True)
    s = want if scale is None else scale
    s = s - s.mean(-1, keepdims=True)
    return np.sqrt((d * d).mean(-1)) / np.sqrt((s * s).mean())


def plain(cfg, w, t, layers=None):
    """-> logits, and which positions no router was undecided about: 16-bit inputs may flip a choice between two experts with nearly
    equal logits, there and (through attention and state) a little behind it."""
    margins = []
    lg = R.forward(cfg, w, t, layers, margins)
    return lg, np.min(margins, axis=0) > 0.1 if margins else np.ones(len(t), bool)


def worst(e, clear, dtype, name=""):
    """The figure that is held against TOL.  A norm of one or two numbers is nearly their signs: where those are close to zero, the last
    bits decide them."""
    if dtype == "float32":
        return e.max() / (5.0 if name == "ones" else 1.0)
    e = e[clear]
    return np.quantile(e, 0.85 if name == "ones" else (1.0 if clear.all() else 0.95))


@pytest.fixture(scope="module")
def bank(tmp_path_factory):
    """name, dtype -> (cfg, float64 weights, loaded model); one checkpoint per name, kept for the module."""
    from mlx_parallm_amd.utils import load_model

    root, kept, loaded = tmp_path_factory.mktemp("beronex"), {}, {}

    def get(name, dtype="float32", cfg=None, edit=None, seed=1):
        if name not in kept:
            c = cfg or CONFIGS[name]
            w = R.random_model(c, seed)
            if edit:
                edit(w)
            w = {k: R.bf16_exact(v) for k, v in w.items()}
            R.save_model(root / name, c, w)
            kept[name] = (c, R.as_f64(w))
        if (name, dtype) not in loaded:
            loaded[name, dtype] = load_model(root / name, dtype=dtype, max_positions=2048)
        return (*kept[name], loaded[name, dtype])

    get.root = root
    yield get
    for m in loaded.values():
        m.engine.close()


def tokens(cfg, n, seed=0):
    return np.random.default_rng(seed).integers(0, cfg["vocab"], n).astype(np.int32)


def run_portions(eng, kv, row, toks, sizes):
    """Feed toks to one row in the given portions; -> logits of every position."""
    out, at = [], 0
    for s in sizes:
        part = toks[at:at + s]
        if len(part) == 0:
            break
        out.append(eng.forward_segments(kv, [row], [part], range(len(part))))
        at += len(part)
    assert at == len(toks)
    return np.concatenate(out)


def check_portions(m, t, want, dtype, all_sizes, block=16, factor=1.0, name="", clear=None):
    clear = np.ones(len(t), bool) if clear is None else clear
    for sizes in all_sizes:
        kv = m.engine.new_paged_kv(1, block_tokens=block, n_blocks=len(t) // block + 2, max_tokens_per_row=(len(t) + block) // block * block)
        e = err(run_portions(m.engine, kv, 0, t, sizes), want)
        kv.close()
        assert worst(e, clear, dtype, name) < factor * TOL[dtype], (sizes[:4], int(e.argmax()), e.max())


@pytest.mark.parametrize("dtype", ["float32", "bfloat16", "float16"])
@pytest.mark.parametrize("name", list(CONFIGS))
def test_whole_prompt_and_residual_stream(bank, name, dtype):
    cfg, w, m = bank(name, dtype)
    for n in (41, 150):                   # (short: the experts' weights are streamed; long: the grouped tile GEMM)
        t, layers = tokens(cfg, n), []
        want, clear = plain(cfg, w, t, layers)
        kv = m.engine.new_kv(1, capacity=n, kv_dtype="model")
        cap = m.engine.capture_residual(n)
        got = m.engine.forward_segments(kv, [0], [t], range(n))
        m.engine.capture_residual(0)
        kv.close()
        assert len(cap) == len(layers)
        for i, (g, x) in enumerate(zip(cap, layers)):
            e = np.sqrt(((g - x) ** 2).mean(-1)) / np.sqrt((x * x).mean())
            assert worst(e, clear, dtype, name) < TOL[dtype], (n, i, e.max())
        e = err(got, want)
        assert worst(e, clear, dtype, name) < TOL[dtype], (n, e.max())


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", list(CONFIGS))
def test_portions_and_decoding_agree_with_the_whole(bank, name, dtype):
    cfg, w, m = bank(name, dtype)
    t = tokens(cfg, 150, 2)
    want, clear = plain(cfg, w, t)
    check_portions(m, t, want, dtype, ([1] * 150, [2] * 75, [3, 2, 1, 5, 64, 2, 1, 1, 65, 6], [63, 1, 1, 64, 2, 19], [130] + [1] * 20), name=name, clear=clear)


def one_sublayer(keep):
    """Zero what the other sublayer adds to the stream."""
    def edit(w):
        for k in w:
            if keep != "mixer" and k.endswith("norm1b") or keep != "feed_forward" and k.endswith("norm2b"):
                w[k] = w[k] * 0
    return edit


KINDS = {"attention": attn(3, 3, 16, 24, 29, 6, dense(40)), "latent": latent(3, 16, 4, 24, 20, 28, moe(4, 2, 16)), "lightning": light(4, 16, 24, None, dense(40))}


@pytest.mark.parametrize("kind", list(KINDS))
@pytest.mark.parametrize("keep", ["mixer", "feed_forward", "none"])
def test_each_sublayer_alone(bank, keep, kind):
    cfg, w, m = bank(f"alone_{kind}_{keep}", "float32", config(72, 112, [KINDS[kind]]), one_sublayer(keep))
    t = tokens(cfg, 70, 3)
    check_portions(m, t, R.forward(cfg, w, t), "float32", ([37, 1, 1, 31], [70]))


BASE = dict(heads=4, kv_heads=2, dim=24, vdim=32, window=0, rot=0, scale=0.4)
ATTENTION = {"plain": {}, "rotation": {"rot": None, "scaling": None}, "stretched": {"rot": None}, "partial": {"rot": 10, "scaling": yarn(64.0)},
             "two_coordinates": {"rot": 2, "scaling": yarn(64.0)}, "step": {"rot": 16, "base": 37.5, "scaling": yarn(2.0, 20, 1.0, 1.0)},
             "all_stretched": {"rot": 24, "scaling": yarn(3.0, 2, 8.0, 4.0)}, "long_original": {"rot": 24, "scaling": yarn(3.0, 10**6)},
             "window": {"window": 19}, "window_of_one": {"window": 1}, "window_of_two": {"window": 2, "rot": 8}, "one_head_group": {"kv_heads": 1, "rot": 8},
             "every_head_its_own": {"kv_heads": 4, "window": 30, "rot": 20}, "one_head": {"heads": 1, "kv_heads": 1, "rot": 4},
             "padded_head": {"dim": 40, "vdim": 72, "rot": 36}, "odd_head": {"dim": 21, "vdim": 19, "rot": 14}}


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", list(ATTENTION))
def test_each_attention_mechanism_alone(bank, name, dtype):
    mix = attn(**{**BASE, **ATTENTION[name]})
    cfg, w, m = bank(f"att_{name}", dtype, config(64, 96, [mix, mix]))
    t = tokens(cfg, 100, 4)
    check_portions(m, t, R.forward(cfg, w, t), dtype, ([100], [18, 1, 1, 20, 60], [1] * 100))


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_norm_stands_behind_a_partial_rotation(bank, dtype):
    """A strong gain on a few of the coordinates: a mean square taken in front of it would be far off."""
    mix = attn(4, 2, 32, 32, 0, 8, None, 1.0, 100.0, yarn(1e6))

    def edit(w):
        w["l0.norm1b"] *= 4
        for k in ("q", "k"):                              # the rotated coordinates are the large ones
            w[f"l0.mix.{k}"].reshape(-1, 32, 64)[:, :8] *= 2
    cfg, w, m = bank("partial", dtype, config(64, 96, [mix]), edit)
    t = tokens(cfg, 120, 5)
    want, after = R.forward(cfg, w, t), R.rotated_rms
    R.rotated_rms = lambda x, rot, eps: R.rotate(R.rms(x, eps), np.arange(len(x)), rot, True)
    try:
        assert (err(R.forward(cfg, w, t), want) > 3 * TOL[dtype]).mean() > 0.2
    finally:
        R.rotated_rms = after
    check_portions(m, t, want, dtype, ([120], [64] + [1] * 56))


LATENT = {"plain": (3, 16, 8, 24, 20, 28), "one_head": (1, 16, 8, 16, 8, 16), "many_heads": (33, 16, 16, 16, 48, 64), "large_rotated_part": (4, 16, 64, 32, 40, 48),
          "two_rotated": (4, 32, 2, 32, 40, 48), "odd": (3, 21, 14, 11, 13, 27), "wide_key": (2, 128, 64, 64, 64, 96), "wide_key_and_value": (3, 100, 40, 128, 64, 200),
          "rank_512": (2, 64, 64, 64, 64, 512), "rank_beyond": (2, 32, 32, 32, 64, 560), "exact_row": (4, 32, 16, 32, 64, 112)}


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", list(LATENT))
def test_each_latent_form_alone(bank, name, dtype):
    size = LATENT[name][1] + LATENT[name][2]
    one = latent(*LATENT[name], None, 1.5 * size ** -0.5)
    two = latent(*LATENT[name], None, 2.5 * size ** -0.5, 200.0, yarn(16.0, 300) if name != "odd" else None)
    cfg, w, m = bank(f"latent_{name}", dtype, config(64, 96, [one, two]))
    t = tokens(cfg, 330, 6)
    check_portions(m, t, R.forward(cfg, w, t), dtype, ([330], [290] + [1] * 40, [18, 1, 1, 20, 60, 2, 228]))
    t = t[:70]
    check_portions(m, t, R.forward(cfg, w, t), dtype, ([1] * 70,))


LIGHT = {"plain": (4, 16, 24), "one_head": (1, 32, 32), "odd": (3, 15, 11), "padded": (2, 36, 20), "full": (4, 128, 128), "wide_value": (2, 20, 100),
         "wide_key": (2, 100, 20), "beyond_the_chunks": (2, 132, 16), "values_beyond": (2, 16, 150), "very_wide": (1, 500, 8)}


@pytest.mark.parametrize("dtype", ["float32", "bfloat16", "float16"])
@pytest.mark.parametrize("name", list(LIGHT))
def test_each_lightning_form_alone(bank, name, dtype):
    """Portions of less and more than a tile of queries and a chunk, and one by one."""
    cfg, w, m = bank(f"light_{name}", dtype, config(64, 96, [light(*LIGHT[name]), light(*LIGHT[name])]))
    t = tokens(cfg, 300, 6)
    check_portions(m, t, R.forward(cfg, w, t), dtype, ([300], [64, 64, 172], [127, 1, 128, 2, 42], [129, 130, 1, 1, 39], [65, 63, 1, 66, 105]))
    t = t[:100]
    check_portions(m, t, R.forward(cfg, w, t), dtype, ([2] * 50, [1] * 100, [3, 97]))


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_ends_of_the_decays_range(bank, dtype):
    """Heads that forget everything, nothing, most of it within a chunk, and next to nothing over thousands of tokens."""
    one = light(6, 32, 32, [0.0, 1.0, 1e-30, 0.5, 0.9999, 1.0 - 1e-12])
    cfg, w, m = bank("decays", dtype, config(64, 96, [one]))
    t = tokens(cfg, 700, 7)
    check_portions(m, t, R.forward(cfg, w, t), dtype, ([700], [350, 1, 1, 348], [20] * 35), 64)
    cfg, w, m = bank("forgets", dtype, config(64, 96, [light(2, 32, 32, [0.0, 0.0])]))
    assert err(R.forward(cfg, w, t[:50])[49:], R.forward(cfg, w, t[49:50])).max() < 1e-12
    check_portions(m, t[:50], R.forward(cfg, w, t[:50]), dtype, ([50], [20, 1, 29]), 64)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_a_single_early_token_is_carried_through_the_state(bank, dtype):
    """One token writes a hundred times as much as the others: a state that is lost, cut at a chunk or decayed once too often shows
    hundreds of tokens later."""
    def edit(w):
        w["l0.norm1b"] *= 4
        w["embed"][60:, :32] += 3.0
        for k in ("k", "v"):
            w[f"l0.mix.{k}"][:, :32] += 0.12
    cfg, w, m = bank("early", dtype, config(64, 64, [light(2, 32, 32, [0.997, 1.0])]), edit)
    t = tokens(cfg, 520, 8) % 60
    without, factor = R.forward(cfg, w, t), 1.0 if dtype == "float32" else 0.2        # (16-bit operands make 0.006 here)
    for at in (0, 63, 64, 127, 128, 200):
        u = t.copy()
        u[at] = 61
        want = R.forward(cfg, w, u)
        assert (err(without, want)[at:at + 250] > 3 * factor * TOL[dtype]).mean() > 0.9
        check_portions(m, u, want, dtype, ([520], [at + 1, 519 - at], [at + 1] + [1] * 40 + [479 - at], [64, 2, 62, 129, 263]), 64, factor)


def test_chunks_of_many_tokens(bank):
    """A call long enough for the larger chunks, unequal segments beside a decoded token."""
    cfg, w, m = bank("many", "bfloat16", config(64, 64, [light(2, 32, 32, [0.98, 0.9995]), light(1, 64, 128, [0.999])]))
    m = __import__("mlx_parallm_amd.utils", fromlist=["x"]).load_model(bank.root / "many", dtype="bfloat16", max_positions=8192)
    a, b, c = tokens(cfg, 7300, 1), tokens(cfg, 901, 2), tokens(cfg, 40, 3)
    wa, wb, wc = (R.forward(cfg, w, t) for t in (a, b, c))
    kv = m.engine.new_paged_kv(3, block_tokens=64, n_blocks=140, max_tokens_per_row=7360)
    assert err(m.engine.forward_segments(kv, [1], [c[:39]], [38]), wc[38:39], wc).max() < TOL["bfloat16"]
    got = m.engine.forward_segments(kv, [0, 1, 2], [a, c[39:], b], range(8202))
    for g, x, s in ((got[:7300], wa, wa), (got[7300:7301], wc[39:], wc), (got[7301:], wb, wb)):
        assert err(g, x, s).max() < TOL["bfloat16"]
    assert err(m.engine.forward_segments(kv, [2], [b[:1]], [0]), R.forward(cfg, w, np.append(b, b[0]))[-1:], wb).max() < TOL["bfloat16"]
    kv.close()
    m.engine.close()


MOE = {"few": (5, 2, 24), "one_of_many": (33, 1, 16), "all": (6, 6, 40), "single": (1, 1, 20), "many": (70, 8, 16), "wide": (8, 3, 200), "narrow": (12, 4, 1)}


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", list(MOE))
def test_each_expert_form_alone(bank, name, dtype):
    """Limits that many units reach, biases that decide choices; few and many tokens."""
    one = light(1, 8, 8, [0.5], moe(*MOE[name], 0.7))

    def edit(w):
        w["l0.norm1b"] *= 0.1
        w["l0.mlp.router.b"] *= 3
    cfg, w, m = bank(f"moe_{name}", dtype, config(72, 112, [one]), edit)
    t = tokens(cfg, 300, 9)
    want, clear = plain(cfg, w, t)
    for change in ({"l0.mlp.router.b": 0}, None):          # both show in the logits
        if change is None:
            moved = R.forward({**cfg, "layers": [{**one, "mlp": moe(*MOE[name], 50.0)}]}, w, t)
        else:
            moved = R.forward(cfg, R.as_f64({**w, **{k: w[k] * f for k, f in change.items()}}), t)
        if change is None or MOE[name][1] > 1 and MOE[name][0] > 1:
            assert (err(moved, want) > 2 * TOL[dtype]).mean() > 0.1, change
    check_portions(m, t, want, dtype, ([300], [63, 64, 65, 1, 1, 106], [16, 17, 32, 33, 202]), 64, clear=clear)


def test_large_tiles_of_the_experts(bank):
    """Enough tokens per expert for the large tile of the grouped matrix product."""
    cfg, w, m = bank("tiles", "bfloat16", config(128, 64, [light(1, 8, 8, [0.5], moe(4, 2, 128, 0.7))]))
    t = tokens(cfg, 1500, 10)
    want, clear = plain(cfg, w, t)
    check_portions(m, t, want, "bfloat16", ([1500],), 64, clear=clear)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16", "float16"])
@pytest.mark.parametrize("width,ff", [(64, 24), (72, 333), (256, 512)])
def test_gated_gelu_of_few_and_many_rows(bank, width, ff, dtype):
    def edit(w):
        w["l0.mlp.gate"] *= 2
        w["l0.norm1b"] *= 0.1
    cfg, w, m = bank(f"gelu_{width}", dtype, config(width, 112, [light(1, 8, 8, [0.5], dense(ff))]), edit)
    t = tokens(cfg, 700, 11)
    check_portions(m, t, R.forward(cfg, w, t), dtype, ([700], [1, 1, 9, 17, 33, 65, 130, 444]), 64)


SHARED = {"wider": 90, "narrower": 7, "everything": 0, "one": 1}


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("dim", [32, 160])
@pytest.mark.parametrize("name", list(SHARED))
def test_keys_and_values_of_another_layer(bank, name, dim, dtype):
    """Masks wider and narrower than that layer's; several layers read the same one; a layer with its own in between."""
    f = dim ** -0.5
    own = attn(6, 2, dim, 24, 30, 12, None, 1.5 * f)
    cfg = config(64, 96, [own, attn(6, 2, dim, 24, SHARED[name], 12, None, 2.5 * f, kv_from=0), attn(4, 4, 16, 16, 11), light(2, 8, 8),
                          attn(6, 2, dim, 24, 45, 12, None, f, kv_from=0)])
    cfg, w, m = bank(f"shared_{name}_{dim}", dtype, cfg)
    t = tokens(cfg, 200, 12)
    check_portions(m, t, R.forward(cfg, w, t), dtype, ([200], [130] + [1] * 70, [16, 1, 16, 2, 31, 134], [2] * 100))


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_batches_of_unequal_requests_against_each_alone(bank, dtype):
    cfg, w, m = bank("odd", dtype)
    eng = m.engine
    reqs = [tokens(cfg, n, 10 + n) for n in (90, 1, 33, 64, 7)]
    ref = [plain(cfg, w, t) for t in reqs]
    kv = eng.new_paged_kv(5, block_tokens=16, n_blocks=24, max_tokens_per_row=96)
    at, step, rng, es = [0] * 5, 0, np.random.default_rng(4), [[] for _ in reqs]
    while any(a < len(t) for a, t in zip(at, reqs)):
        rows = [i for i in rng.permutation(5) if at[i] < len(reqs[i]) and (rng.random() < 0.8 or step > 60)]
        if not rows:
            continue
        parts = [reqs[i][at[i]:at[i] + int(rng.choice([1, 1, 1, 2, 5, 17, 40]))] for i in rows]
        got = eng.forward_segments(kv, rows, parts, range(sum(map(len, parts))))
        j = 0
        for i, p in zip(rows, parts):
            es[i].append(err(got[j:j + len(p)], ref[i][0][at[i]:at[i] + len(p)], ref[0][0]))
            j += len(p)
            at[i] += len(p)
        step += 1
    kv.close()
    e, clear = np.concatenate([x for r in es for x in r]), np.concatenate([c for _, c in ref])
    assert worst(e, clear, dtype) < TOL[dtype]


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_rows_and_blocks_are_used_again(bank, dtype):
    cfg, w, m = bank("odd", dtype)
    eng = m.engine
    kv = eng.new_paged_kv(2, block_tokens=16, n_blocks=9, max_tokens_per_row=96)     # eight blocks for both rows
    es, cs = [], []
    for k in range(6):
        a, b = tokens(cfg, 70 - 9 * k, 30 + k), tokens(cfg, 20 + 3 * k, 60 + k)
        ra = k % 2
        for t, row, sizes in ((a, ra, [40, 1, 2, 100]), (b, 1 - ra, [1, 1, 100])):
            want, clear = plain(cfg, w, t)
            es.append(err(run_portions(eng, kv, row, t, sizes), want))
            cs.append(clear)
        kv.reset_row(0)
        kv.reset_row(1)
        assert kv.stats()["free_blocks"] == 8
    kv.close()
    assert worst(np.concatenate(es), np.concatenate(cs), dtype) < TOL[dtype]


def peaky(w, proj_q, proj_k, n_special, V):
    """Keys that stand out: the last n_special tokens of the vocabulary score far above everything else where they are seen (plain
    query and key projections without rotation)."""
    rng = np.random.default_rng(9)
    e, k, q = w["embed"], w[proj_k], w[proj_q]
    w["l0.norm1"][:] = 1.0
    d = rng.standard_normal(e.shape[1]).astype(np.float32)
    e[V - n_special:] += 3 * d                               # special tokens share a direction ..
    u = np.sign(rng.standard_normal(k.shape[0])).astype(np.float32)
    k += 3 * np.outer(u, d).astype(np.float32) / e.shape[1]  # .. that points every key of theirs along u,
    rep, half = q.shape[0] // k.shape[0], k.shape[0] // 2
    uq = np.concatenate([np.tile(u[g * half:(g + 1) * half], rep) for g in range(2)])
    q += 2 * np.outer(uq, np.ones(e.shape[1])).astype(np.float32) / np.sqrt(e.shape[1])     # and the queries' common part as well
    e += 0.7


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name,dim", [("matrix_cores", 32), ("generic", 160)])
def test_single_keys_stand_out_at_the_edges_of_the_windows(bank, name, dim, dtype):
    """A few tokens whose keys outscore everything: a key that is missing, or seen one token too long, changes the logits completely.
    The second layer looks at the first one's keys through a window of its own."""
    size, other, n = 100, 70, 420
    own = attn(4, 2, dim, 24, size, 0, None, 30.0 / dim)
    lent = attn(4, 2, dim, 24, other, 0, None, 30.0 / dim, kv_from=0)

    def edit(w):
        peaky(w, "l0.mix.q", "l0.mix.k", 4, 64)
        w["l1.mix.q"][:] = w["l0.mix.q"]
        w["l0.norm1b"] *= 3
        w["l1.norm1"][:] = 1.0
        w["l1.norm1b"] *= 3
        w["l0.mix.g"] *= 0.2
        w["l1.mix.g"] *= 0.2
    cfg, w, m = bank(f"peaky_{name}", dtype, config(96, 64, [own, lent], 1.0), edit)
    t = tokens(cfg, n, 5) % 60
    for i, p in enumerate((63, 192, 319)):                   # ends of blocks, alone in their windows
        t[p] = 60 + i
    want = R.forward(cfg, w, t)

    def moved(a, b):
        layers = [{**x, "mixer": {**x["mixer"], "mask": {"size": s}}} for x, s in ((own, a), (lent, b))]
        return err(R.forward({**cfg, "layers": layers}, w, t), want)
    for a, b in ((size - 1, other), (size + 1, other), (size, other - 1), (size, other + 1)):
        assert (moved(a, b) > 4 * TOL[dtype]).sum() >= 2, (a, b)
    check_portions(m, t, want, dtype, ([n], [162, 1, 1, 1, 126, 1, 1, 1, 126], [33] * 13, [4, 2] + [1] * 414, [99, 2, 98, 2, 98, 1, 1, 119]), 64, 2.0)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name,size", [("matrix_cores", (4, 32, 16, 24, 64, 64)), ("wide", (3, 128, 64, 64, 64, 96)), ("generic", (2, 160, 40, 24, 64, 64))])
def test_single_far_keys_stand_out_in_the_latent_attention(bank, name, size, dtype):
    """Queries that look for one token of the past by its latent, at pages' and blocks' borders and hundreds of tokens away."""
    H, d, r, e, qr, rank = size

    def edit(w):
        rng = np.random.default_rng(3)
        emb = w["embed"]
        a, u = rng.standard_normal(emb.shape[1]).astype(np.float32), np.sign(rng.standard_normal((H, d))).astype(np.float32)
        emb[60:] += 4 * a
        emb += 0.8
        w["l0.norm1"][:] = 1.0
        w["l0.norm1b"] *= 4
        w["l0.mix.dq"][0] = 0.3
        w["l0.mix.dkv"][0] = 0.5 * a / np.sqrt(emb.shape[1])
        w["l0.mix.uq"].reshape(H, d + r, qr)[:, :d, 0] = 2 * u
        w["l0.mix.uk"].reshape(H, d, rank)[:, :, 0] = 2 * u
        w["l0.mix.dkv.norm"][:] = 1.0
        w["l0.mix.dq.norm"][:] = 1.0
    cfg, w, m = bank(f"far_{name}", dtype, config(96, 64, [latent(*size, None, 1.0 / d)], 1.0), edit)
    t = tokens(cfg, 450, 5) % 60
    calm = R.forward(cfg, w, t)
    for p in (0, 1, 63, 64, 127, 130):
        x = t.copy()
        x[p] = 61
        want = R.forward(cfg, w, x)
        assert (err(calm, want)[p + 1:] > 4 * TOL[dtype]).mean() > 0.9, p
        check_portions(m, x, want, dtype, ([450], [p + 1, 449 - p], [300] + [1] * 150, [64, 1, 1, 2, 130, 252]), 64, 1.5)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_rotated_parts_find_distances(bank, dtype):
    """Queries and keys that consist of the rotated part alone: scores depend on the distance, on every frequency and on the gain."""
    def edit(w):
        w["l0.norm1b"] *= 4
        w["l0.norm1"][:] = 1.0
        w["embed"] += 1.5
        q = w["l0.mix.uq"].reshape(2, 24, 16)
        q[:, :8] = 0
        q[:, 8:] *= 3
        w["l0.mix.dkv"][32:] += 0.1
        w["l0.mix.dq"] += 0.1
    base = latent(2, 8, 16, 16, 16, 32, None, 0.3, 50.0, yarn(4.0, 100, 8.0, 1.0))
    cfg, w, m = bank("distances", dtype, config(64, 96, [base], 1.0), edit)
    t = tokens(cfg, 260, 6)
    want = R.forward(cfg, w, t)
    for s in (None, yarn(4.0, 100, 8.0, 3.0), yarn(5.0, 100, 8.0, 1.0), yarn(4.0, 130, 8.0, 1.0)):
        mix = {**base, "mixer": {**base["mixer"], "rot": {"base": 50.0, "dims": 16, **({"scaling": s} if s else {})}}}
        assert (err(R.forward({**cfg, "layers": [mix]}, w, t), want) > TOL["float32"] * 50).mean() > 0.3, s
    check_portions(m, t, want, dtype, ([260], [100, 1, 1, 158], [220] + [1] * 40), 64)


def test_long_decoding_behind_a_long_prompt(bank):
    """700 tokens at once, then 330 one by one, beside a row that does the opposite: positions, windows, states and blocks far out; a
    window longer than one split of the decode attention."""
    cfg = config(64, 96, [attn(4, 2, 32, 32, 700, 16, dense(48)), light(2, 32, 32, [0.99, 0.9999]), latent(4, 32, 16, 32, 48, 48), attn(4, 2, 32, 32, 333, 16, kv_from=0),
                          attn(16, 1, 64, 64, 0, 32, None, 0.2)])
    cfg, w, m = bank("long", "bfloat16", cfg)
    a, b = tokens(cfg, 1030, 40), tokens(cfg, 1030, 41)
    wa, wb = R.forward(cfg, w, a), R.forward(cfg, w, b)
    kv = m.engine.new_paged_kv(2, block_tokens=64, n_blocks=36, max_tokens_per_row=1088)
    eng = m.engine
    ea, eb = [err(eng.forward_segments(kv, [0], [a[:700]], range(700)), wa[:700])], []
    for i in range(330):
        got = eng.forward_segments(kv, [1, 0], [b[i:i + 1], a[700 + i:701 + i]], [0, 1])
        eb.append(err(got[:1], wb[i:i + 1], wb))
        ea.append(err(got[1:], wa[700 + i:701 + i], wa))
    eb.append(err(eng.forward_segments(kv, [1], [b[330:]], range(700)), wb[330:]))
    kv.close()
    for e in (np.concatenate(ea), np.concatenate(eb)):
        assert e.max() < TOL["bfloat16"]


def test_growth_of_a_contiguous_cache_keeps_everything(bank):
    cfg, w, m = bank("odd")
    t = tokens(cfg, 120, 9)
    kv = m.engine.new_kv(2, capacity=16, kv_dtype="model", step=16)
    got = run_portions(m.engine, kv, 1, t, [10, 1, 30, 1, 1, 77])
    assert kv.capacity >= 120 and err(got, R.forward(cfg, w, t)).max() < TOL["float32"]
    kv.close()


def test_prefix_blocks_are_shared_unless_a_layer_is_recurrent(bank):
    cfg, w, m = bank("prefix", cfg=config(64, 96, [attn(2, 1, 16, 16, 30, 8, dense(24)), latent(2, 16, 8, 8, 12, 20), attn(2, 1, 16, 16, 50, 8, kv_from=0)]))
    a = tokens(cfg, 70, 50)
    b = np.concatenate([a[:50], tokens(cfg, 30, 51)]).astype(np.int32)
    kv = m.engine.new_paged_kv(2, block_tokens=16, n_blocks=14, max_tokens_per_row=96)
    run_portions(m.engine, kv, 0, a, [70])
    kv.prefix_publish(0, a)
    assert kv.prefix_attach(1, b) == 48
    got = m.engine.forward_segments(kv, [1], [b[48:]], range(len(b) - 48))
    assert err(got, R.forward(cfg, w, b)[48:]).max() < TOL["float32"]
    kv.close()
    cfg, w, m = bank("odd")
    kv = m.engine.new_paged_kv(2, block_tokens=16, n_blocks=14, max_tokens_per_row=96)
    run_portions(m.engine, kv, 0, a, [70])
    kv.prefix_publish(0, a)
    assert kv.prefix_attach(1, b) == 0
    kv.close()


def greedy(cfg, w, prompt, n):
    t = list(prompt)
    for _ in range(n):
        t.append(int(R.forward(cfg, w, t)[-1].argmax()))
    return t[len(prompt):]


def test_greedy_generation_of_ragged_prompts(bank):
    from mlx_parallm_amd import utils

    cfg, w, m = bank("odd")
    prompts = [tokens(cfg, n, 70 + n).tolist() for n in (9, 1, 30)]
    got = [[] for _ in prompts]
    for _, (ids, _p) in utils._take(utils.generate_step(prompts, m), 12):
        for g, i in zip(got, ids[:, 0]):
            g.append(int(i))
    assert got == [greedy(cfg, w, p, 12) for p in prompts]
    # a rectangular batch and the callable model
    same = np.asarray([p[:1] for p in prompts])
    ids = [x[0][:, 0].tolist() for _, x in utils._take(utils.generate_step(same, m), 5)]
    assert np.array_equal(np.asarray(ids).T, [greedy(cfg, w, p, 5) for p in same.tolist()])
    assert err(m(np.asarray([prompts[0]]))[0], R.forward(cfg, w, prompts[0])).max() < TOL["float32"]


class _Tok:
    """Ids joined by blanks, no end token."""

    eos_token_id = -1
    eos_token = pad_token = "<e>"
    pad_token_id = 0

    def decode(self, ids, **kw):
        return "".join(f"{int(i)} " for i in ids)


def test_scheduler_admits_chunks_and_reuses_rows(bank):
    import threading

    from mlx_parallm_amd.server.scheduler import ContinuousScheduler

    cfg, w, m = bank("odd")
    sched = ContinuousScheduler(m, _Tok(), max_slots=2, kv_dtype="model", chunk_tokens=16, kv_blocks=9)
    sched.start()
    prompts = [tokens(cfg, n, 90 + n) for n in (50, 3, 21, 70, 2)]
    done, seqs = [threading.Event() for _ in prompts], []
    for i, p in enumerate(prompts):
        seqs.append(sched.submit(p, 8, 0.0, 1.0, lambda s, d, r, i=i: done[i].set() if r else None))
    assert all(d.wait(60) for d in done)
    got = [s.generated for s in seqs]
    assert sched.mixed_steps > 0 and sched.max_rows_seen == 2
    sched.stop()
    assert got == [greedy(cfg, w, p.tolist(), 8) for p in prompts]


def test_scores_of_given_tokens(bank):
    cfg, w, m = bank("odd")
    t = tokens(cfg, 20, 11)
    lg = R.forward(cfg, w, t)
    want = (lg - np.log(np.exp(lg).sum(-1, keepdims=True)))[np.arange(19), t[1:]]
    kv = m.engine.new_kv(1, capacity=32, kv_dtype="model")
    got = m.engine.score_tokens(kv, t[None, :-1], t[None, 1:])["logprobs"][0]
    kv.close()
    assert np.allclose(got, want, atol=1e-3)


def test_wrong_use_is_refused(bank, tmp_path):
    from mlx_parallm_amd.engine import Engine
    from mlx_parallm_amd.utils import load_model

    cfg, w, m = bank("odd", "bfloat16")
    with pytest.raises(NotImplementedError):
        m.engine.new_kv(1, capacity=16, kv_dtype="float32")
    one = attn(2, 1, 16, 16, 8)
    bad = [[attn(3, 2, 16, 16, 8)], [attn(2, 1, 16, 16, 8, 7)], [attn(2, 1, 16, 16, 8, 18)], [attn(2, 1, 16, 16, -3)], [one, attn(2, 2, 16, 16, 8, kv_from=0)],
           [one, attn(2, 1, 16, 8, 8, kv_from=0)], [attn(2, 1, 16, 16, 8, kv_from=0)], [one, light(1, 8, 8), attn(2, 1, 16, 16, 8, kv_from=1)],
           [one, attn(2, 1, 16, 16, 8, kv_from=0), attn(2, 1, 16, 16, 8, kv_from=1)], [light(2, 8, 8, [0.5, 1.5])], [light(1, 8, 8, [-0.1])],
           [dict(one, mlp=moe(4, 5, 8))], [dict(one, mlp=moe(4, 2, 8, 0.0))]]
    for layers in bad:
        with pytest.raises(ValueError):
            Engine({**config(64, 96, layers), "model_type": "beronex"})
    for layers in ([attn(1, 1, 600, 16, 8)], [light(1, 600, 8)], [latent(1, 8, 8, 8, 8, 1020)]):
        with pytest.raises(NotImplementedError):
            Engine({**config(64, 96, layers), "model_type": "beronex"})
    few = config(64, 96, [attn(2, 1, 16, 16, 8, None, moe(2, 1, 24)), light(1, 8, 8, [0.5], dense(16)), latent(1, 8, 8, 8, 8, 8)])
    for gone in ("l0.norm1b", "l1.norm2b", "l0.mix.g", "l0.mlp.router.b", "l0.mlp.e1.up", "l1.mix.norm", "l2.mix.uq", "l2.mix.dq.norm", "l2.mix.uv"):
        R.save_model(tmp_path / gone, few, {k: v for k, v in R.random_model(few).items() if k != gone})
        with pytest.raises(FileNotFoundError, match=gone.replace(".uv", ".u")):
            load_model(tmp_path / gone)


def test_trace_replay_program(bank, tmp_path):
    cfg, w, _ = bank("odd")
    a, b = tokens(cfg, 70, 20), tokens(cfg, 9, 21)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": a[:60].tolist(), "want": [59, 3]}], "end": []},
             {"step": 1, "entries": [{"id": "b", "tokens": b.tolist(), "want": []}, {"id": "a", "tokens": a[60:61].tolist(), "want": [0]}],
              "end": ["b"]},
             {"step": 2, "entries": [{"id": "a", "tokens": a[61:].tolist(), "want": [8]}, {"id": "c", "tokens": b.tolist(), "want": [8]}],
              "end": ["a", "c"]}]
    res = subprocess.run([str(ROOT / "bin" / "trace_run"), "--model", str(bank.root / "odd"), "--dtype", "float32", "--out", str(tmp_path),
                          "--max-tokens", "192"], input="\n".join(map(json.dumps, steps)) + "\n", capture_output=True, text=True, timeout=100)
    assert res.returncode == 0, res.stderr[-2000:]
    assert [x for x in res.stdout.splitlines() if x.startswith("done")] == ["done 0", "done 1", "done 2"]
    wa, wb = R.forward(cfg, w, a), R.forward(cfg, w, b)
    for step, want in ((0, wa[[59, 3]]), (1, wa[[60]]), (2, np.stack([wa[69], wb[8]]))):
        got = np.fromfile(tmp_path / f"{step}.f32", "<f4").reshape(want.shape)
        assert err(got, want).max() < TOL["float32"]


@pytest.mark.parametrize("scheduler", ["default", "continuous"])
def test_server_program_completes_and_streams(tmp_path, scheduler):
    from mlx_parallm_amd.tiny_model import build_byte_tokenizer

    cfg = config(72, build_byte_tokenizer(tmp_path), [attn(4, 2, 20, 24, 33, 12, moe(4, 2, 24)), light(3, 16, 16), latent(2, 16, 8, 16, 20, 24, dense(40)),
                                                      attn(4, 2, 20, 24, 50, 12, kv_from=0)])
    serve_and_compare(tmp_path, scheduler, R, cfg, greedy)
