"""Temetar on the GPU against the plain implementation (oracle/ref_temetar.py): whole prompts, portions, decoding, batches,
reused rows and blocks, each mechanism alone, greedy generation through the framework's own entry points."""
import json
import subprocess
from pathlib import Path

import numpy as np
import pytest

from oracle import ref_temetar as R
from tests.gpu_helpers import serve_and_compare
from tests.temetar_models import CONFIGS, attn, config, delta

pytestmark = pytest.mark.gpu
ROOT = Path(__file__).resolve().parent.parent
# error = rms over the vocabulary of the centred difference / rms of the centred logits
# (rounding the operands of the plain implementation's products to bfloat16 gives up to 0.02 for these configurations)
TOL = {"float32": 2e-5, "bfloat16": 0.04, "float16": 0.005}


def err(got, want, scale=None):
    """scale: the logits whose rms counts (default: these positions')"""
    d = got - want
    d = d - d.mean(-1, keepdims=True)
    s = want if scale is None else scale
    s = s - s.mean(-1, keepdims=True)
    return np.sqrt((d * d).mean(-1)) / np.sqrt((s * s).mean())


def worst(e, name, dtype):
    """The figure that is held against TOL.  A unit vector of one number is its sign: where that is nearly zero, 16-bit inputs decide it."""
    return np.quantile(e, 0.85) if name == "ones" and dtype != "float32" else e.max()


@pytest.fixture(scope="module")
def bank(tmp_path_factory):
    """name, dtype -> (cfg, float64 weights, loaded model); one checkpoint per name, kept for the module."""
    from mlx_parallm_amd.utils import load_model

    root, plain, loaded = tmp_path_factory.mktemp("temetar"), {}, {}

    def get(name, dtype="float32", cfg=None, edit=None, seed=1, ranks=(5, 7)):
        if name not in plain:
            c = cfg or CONFIGS[name]
            w = R.random_model(c, seed, *ranks)
            if edit:
                edit(w)
            R.save_model(root / name, c, w)
            plain[name] = (c, R.as_f64(w))
        if (name, dtype) not in loaded:
            loaded[name, dtype] = load_model(root / name, dtype=dtype, max_positions=2048)
        return (*plain[name], loaded[name, dtype])

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


def check_portions(m, t, want, dtype, all_sizes, block=16, factor=1.0, name=""):
    for sizes in all_sizes:
        kv = m.engine.new_paged_kv(1, block_tokens=block, n_blocks=len(t) // block + 2, max_tokens_per_row=(len(t) + block) // block * block)
        e = err(run_portions(m.engine, kv, 0, t, sizes), want)
        kv.close()
        assert worst(e, name, dtype) < factor * TOL[dtype], (sizes[:4], int(e.argmax()), e.max())


@pytest.mark.parametrize("dtype", ["float32", "bfloat16", "float16"])
@pytest.mark.parametrize("name", list(CONFIGS))
def test_whole_prompt_and_residual_stream(bank, name, dtype):
    cfg, w, m = bank(name, dtype)
    for n in (41, 150):
        t, layers = tokens(cfg, n), []
        want = R.forward(cfg, w, t, layers)
        kv = m.engine.new_kv(1, capacity=n, kv_dtype="model")
        cap = m.engine.capture_residual(n)
        got = m.engine.forward_segments(kv, [0], [t], range(n))
        m.engine.capture_residual(0)
        kv.close()
        assert len(cap) == len(layers)
        for i, (g, x) in enumerate(zip(cap, layers)):
            e = np.sqrt(((g - x) ** 2).mean(-1)) / np.sqrt((x * x).mean())
            assert worst(e, name, dtype) < TOL[dtype], (n, i, e.max())
        e = err(got, want)
        assert worst(e, name, dtype) < TOL[dtype], (n, e.max())


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", list(CONFIGS))
def test_portions_and_decoding_agree_with_the_whole(bank, name, dtype):
    cfg, w, m = bank(name, dtype)
    t = tokens(cfg, 150, 2)
    check_portions(m, t, R.forward(cfg, w, t), dtype, ([1] * 150, [2] * 75, [3, 2, 1, 5, 64, 2, 1, 1, 65, 6], [63, 1, 1, 64, 2, 19], [130] + [1] * 20), name=name)


def one_sublayer(keep):
    """Nothing of the other kind of sublayer reaches the streams."""
    def edit(w):
        for k in w:
            if keep != "mixer" and k.endswith("hc1.out") or keep != "feed_forward" and k.endswith("hc2.out"):
                w[k] = w[k] * 0
    return edit


@pytest.mark.parametrize("kind", ["attention", "delta"])
@pytest.mark.parametrize("keep", ["mixer", "feed_forward", "none"])
def test_each_sublayer_alone(bank, keep, kind):
    one = attn(3, 3, 16, 24, 29, 2, 6, ff=40) if kind == "attention" else delta(4, 2, 16, 24, 3, 40)
    cfg, w, m = bank(f"alone_{kind}_{keep}", "float32", config(72, 112, [one]), one_sublayer(keep))
    t = tokens(cfg, 70, 3)
    check_portions(m, t, R.forward(cfg, w, t), "float32", ([37, 1, 1, 31], [70]))


BASE = dict(heads=4, kv_heads=2, dim=24, vdim=32, window=0, rot=0, scale=0.4)
ATTENTION = {"plain": {}, "rotation": {"rot": None}, "partial_rotation": {"rot": 10}, "two_coordinates": {"rot": 2}, "other_base": {"rot": 16, "base": 37.5},
             "window": {"window": 19}, "window_of_one": {"window": 1}, "window_of_one_with_kept": {"window": 1, "keep": 2},
             "kept": {"window": 19, "keep": 3}, "more_kept_than_window": {"window": 5, "keep": 40}, "kept_block": {"window": 16, "keep": 64},
             "one_head_group": {"kv_heads": 1, "rot": 8}, "every_head_its_own": {"kv_heads": 4, "window": 30, "keep": 1}}


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", list(ATTENTION))
def test_each_attention_mechanism_alone(bank, name, dtype):
    mix = attn(**{**BASE, **ATTENTION[name]})
    cfg, w, m = bank(f"mech_{name}", dtype, config(64, 96, [mix, mix], 1, None, None))
    t = tokens(cfg, 100, 4)
    check_portions(m, t, R.forward(cfg, w, t), dtype, ([100], [18, 1, 1, 20, 60], [1] * 100))


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("sink", [-40.0, 0.0, 6.0, 200.0])
def test_sinks_of_every_size(bank, sink, dtype):
    """A sink far below the scores does nothing, one far above takes all the weight; several splits in decoding."""
    mix = attn(4, 2, 32, 32, 0, rot=16, scale=0.2)

    def edit(w):
        w["l0.mix.sink"][:] = sink
        w["l0.hc1.out"] *= 4
    cfg, w, m = bank(f"sink_{sink}", dtype, config(64, 96, [mix], 2, None, None), edit)
    t = tokens(cfg, 600, 5)
    check_portions(m, t, R.forward(cfg, w, t), dtype, ([600], [560] + [1] * 40), 64)


DELTA = {"one_tap": (4, 2, 16, 24, 1), "six_taps": (4, 2, 16, 24, 6), "groups_of_three": (6, 2, 32, 16, 4), "odd_sizes": (3, 3, 15, 11, 3),
         "padded": (2, 1, 36, 20, 2), "two_pieces": (2, 2, 100, 36, 3), "full": (4, 2, 128, 128, 4), "too_wide_for_chunks": (2, 1, 132, 16, 3)}


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", list(DELTA))
def test_each_delta_form_alone(bank, name, dtype):
    """Sizes of the chunk kernels and beyond; portions of less and more than a chunk, short ones token by token."""
    one = delta(*DELTA[name])
    cfg, w, m = bank(f"delta_{name}", dtype, config(64, 96, [one, one], 2, None, None), ranks=(3, 70))
    t = tokens(cfg, 140, 6)
    check_portions(m, t, R.forward(cfg, w, t), dtype, ([140], [64, 64, 12], [65, 1, 63, 2, 9], [24, 23, 25, 2, 66], [2] * 70, [1] * 140))


@pytest.mark.parametrize("dtype", ["bfloat16", "float16"])
@pytest.mark.parametrize("ranks", [(5, 7), (100, 128), (70, 190), (130, 192), (256, 250), (300, 270)])
def test_low_rank_maps_of_many_rows(bank, ranks, dtype):
    """Inner sizes of every form of the kernel for many rows, unequal ones and larger ones, beside one-token segments."""
    cfg, w, m = bank(f"ranks_{ranks}", dtype, config(72, 96, [delta(3, 1, 20, 36, 3), delta(5, 5, 36, 17, 2)], 2, None, None), ranks=ranks)
    t = tokens(cfg, 340, 12)
    check_portions(m, t, R.forward(cfg, w, t), dtype, ([340], [260, 1, 1, 78]), 64)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("decay", ["none", "strong", "extreme", "mixed", "steps"])
def test_ends_of_the_decays_range(bank, decay, dtype):
    """Channels that forget nothing, everything, e^-1000s in a chunk, and both kinds beside each other in one key."""
    def edit(w):
        for i in range(2):
            p, rng = f"l{i}.mix.", np.random.default_rng(i)
            b = w[p + "dt_bias"]
            if decay == "none":
                b[:] = -40.0
            elif decay in ("strong", "extreme"):
                b[:] = 3.0
                w[p + "A_log"][:] = 0.5 if decay == "strong" else 5.0
            elif decay == "mixed":
                b[:] = rng.choice([-40.0, -3.0, 2.0, 30.0], len(b))
                w[p + "A_log"][:] = 1.0
            else:                                         # decays that jump between tokens: nothing, then e^-10s
                w[p + "a2"] *= 30
                w[p + "A_log"][:] = 0.0
            for k in ("dt_bias", "A_log", "a2"):
                u = np.ascontiguousarray(w[p + k], np.float32).view(np.uint32)
                w[p + k] = ((u + 0x8000) & np.uint32(0xFFFF0000)).view(np.float32)
    one = delta(4, 2, 64, 32, 3)
    cfg, w, m = bank(f"decay_{decay}", dtype, config(64, 96, [one, one], 2, None, None), edit)
    t = tokens(cfg, 200, 7)
    want = R.forward(cfg, w, t)
    assert np.isfinite(want).all()
    check_portions(m, t, want, dtype, ([200], [130, 1, 1, 68], [20] * 10), factor=2.0 if decay == "steps" else 1.0)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("streams", [1, 2, 3, 4, 6, 16])
def test_streams_and_loops(bank, streams, dtype):
    layers = [attn(2, 1, 16, 16, 20, 2, ff=24), delta(2, 1, 16, 16, 2), attn(2, 2, 8, 24, 9, 0, 4, ff=40)]
    for loop in ((0, 1, 3), (1, 3, 2), (2, 3, 0)):
        cfg, w, m = bank(f"streams_{streams}_{loop}", dtype, config(56, 80, layers, streams, loop, (13, 5, 6)))
        t = tokens(cfg, 60, 8)
        check_portions(m, t, R.forward(cfg, w, t), dtype, ([60], [31, 1, 1, 1, 26]))


def test_plain_residual_without_streams(bank):
    """No streams in the configuration: plain sums, no tensors of the connections."""
    cfg = config(64, 96, [attn(2, 1, 16, 16, 20, 2, ff=24), delta(2, 1, 16, 16, 2, 32)], 1)
    w = R.random_model(cfg, 2)
    for k in w:
        if ".hc" in k:
            w[k] = np.ones_like(w[k])
    bare = {k: v for k, v in cfg.items() if k != "streams"}
    R.save_model(bank.root / "bare", bare, {k: v for k, v in w.items() if ".hc" not in k})
    from mlx_parallm_amd.utils import load_model

    m = load_model(bank.root / "bare", dtype="float32", max_positions=256)
    t = tokens(cfg, 50, 3)
    check_portions(m, t, R.forward(cfg, w, t), "float32", ([50], [24, 1, 1, 24]))
    m.engine.close()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_previous_token_travels_with_its_row(bank, dtype):
    """Nearly everything of the embedding is the pair's: a token that took another row's previous token, a stale one or the first
    token's row would be far off.  Multipliers far beyond the buckets."""
    cfg = config(48, 300, [attn(2, 1, 16, 16, 0)], 2, None, (49999, 2147483629, 10**12 + 39), 0.125)

    def edit(w):
        w["embed"] *= 0.25
    cfg, w, m = bank("pairs", dtype, cfg, edit)
    a, b = tokens(cfg, 60, 6), tokens(cfg, 60, 7)
    wa, wb = R.forward(cfg, w, a), R.forward(cfg, w, b)
    kv = m.engine.new_paged_kv(3, block_tokens=16, n_blocks=10, max_tokens_per_row=64)
    for again in range(2):
        ia = ib = 0
        for na, nb in ((1, 2), (2, 1), (20, 1), (1, 1), (1, 40), (30, 1), (5, 14)):
            got = m.engine.forward_segments(kv, [2, 0], [b[ib:ib + nb], a[ia:ia + na]], range(na + nb))
            assert err(got[:nb], wb[ib:ib + nb], wb).max() < TOL[dtype] and err(got[nb:], wa[ia:ia + na], wa).max() < TOL[dtype], (na, nb)
            ia, ib = ia + na, ib + nb
        kv.reset_row(0)
        kv.reset_row(2)
    kv.close()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_batches_of_unequal_requests_against_each_alone(bank, dtype):
    cfg, w, m = bank("odd", dtype)
    eng = m.engine
    reqs = [tokens(cfg, n, 10 + n) for n in (90, 1, 33, 64, 7)]
    want = [R.forward(cfg, w, t) for t in reqs]
    kv = eng.new_paged_kv(5, block_tokens=16, n_blocks=24, max_tokens_per_row=96)
    at, step, rng = [0] * 5, 0, np.random.default_rng(4)
    while any(a < len(t) for a, t in zip(at, reqs)):
        rows = [i for i in rng.permutation(5) if at[i] < len(reqs[i]) and (rng.random() < 0.8 or step > 60)]
        if not rows:
            continue
        parts = [reqs[i][at[i]:at[i] + int(rng.choice([1, 1, 1, 2, 5, 17, 40]))] for i in rows]
        got = eng.forward_segments(kv, rows, parts, range(sum(map(len, parts))))
        j = 0
        for i, p in zip(rows, parts):
            e = err(got[j:j + len(p)], want[i][at[i]:at[i] + len(p)], want[0])
            assert e.max() < TOL[dtype], (step, i, e.max())
            j += len(p)
            at[i] += len(p)
        step += 1
    kv.close()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_rows_and_blocks_are_used_again(bank, dtype):
    cfg, w, m = bank("odd", dtype)
    eng = m.engine
    kv = eng.new_paged_kv(2, block_tokens=16, n_blocks=9, max_tokens_per_row=96)     # eight blocks for both rows
    for k in range(6):
        a, b = tokens(cfg, 70 - 9 * k, 30 + k), tokens(cfg, 20 + 3 * k, 60 + k)
        ra = k % 2
        for t, row, sizes in ((a, ra, [40, 1, 2, 100]), (b, 1 - ra, [1, 1, 100])):
            e = err(run_portions(eng, kv, row, t, sizes), R.forward(cfg, w, t)).max()
            assert e < TOL[dtype]
        kv.reset_row(0)
        kv.reset_row(1)
        assert kv.stats()["free_blocks"] == 8
    kv.close()


def peaky(w, n_special, V):
    """Keys that stand out: the last n_special tokens of the vocabulary score far above everything else where they are seen."""
    rng = np.random.default_rng(9)
    e, k, q = w["embed"], w["l0.mix.k"], w["l0.mix.q"]
    w["l0.mix.q.norm"][:] = 4.0
    w["l0.mix.k.norm"][:] = 4.0
    w["l0.norm1"][:] = 0.0
    d = rng.standard_normal(e.shape[1]).astype(np.float32)
    e[V - n_special:] += 3 * d                               # special tokens share a direction ..
    u = np.sign(rng.standard_normal(k.shape[0])).astype(np.float32)
    k += np.outer(u, d).astype(np.float32) / e.shape[1]      # .. that points every key of theirs along u,
    rep, half = q.shape[0] // k.shape[0], k.shape[0] // 2
    uq = np.concatenate([np.tile(u[g * half:(g + 1) * half], rep) for g in range(2)])
    q += 2 * np.outer(uq, np.ones(e.shape[1])).astype(np.float32) / np.sqrt(e.shape[1])     # and the queries' common part as well
    e += 0.7
    for name in ("embed", "l0.mix.k", "l0.mix.q"):
        u32 = np.ascontiguousarray(w[name], np.float32).view(np.uint32)
        w[name] = ((u32 + 0x8000) & np.uint32(0xFFFF0000)).view(np.float32)


# places of the keys that stand out (alone in their window; at the ends of blocks), masks that the logits tell from the true one
EDGES = {"window": ((63, 192, 319), [(99, 5), (101, 5)]), "last_kept": ((4,), [(100, 4)]), "first_not_kept": ((5,), [(100, 6), (101, 5)])}


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("edge", list(EDGES))
@pytest.mark.parametrize("name,dim", [("matrix_cores", 32), ("generic", 160)])
def test_single_keys_stand_out_at_the_edges_of_the_window_and_of_the_kept_tokens(bank, name, dim, edge, dtype):
    """A few tokens whose keys outscore everything: a key that is missing, or seen one token too long, changes the logits
    completely."""
    size, keep, n = 100, 5, 420
    mix = attn(4, 2, dim, 24, size, keep, 6, 3.5 / dim)

    def edit(w):
        peaky(w, 4, 64)
        w["l0.mix.sink"][:] = 3.0
        w["l0.hc1.out"][:] = 6.0
    cfg = config(96, 64, [mix], 1, None, None, 1.0)
    cfg, w, m = bank(f"peaky_{name}", dtype, cfg, edit)
    t = tokens(cfg, n, 5) % 60
    places, others = EDGES[edge]
    for i, p in enumerate(places):
        t[p] = 60 + i
    want = R.forward(cfg, w, t)
    for s, k in others:
        moved = R.forward({**cfg, "layers": [{**mix, "mixer": {**mix["mixer"], "mask": {"size": s, "keep_first": k}}}]}, w, t)
        assert (err(moved, want) > 6 * TOL[dtype]).sum() >= (2 if edge == "window" else 1), (s, k)
    bare = R.as_f64({**w, "l0.mix.sink": np.full(4, -99.0)})
    assert (err(R.forward(cfg, bare, t), want) > 6 * TOL[dtype]).sum() >= 1
    check_portions(m, t, want, dtype, ([n], [162, 1, 1, 1, 126, 1, 1, 1, 126], [33] * 13, [4, 2] + [1] * 414, [99, 2, 98, 2, 98, 1, 1, 119]), 64, 3.0)


def test_long_decoding_behind_a_long_prompt(bank):
    """700 tokens at once, then 330 one by one, beside a row that does the opposite: positions, windows and blocks far out; a window
    longer than one split of the decode attention."""
    cfg = config(64, 96, [attn(4, 2, 32, 32, 700, 3, 16, 0.3, 48), delta(2, 1, 32, 32, 3), attn(16, 1, 64, 64, 0, 0, 32, 0.2), attn(4, 4, 16, 16, 333, 70)],
                 2, (1, 3, 2))
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


def test_growth_of_a_contiguous_cache_keeps_keys_values_and_state(bank):
    cfg, w, m = bank("odd")
    t = tokens(cfg, 120, 9)
    kv = m.engine.new_kv(2, capacity=16, kv_dtype="model", step=16)
    got = run_portions(m.engine, kv, 1, t, [10, 1, 30, 1, 1, 77])
    assert kv.capacity >= 120 and err(got, R.forward(cfg, w, t)).max() < TOL["float32"]
    kv.close()


def test_prefix_blocks_are_shared_unless_a_layer_is_recurrent(bank):
    cfg, w, m = bank("shared", cfg=config(64, 96, [attn(2, 1, 16, 16, 30, 2, ff=24), attn(2, 2, 16, 8, 0)], 2, (0, 2, 2)))
    a = tokens(cfg, 70, 50)
    b = np.concatenate([a[:50], tokens(cfg, 30, 51)]).astype(np.int32)
    kv = m.engine.new_paged_kv(2, block_tokens=16, n_blocks=14, max_tokens_per_row=96)
    run_portions(m.engine, kv, 0, a, [70])
    kv.prefix_publish(0, a)
    assert kv.prefix_attach(1, b) == 48
    got = m.engine.forward_segments(kv, [1], [b[48:]], range(len(b) - 48))      # (its first token's pair: the last one of the prefix)
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
    for bad in (attn(3, 2, 16, 16, 8), attn(2, 1, 16, 16, 8, 0, 7), attn(2, 1, 16, 16, 8, 0, 18), attn(2, 1, 16, 16, -3)):
        with pytest.raises(ValueError):
            Engine({**config(64, 96, [bad]), "model_type": "temetar"})
    with pytest.raises(ValueError):
        Engine({**config(64, 96, [one], 17), "model_type": "temetar"})
    with pytest.raises(NotImplementedError):
        Engine({**config(64, 96, [attn(1, 1, 600, 16, 8)]), "model_type": "temetar"})
    few = config(64, 96, [attn(2, 1, 16, 16, 8, ff=24)], 2)
    for gone in ("bigram", "l0.hc2.mix", "l0.mix.sink", "l0.mlp.up"):
        R.save_model(tmp_path / gone, few, {k: v for k, v in R.random_model(few).items() if k != gone})
        with pytest.raises(FileNotFoundError, match=gone):
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

    cfg = config(72, build_byte_tokenizer(tmp_path), [attn(4, 2, 20, 24, 33, 2, 12, ff=24), delta(3, 1, 16, 16, 3), attn(2, 1, 32, 48, 0, ff=40)], 2, (1, 3, 2))
    serve_and_compare(tmp_path, scheduler, R, cfg, greedy)
