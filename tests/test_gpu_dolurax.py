"""Dolurax on the GPU against the plain implementation (oracle/ref_dolurax.py): whole prompts, portions, decoding, batches,
reused rows and blocks, each mechanism alone, greedy generation through the framework's own entry points."""
import json
import subprocess
from pathlib import Path

import numpy as np
import pytest

from oracle import ref_dolurax as R
from tests.dolurax_models import CONFIGS, attn, config, layer, moe
from tests.gpu_helpers import serve_and_compare

pytestmark = pytest.mark.gpu
ROOT = Path(__file__).resolve().parent.parent
# error = rms over the vocabulary of the centred difference / rms of the centred logits
# (rounding every operand of the plain implementation's products to bfloat16 gives 0.06 for the configuration "odd")
TOL = {"float32": 2e-5, "bfloat16": 0.09, "float16": 0.0125}


def err(got, want):
    d = got - want
    d = d - d.mean(-1, keepdims=True)
    s = want - want.mean(-1, keepdims=True)
    return np.sqrt((d * d).mean(-1)) / np.sqrt((s * s).mean())


def plain(cfg, w, t, layers=None):
    """-> logits, and which positions no router was undecided about: 16-bit inputs may flip a choice between two experts with nearly
    equal scores, there and (through the attention) a little behind it."""
    margins = []
    lg = R.forward(cfg, w, t, layers, margins)
    return lg, np.min(margins, axis=0) > 0.1 if margins else np.ones(len(t), bool)


def worst(e, clear, dtype):
    """The figure that is held against TOL."""
    return e.max() if dtype == "float32" else np.quantile(e[clear], 0.95)


@pytest.fixture(scope="module")
def bank(tmp_path_factory):
    """name, dtype -> (cfg, float64 weights, loaded model); one checkpoint per name, kept for the module."""
    from mlx_parallm_amd.utils import load_model

    root, plain, loaded = tmp_path_factory.mktemp("dolurax"), {}, {}

    def get(name, dtype="float32", cfg=None, edit=None, seed=1):
        if name not in plain:
            c = cfg or CONFIGS[name]
            w = R.random_model(c, seed)
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
        for i, (g, x) in enumerate(zip(cap, layers)):
            assert worst(np.sqrt(((g - x) ** 2).mean(-1)), clear, dtype) < TOL[dtype] * np.sqrt((x * x).mean()), (n, i)
        assert worst(err(got, want), clear, dtype) < TOL[dtype], n


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", list(CONFIGS))
def test_portions_and_decoding_agree_with_the_whole(bank, name, dtype):
    cfg, w, m = bank(name, dtype)
    t = tokens(cfg, 150, 2)
    want, clear = plain(cfg, w, t)
    eng = m.engine
    for sizes in ([1] * 150, [2] * 75, [3, 2, 1, 5, 64, 2, 1, 1, 65, 6], [63, 1, 1, 64, 2, 19], [130] + [1] * 20):
        kv = eng.new_paged_kv(2, block_tokens=16, n_blocks=12, max_tokens_per_row=160)
        got = run_portions(eng, kv, 1, t, sizes)
        kv.close()
        assert worst(err(got, want), clear, dtype) < TOL[dtype], sizes[:4]


def one_mechanism(keep):
    """Zero what the other sublayer adds to the stream (its norm's weight and bias)."""
    def edit(w):
        for k in w:
            if keep != "attention" and ".norm1" in k or keep != "experts" and ".norm2" in k:
                w[k] = w[k] * 0
    return edit


@pytest.mark.parametrize("keep", ["attention", "experts", "none"])
def test_each_sublayer_alone(bank, keep):
    cfg = config(72, 112, [layer(attn(3, 3, 16, 24, 29, v_mix=False), moe(6, 2, 40, 3, 2, 24))])
    cfg, w, m = bank(f"alone_{keep}", "float32", cfg, one_mechanism(keep))
    t = tokens(cfg, 70, 3)
    want = R.forward(cfg, w, t)
    kv = m.engine.new_kv(1, capacity=128, kv_dtype="model")
    assert err(run_portions(m.engine, kv, 0, t, [37, 1, 1, 31]), want).max() < TOL["float32"]
    kv.close()


BASE = dict(heads=4, kv_heads=2, dim=24, vdim=32, chunk=0, scale=0.4, softcap=None, v_mix=False)
MECHANISMS = {"plain": {}, "cap": {"softcap": 3.0}, "chunk": {"chunk": 19}, "v_mix": {"v_mix": True}, "one_head_group": {"kv_heads": 1},
              "every_head_its_own": {"kv_heads": 4}}


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", list(MECHANISMS))
def test_each_attention_mechanism_alone(bank, name, dtype):
    mix = attn(**{**BASE, **MECHANISMS[name]})
    cfg, w, m = bank(f"mech_{name}", dtype, config(64, 96, [layer(mix), layer(mix), layer(mix)], logit_scale=1.0, logit_softcap=None))
    t = tokens(cfg, 90, 4)
    want = R.forward(cfg, w, t)
    for sizes in ([90], [18, 1, 1, 20, 50], [1] * 90):
        kv = m.engine.new_paged_kv(1, block_tokens=16, n_blocks=8, max_tokens_per_row=96)
        assert err(run_portions(m.engine, kv, 0, t, sizes), want).max() < TOL[dtype], sizes[:2]
        kv.close()


ROUTERS = {"top1": (8, 1, 1, 1, 0), "all": (6, 6, 1, 1, 0), "one_group": (12, 3, 4, 1, 0), "all_groups": (12, 3, 4, 4, 0), "groups_of_one": (8, 2, 8, 3, 0),
           "shared": (8, 2, 2, 1, 50), "uneven": (90, 7, 9, 4, 20), "large_tiles": (4, 2, 2, 2, 200, 136),
           "large_tiles_no_shared": (3, 2, 1, 1, 0, 128)}


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", list(ROUTERS))
def test_each_router_form_alone(bank, name, dtype):
    E, top, groups, keep, shared, ff, width = (*ROUTERS[name], 48, 64)[:7] if len(ROUTERS[name]) == 5 else (*ROUTERS[name], 150)
    cfg = config(width, 96, [layer(attn(2, 1, 16, 16, 40), moe(E, top, ff, groups, keep, shared))])
    cfg, w, m = bank(f"router_{name}", dtype, cfg)
    t = tokens(cfg, 333, 5)
    want, clear = plain(cfg, w, t)
    for sizes in ([333], [70, 200, 63], [17] * 20):
        kv = m.engine.new_kv(1, capacity=340, kv_dtype="model")
        assert worst(err(run_portions(m.engine, kv, 0, t, sizes), want), clear, dtype) < TOL[dtype], sizes[:2]
        kv.close()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_batches_of_unequal_requests_against_each_alone(bank, dtype):
    cfg, w, m = bank("odd", dtype)
    eng = m.engine
    reqs = [tokens(cfg, n, 10 + n) for n in (90, 1, 33, 64, 7)]
    want, clear = zip(*(plain(cfg, w, t) for t in reqs))
    kv = eng.new_paged_kv(5, block_tokens=16, n_blocks=24, max_tokens_per_row=96)
    at, step, rng, errs = [0] * 5, 0, np.random.default_rng(4), [np.zeros(len(t)) for t in reqs]
    while any(a < len(t) for a, t in zip(at, reqs)):
        rows = [i for i in rng.permutation(5) if at[i] < len(reqs[i]) and (rng.random() < 0.8 or step > 60)]
        if not rows:
            continue
        parts = [reqs[i][at[i]:at[i] + int(rng.choice([1, 1, 1, 2, 5, 17, 40]))] for i in rows]
        got = eng.forward_segments(kv, rows, parts, range(sum(map(len, parts))))
        j = 0
        for i, p in zip(rows, parts):
            errs[i][at[i]:at[i] + len(p)] = err(got[j:j + len(p)], want[i][at[i]:at[i] + len(p)])
            j += len(p)
            at[i] += len(p)
        step += 1
    kv.close()
    assert worst(np.concatenate(errs), np.concatenate(clear), dtype) < TOL[dtype]


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_rows_and_blocks_are_used_again(bank, dtype):
    cfg, w, m = bank("odd", dtype)
    eng = m.engine
    kv = eng.new_paged_kv(2, block_tokens=16, n_blocks=9, max_tokens_per_row=96)     # eight blocks for both rows
    for k in range(6):
        a, b = tokens(cfg, 70 - 9 * k, 30 + k), tokens(cfg, 20 + 3 * k, 60 + k)
        ra = k % 2
        for t, row, sizes in ((a, ra, [40, 1, 2, 100]), (b, 1 - ra, [1, 1, 100])):
            want, clear = plain(cfg, w, t)
            assert worst(err(run_portions(eng, kv, row, t, sizes), want), clear, dtype) < TOL[dtype]
        kv.reset_row(0)
        kv.reset_row(1)
        assert kv.stats()["free_blocks"] == 8
    kv.close()


def peaky(cfg, w, n_special):
    """Keys that stand out: the last n_special tokens of the vocabulary score far above everything else where they are seen."""
    V = cfg["vocab"]
    w["l0.mix.q.norm"][:] = 4.0
    w["l0.mix.k.norm"][:] = 4.0
    e = w["embed"]
    rng = np.random.default_rng(9)
    d = rng.standard_normal(e.shape[1]).astype(np.float32)
    e[V - n_special:] += 3 * d                               # special tokens share a direction ..
    kd, W = w["l0.mix.k"].shape[0] // 2, e.shape[1]
    u = np.sign(rng.standard_normal(w["l0.mix.k"].shape[0])).astype(np.float32)
    w["l0.mix.k"] += np.outer(u, d).astype(np.float32) / W   # .. that points every key of theirs along u,
    q = w["l0.mix.q"]
    rep = q.shape[0] // w["l0.mix.k"].shape[0]
    uq = np.concatenate([np.tile(u[g * kd:(g + 1) * kd], rep) for g in range(2)])
    q += 2 * np.outer(uq, np.ones(W)).astype(np.float32) / np.sqrt(W)       # and the queries' common part as well
    e[:, :] += 0.7
    for k in ("embed", "l0.mix.k", "l0.mix.q"):
        u32 = np.ascontiguousarray(w[k], np.float32).view(np.uint32)
        w[k] = ((u32 + 0x8000) & np.uint32(0xFFFF0000)).view(np.float32)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name,dim", [("matrix_cores", 32), ("generic", 160)])
def test_single_keys_stand_out_at_chunk_and_block_borders(bank, name, dim, dtype):
    """A few tokens whose keys outscore everything in their chunk: a key that is missing, or seen from the next chunk, changes the
    logits completely.  They stand at the last and first places of chunks, at block borders and far from the asking positions."""
    chunk, n = 100, 420
    mix = attn(64, 2, dim, 24, chunk, 2.5 / dim, 40.0, False)        # (64 heads: the last slopes are small, far keys stay visible)
    cfg = config(96, 64, [layer(mix)], logit_scale=1.0, logit_softcap=None)
    cfg, w, m = bank(f"peaky_{name}", dtype, cfg, lambda w: peaky(cfg, w, 4))
    t = tokens(cfg, n, 5) % 60
    for i, p in enumerate((0, 1, 63, 64, 99, 100, 127, 128, 199, 201, 255, 256, 299, 300, 319, 320, 399, 400, 401)):
        t[p] = 60 + i % 4
    want = R.forward(cfg, w, t)
    # the mask is what decides: one token off, either way, shows
    for off in (99, 101):
        other = R.forward({**cfg, "layers": [layer({**mix, "mask": {"size": off}})]}, w, t)
        assert (err(other, want) > 4 * TOL[dtype]).sum() >= 3
    eng = m.engine
    for sizes in ([n], [198] + [1] * 222, [33] * 13, [2] * 210, [99, 2, 98, 2, 98, 1, 1, 119]):
        kv = eng.new_paged_kv(1, block_tokens=64, n_blocks=9, max_tokens_per_row=448)
        e = err(run_portions(eng, kv, 0, t, sizes), want)
        kv.close()
        assert e.max() < 3 * TOL[dtype], (sizes[:3], int(e.argmax()))


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_values_of_the_first_layer_travel_with_their_tokens(bank, dtype):
    """Nearly everything of a later layer's values is the first mixing layer's: in a mixed batch a token that took another token's
    values would be far off."""
    one = attn(4, 2, 32, 40, 50)
    cfg = config(64, 96, [layer(attn(2, 2, 16, 24, 30, v_mix=False)), layer(one), layer(attn(8, 1, 64, 80, 50)), layer(one)])

    def edit(w):
        for i in (2, 3):
            w[f"l{i}.mix.vmix"] = np.asarray(0.984375, np.float32)
        w["l1.mix.vmix"] = np.asarray(0.5, np.float32)           # (not used)
    cfg, w, m = bank("v_first", dtype, cfg, edit)
    a, b = tokens(cfg, 80, 6), tokens(cfg, 80, 7)
    wa, wb = R.forward(cfg, w, a), R.forward(cfg, w, b)
    kv = m.engine.new_paged_kv(2, block_tokens=16, n_blocks=12, max_tokens_per_row=80)
    ia = ib = 0
    for na, nb in ((1, 20), (2, 1), (30, 1), (1, 1), (1, 40), (40, 1), (5, 16)):
        got = m.engine.forward_segments(kv, [1, 0], [b[ib:ib + nb], a[ia:ia + na]], range(na + nb))
        assert err(got[:nb], wb[ib:ib + nb]).max() < TOL[dtype] and err(got[nb:], wa[ia:ia + na]).max() < TOL[dtype], (na, nb)
        ia, ib = ia + na, ib + nb
    kv.close()


def test_long_decoding_behind_a_long_prompt(bank):
    """700 tokens at once, then 330 one by one, beside a row that does the opposite: positions, chunks and blocks far out; a chunk
    longer than one split of the decode attention."""
    cfg = config(64, 96, [layer(attn(4, 2, 32, 32, 1000, 0.3), moe(8, 2, 32, 4, 2, 32)), layer(attn(16, 1, 64, 64, 0, 0.3)), layer(attn(4, 4, 16, 16, 333))])
    cfg, w, m = bank("long", "bfloat16", cfg)
    a, b = tokens(cfg, 1030, 40), tokens(cfg, 1030, 41)
    (wa, ca), (wb, cb) = plain(cfg, w, a), plain(cfg, w, b)
    kv = m.engine.new_paged_kv(2, block_tokens=64, n_blocks=36, max_tokens_per_row=1088)
    eng = m.engine
    ea, eb = [err(eng.forward_segments(kv, [0], [a[:700]], range(700)), wa[:700])], []
    for i in range(330):
        got = eng.forward_segments(kv, [1, 0], [b[i:i + 1], a[700 + i:701 + i]], [0, 1])
        eb.append(err(got[:1], wb[i:i + 1]))
        ea.append(err(got[1:], wa[700 + i:701 + i]))
    eb.append(err(eng.forward_segments(kv, [1], [b[330:]], range(700)), wb[330:]))
    kv.close()
    for e, clear in ((np.concatenate(ea), ca), (np.concatenate(eb), cb)):
        assert worst(e, clear, "bfloat16") < TOL["bfloat16"] and (e[clear] > TOL["bfloat16"]).mean() < 0.02


@pytest.mark.parametrize("dtype", ["bfloat16", "float16"])
@pytest.mark.parametrize("cap", [1.0, 6.0, None])
def test_keys_beyond_the_reach_of_the_distance_bias(bank, cap, dtype):
    """Steep slopes and small caps: the kernels leave out keys whose capped score cannot matter any more, nothing else.  Large norms:
    scores run into the cap, where its polynomial does not hold."""
    mix = attn(6, 2, 32, 48, 0, 0.4, cap, False)
    cfg = config(64, 96, [layer(mix), layer({**mix, "mask": {"size": 300}})], logit_scale=1.0, logit_softcap=None)

    def edit(w):
        for k in w:
            if k.endswith(("q.norm", "k.norm")):
                w[k] = w[k] * (1.5 if k.startswith("l1") else 0.5)
    cfg, w, m = bank(f"reach_{cap}", dtype, cfg, edit)
    t = tokens(cfg, 700, 8)
    want = R.forward(cfg, w, t)
    for sizes in ([700], [299, 2, 1, 1, 1, 96, 300], [600] + [1] * 100):
        kv = m.engine.new_paged_kv(1, block_tokens=64, n_blocks=12, max_tokens_per_row=704)
        assert np.quantile(err(run_portions(m.engine, kv, 0, t, sizes), want), 0.99) < TOL[dtype], sizes[:2]
        kv.close()


def test_growth_of_a_contiguous_cache_keeps_keys_and_values(bank):
    cfg, w, m = bank("odd")
    t = tokens(cfg, 120, 9)
    kv = m.engine.new_kv(2, capacity=16, kv_dtype="model", step=16)
    got = run_portions(m.engine, kv, 1, t, [10, 1, 30, 1, 1, 77])
    assert kv.capacity >= 120 and err(got, R.forward(cfg, w, t)).max() < TOL["float32"]
    kv.close()


def test_blocks_of_a_common_prefix_are_shared(bank):
    cfg, w, m = bank("odd")
    a = tokens(cfg, 70, 50)
    b = np.concatenate([a[:50], tokens(cfg, 30, 51)]).astype(np.int32)
    kv = m.engine.new_paged_kv(2, block_tokens=16, n_blocks=14, max_tokens_per_row=96)
    run_portions(m.engine, kv, 0, a, [70])
    kv.prefix_publish(0, a)
    assert kv.prefix_attach(1, b) == 48
    got = m.engine.forward_segments(kv, [1], [b[48:]], range(len(b) - 48))
    assert err(got, R.forward(cfg, w, b)[48:]).max() < TOL["float32"]
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


def test_wrong_use_is_refused(bank):
    from mlx_parallm_amd.engine import Engine

    cfg, w, m = bank("odd", "bfloat16")
    eng = m.engine
    with pytest.raises(NotImplementedError):
        eng.new_kv(1, capacity=16, kv_dtype="float32")
    one = attn(2, 1, 16, 16, 8)
    for bad in (layer(attn(3, 2, 16, 16, 8)), layer(one, moe(6, 5, 8, 3, 2)), layer(one, moe(7, 2, 8, 2, 1)), layer(one, moe(4, 0, 8))):
        with pytest.raises(ValueError):
            Engine({**config(64, 96, [bad]), "model_type": "dolurax"})
    with pytest.raises(ValueError):                            # mixed values of unequal size
        Engine({**config(64, 96, [layer(one), layer(attn(2, 2, 16, 16, 8))]), "model_type": "dolurax"})
    with pytest.raises(NotImplementedError):
        Engine({**config(64, 96, [layer(attn(1, 1, 600, 16, 8))]), "model_type": "dolurax"})


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

    cfg = config(72, build_byte_tokenizer(tmp_path), [layer(attn(4, 2, 20, 24, 33), moe(6, 2, 40, 3, 2, 24)), layer(attn(3, 3, 16, 16, 50)),
                                                     layer(attn(2, 1, 32, 48, 0), moe(5, 3, 24))])
    serve_and_compare(tmp_path, scheduler, R, cfg, greedy)
