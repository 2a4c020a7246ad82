"""Runevik on the GPU against the plain implementation (oracle/ref_runevik.py): whole prompts, portions, decoding, batches,
reused rows and blocks, each mechanism alone, greedy generation through the framework's own entry points."""
import json
import subprocess
from pathlib import Path

import numpy as np
import pytest

from oracle import ref_runevik as R
from tests.gpu_helpers import serve_and_compare
from tests.runevik_models import CONFIGS, config, delta, latent

pytestmark = pytest.mark.gpu
ROOT = Path(__file__).resolve().parent.parent
# error = rms over the vocabulary of the centred difference / rms of the centred logits
TOL = {"float32": 2e-5, "bfloat16": 0.05, "float16": 0.01}


def err(got, want):
    d = got - want
    d = d - d.mean(-1, keepdims=True)
    s = want - want.mean(-1, keepdims=True)
    return np.sqrt((d * d).mean(-1)) / np.sqrt((s * s).mean())


def worst(e, name, dtype):
    """The figure that is held against TOL.  With head size 1 a unit vector is a sign: where it is about to flip, 16-bit
    inputs may flip it, so that configuration is judged by its ninth decile outside float32."""
    return np.quantile(e, 0.9) if name == "ones" and dtype != "float32" else e.max()


@pytest.fixture(scope="module")
def bank(tmp_path_factory):
    """name, dtype -> (cfg, float64 weights, loaded model); one checkpoint per name, kept for the module."""
    from mlx_parallm_amd.utils import load_model

    root, plain, loaded = tmp_path_factory.mktemp("runevik"), {}, {}

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
    t, layers = tokens(cfg, 41), []
    want = R.forward(cfg, w, t, layers)
    kv = m.engine.new_kv(1, capacity=64, kv_dtype="model")
    cap = m.engine.capture_residual(len(t))
    got = m.engine.forward_segments(kv, [0], [t], range(len(t)))
    m.engine.capture_residual(0)
    kv.close()
    assert worst(err(got, want), name, dtype) < TOL[dtype]
    for g, x in zip(cap, layers):
        assert worst(np.sqrt(((g - x) ** 2).mean(-1)), name, dtype) < TOL[dtype] * np.sqrt((x * x).mean())


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", list(CONFIGS))
def test_portions_and_decoding_agree_with_the_whole(bank, name, dtype):
    cfg, w, m = bank(name, dtype)
    t = tokens(cfg, 150, 2)
    want = R.forward(cfg, w, t)
    eng = m.engine
    for sizes in ([1] * 150, [2] * 75, [3, 2, 1, 5, 64, 2, 1, 1, 65, 6], [63, 1, 1, 64, 2, 19], [130] + [1] * 20):
        kv = eng.new_paged_kv(2, block_tokens=16, n_blocks=12, max_tokens_per_row=160)
        got = run_portions(eng, kv, 1, t, sizes)
        kv.close()
        assert worst(err(got, want), name, dtype) < TOL[dtype], sizes[:4]


def one_mechanism(cfg, keep):
    """Zero what every other mechanism adds to the stream."""
    def edit(w):
        for k in w:
            if keep != "mix" and k.endswith("mix.o") or keep != "mlp" and k.endswith("mlp.down") or keep != "side" and k.endswith("side.norm"):
                w[k] = w[k] * 0
    return edit


@pytest.mark.parametrize("keep", ["mix", "mlp", "side", "none"])
@pytest.mark.parametrize("kind", ["delta", "latent"])
def test_each_mechanism_alone(bank, kind, keep):
    layer = delta(3, 3, 16, 24, 3, 80) if kind == "delta" else latent(3, 16, 24, 48, 0.4, 80)
    cfg = config(72, 112, [layer], 20)
    cfg, w, m = bank(f"alone_{kind}_{keep}", "float32", cfg, one_mechanism(cfg, keep))
    t = tokens(cfg, 70, 3)
    want = R.forward(cfg, w, t)
    kv = m.engine.new_kv(1, capacity=128, kv_dtype="model")
    assert err(run_portions(m.engine, kv, 0, t, [37, 1, 1, 31]), want).max() < TOL["float32"]
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
            assert err(got[j:j + len(p)], want[i][at[i]:at[i] + len(p)]).max() < TOL[dtype], (step, i, at[i], len(p))
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
            assert err(run_portions(eng, kv, row, t, sizes), R.forward(cfg, w, t)).max() < TOL[dtype]
        kv.reset_row(0)
        kv.reset_row(1)
        assert kv.stats()["free_blocks"] == 8
    kv.close()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", ["peaky", "peaky_generic"])
def test_single_keys_stand_out_far_away_and_at_block_borders(bank, name, dtype):
    """One latent layer whose scores are so large that a position attends to one or two keys: a key that is missing, or seen
    too early, changes the logits completely.  Keys of every distance, around every block border."""
    r = 72 if name == "peaky" else 560
    cfg = config(96, 64, [latent(4, 32, 48, r, 2.0, 0)], 0)

    def edit(w):
        w["l0.mix.o"] = w["l0.mix.o"] * 4
        w["embed"] = w["embed"] * 4          # token identity dominates the position: equal tokens are found wherever they are
    cfg, w, m = bank(name, dtype, cfg, edit)
    n = 420
    t = tokens(cfg, n, 5)
    t[:2] = [63, 62]
    t[2:][t[2:] >= 60] = 1
    for p in (64, 65, 127, 128, 129, 255, 256, 257, 415, 416):   # the first tokens are asked for again from far away
        t[p] = 63 if p % 2 else 62
    want = R.forward(cfg, w, t)
    eng = m.engine
    for sizes in ([n], [200] + [1] * 220, [33] * 13, [2] * 210):
        kv = eng.new_paged_kv(1, block_tokens=64, n_blocks=9, max_tokens_per_row=448)
        e = err(run_portions(eng, kv, 0, t, sizes), want)
        kv.close()
        assert e.max() < 3 * TOL[dtype], (sizes[:3], int(e.argmax()))


def test_state_remembers_an_early_token(bank):
    """Decays near one and a large write: the first token's write is read hundreds of tokens later, across every cut."""
    cfg = config(64, 64, [delta(2, 1, 16, 16, 4, 0)], 0)

    def edit(w):
        w["l0.mix.A_log"][:] = -6.0
        w["l0.mix.o"] = w["l0.mix.o"] * 4
    cfg, w, m = bank("memory", "float32", cfg, edit)
    t = tokens(cfg, 300, 8)
    want = R.forward(cfg, w, t)
    other = t.copy()
    other[0] = (other[0] + 1) % 64
    assert err(R.forward(cfg, w, other)[250:], want[250:]).max() > 1e-3          # it does matter
    for sizes in ([300], [3] * 100, [150] + [1] * 150):
        kv = m.engine.new_kv(1, capacity=320, kv_dtype="model")
        assert err(run_portions(m.engine, kv, 0, t, sizes), want).max() < TOL["float32"]
        kv.close()


@pytest.mark.parametrize("kind", ["forget", "keep", "same_token"])
def test_recurrence_at_the_ends_of_its_range(bank, kind):
    """Decays from e^-100 to nearly one within one chunk of the recurrence, step sizes next to one, and runs of one token
    (equal keys: every write undoes the one before it)."""
    cfg = config(64, 64, [delta(4, 2, 20, 12, 3, 0), delta(2, 2, 64, 40, 2, 0)], 0)

    def edit(w):
        for i in (0, 1):
            n = len(w[f"l{i}.mix.A_log"])
            w[f"l{i}.mix.A_log"] = {"forget": np.linspace(1.0, 3.5, n), "keep": np.full(n, -7.0), "same_token": np.full(n, -5.0)}[kind].astype(np.float32)
            w[f"l{i}.mix.A_log"] = (w[f"l{i}.mix.A_log"].view(np.uint32) & np.uint32(0xFFFF0000)).view(np.float32)
            w[f"l{i}.mix.a"] = w[f"l{i}.mix.a"] * 4          # some tokens forget everything, others nothing
            w[f"l{i}.mix.b"] = w[f"l{i}.mix.b"] * 8
    cfg, w, m = bank(f"range_{kind}", "float32", cfg, edit)
    t = tokens(cfg, 333, 12)
    if kind == "same_token":
        t[20:150] = 7
        t[190:260] = 9
        w["embed"][:] = 8 * w["embed"]                       # equal tokens have nearly equal keys wherever they are
        R.save_model(bank.root / "range_big", cfg, w)
        from mlx_parallm_amd.utils import load_model
        m = load_model(bank.root / "range_big", dtype="float32", max_positions=2048)
    want = R.forward(cfg, w, t)
    for sizes in ([333], [64, 65, 63, 128, 13], [1, 127, 2, 63, 140], [30] * 12):
        kv = m.engine.new_kv(1, capacity=340, kv_dtype="model")
        assert err(run_portions(m.engine, kv, 0, t, sizes), want).max() < TOL["float32"], (kind, sizes[:3])
        kv.close()
    if kind == "same_token":
        m.engine.close()


def test_long_decoding_behind_a_long_prompt(bank):
    """700 tokens at once, then 330 one by one, beside a row that does the opposite: positions, chunks and blocks far out."""
    cfg, w, m = bank("odd", "bfloat16")
    a, b = tokens(cfg, 1030, 40), tokens(cfg, 1030, 41)
    wa, wb = R.forward(cfg, w, a), R.forward(cfg, w, b)
    kv = m.engine.new_paged_kv(2, block_tokens=64, n_blocks=36, max_tokens_per_row=1088)
    eng = m.engine
    got = eng.forward_segments(kv, [0], [a[:700]], range(700))
    assert err(got, wa[:700]).max() < TOL["bfloat16"]
    for i in range(330):
        got = eng.forward_segments(kv, [1, 0], [b[i:i + 1], a[700 + i:701 + i]], [0, 1])
        assert err(got[:1], wb[i:i + 1]).max() < TOL["bfloat16"] and err(got[1:], wa[700 + i:701 + i]).max() < TOL["bfloat16"], i
    got = eng.forward_segments(kv, [1], [b[330:]], range(700))
    assert err(got, wb[330:]).max() < TOL["bfloat16"]
    kv.close()


def test_growth_of_a_contiguous_cache_keeps_latents_and_state(bank):
    cfg, w, m = bank("odd")
    t = tokens(cfg, 120, 9)
    kv = m.engine.new_kv(2, capacity=16, kv_dtype="model", step=16)
    got = run_portions(m.engine, kv, 1, t, [10, 1, 30, 1, 1, 77])
    assert kv.capacity >= 120 and err(got, R.forward(cfg, w, t)).max() < TOL["float32"]
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
    cfg, w, m = bank("odd", "bfloat16")
    eng = m.engine
    with pytest.raises(NotImplementedError):
        eng.new_kv(1, capacity=16, kv_dtype="float32")
    with pytest.raises(NotImplementedError):
        eng.set_lora(0, "self_attn.q_proj", np.zeros((4, 2), np.float32), np.zeros((2, 4), np.float32), 1.0)
    kv = eng.new_paged_kv(2, block_tokens=16, n_blocks=4, max_tokens_per_row=32)
    with pytest.raises(ValueError):
        eng.forward_segments(kv, [0], [[cfg["vocab"]]], [0])
    with pytest.raises(ValueError):
        eng.forward_segments(kv, [0, 0], [[1], [2]], [0])
    kv.close()


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

    cfg = config(72, build_byte_tokenizer(tmp_path), [delta(4, 2, 20, 24, 3, 80), latent(3, 16, 24, 40, 0.4, 72), latent(2, 24, 16, 40, 0.3, 0, 1)], 8)
    serve_and_compare(tmp_path, scheduler, R, cfg, greedy)
