"""Temetar on the CPU: the plain implementation's mechanisms, the configuration reader, the ABI fields of the design."""
import json

import numpy as np
import pytest

from oracle import ref_temetar as R
from tests.temetar_models import CONFIGS, attn, config, delta


def test_norm_weight_is_stored_around_zero():
    x = np.random.default_rng(0).standard_normal((4, 9))
    assert np.allclose(R.norm(x, np.zeros(9), 0.0), x / np.sqrt((x * x).mean(-1, keepdims=True)))
    assert np.allclose(R.norm(x, np.full(9, 0.5), 1e-3), 1.5 * R.rms(x, 1e-3))


def test_pair_rows_and_the_first_token():
    assert R.bigram_rows([5, 7, 5], 11, 3, 2) == [11, (15 + 14) % 11, (21 + 10) % 11]
    assert R.bigram_rows([4], 1, 0, 0) == [1]


def test_rotation_pairs_distant_coordinates_and_keeps_the_rest():
    rng = np.random.default_rng(1)
    x = rng.standard_normal((5, 2, 10))
    y = R.rotate(x, np.arange(5), 100.0, 6)
    assert np.array_equal(y[..., 6:], x[..., 6:]) and np.allclose(y[0], x[0])
    assert np.allclose(y[..., 1] ** 2 + y[..., 4] ** 2, x[..., 1] ** 2 + x[..., 4] ** 2)
    a = 3 * 100.0 ** (-2 / 6)
    assert np.allclose(y[3, 1, 1], x[3, 1, 1] * np.cos(a) - x[3, 1, 4] * np.sin(a))
    # scores depend on the distance only
    q, k = np.tile(x[:1], (9, 1, 1)), np.tile(x[1:2], (9, 1, 1))
    q, k = R.rotate(q, np.arange(9), 50.0, 10), R.rotate(k, np.arange(9), 50.0, 10)
    assert np.isclose((q[7, 0] * k[4, 0]).sum(), (q[3, 0] * k[0, 0]).sum())


def test_window_and_kept_first_tokens():
    v = R.visible(8, {"size": 3, "keep_first": 2})
    assert v[5].tolist() == [1, 1, 0, 1, 1, 1, 0, 0] and v[1].tolist() == [1, 1, 0, 0, 0, 0, 0, 0] and v[3].tolist() == [1, 1, 1, 1, 0, 0, 0, 0]
    assert np.array_equal(R.visible(6, None), np.tril(np.ones((6, 6), bool)))
    assert np.array_equal(R.visible(4, {"size": 1}), np.eye(4, dtype=bool))


def test_sink_takes_weight_and_gives_nothing():
    s, m = np.zeros((1, 3)), np.ones((1, 3), bool)
    assert np.allclose(R.softmax_sink(s, m, 0.0), 0.25) and np.allclose(R.softmax_sink(s, m, np.log(5.0)).sum(), 3 / 8)
    assert np.allclose(R.softmax_sink(s + 700, m, -700.0), 1 / 3)


def test_channel_decay_with_equal_channels_is_the_rule_with_one_decay():
    from oracle import ref_runevik as U

    rng = np.random.default_rng(2)
    q, k, v = (rng.standard_normal((9, 2, n)) for n in (4, 4, 5))
    beta, g = rng.uniform(0, 1, (9, 2)), -rng.uniform(0, 2, (9, 2))
    a, sa = R.channel_delta_rule(q, k, v, beta, np.repeat(g[:, :, None], 4, 2))
    b, sb = U.delta_rule(q, k, v, beta, g)
    assert np.allclose(a, b) and np.allclose(sa, sb)
    # a channel that forgets everything leaves only the current token's write in its row
    lg = np.zeros((9, 2, 4))
    lg[:, :, 1] = -np.inf
    _, s = R.channel_delta_rule(q, k, v, beta, lg)
    s0 = R.channel_delta_rule(q[:8], k[:8], v[:8], beta[:8], lg[:8])[1]
    s0[:, 1] = 0
    u = beta[8][:, None] * (v[8] - np.einsum("hde,hd->he", s0, k[8]))
    assert np.allclose(s[:, 1], k[8][:, 1:2] * u)


def test_streams_are_mixed_from_the_old_ones():
    xs = np.arange(6.0).reshape(2, 1, 3)
    mix, out = np.array([[1.0, 2.0], [3.0, 4.0]]), np.array([10.0, 20.0])
    y = np.ones((1, 3))
    got = R.hyper_write(xs, y, mix, out, 0.5)
    assert np.allclose(got[0], xs[0] + 3 * xs[1] + 5) and np.allclose(got[1], 2 * xs[0] + 4 * xs[1] + 10)
    assert np.allclose(R.hyper_read(xs, np.array([0.5, -1.0])), 0.5 * xs[0] - xs[1])


def test_layer_runs_of_a_loop():
    cfg = {"layers": [0] * 5, "loop": {"start": 1, "stop": 3, "times": 2}}
    assert R.layer_runs(cfg) == [0, 1, 2, 1, 2, 3, 4]
    assert R.layer_runs({"layers": [0] * 2, "loop": None}) == [0, 1]


def test_later_tokens_do_not_change_logits_and_each_pass_has_its_own_state():
    cfg = config(40, 50, [attn(2, 1, 8, 8, 4, 1, ff=16), delta(2, 1, 4, 6, 3)], 2, (0, 2, 2))
    w = R.random_model(cfg, 3)
    t = np.random.default_rng(0).integers(0, 50, 14)
    a, layers = R.forward(cfg, w, t), []
    assert np.allclose(a[:5], R.forward(cfg, w, t[:5], layers)) and len(layers) == 4


def test_configuration_becomes_layer_descriptions():
    from mlx_parallm_amd import _lib as L
    from mlx_parallm_amd.models.temetar import Model, layer_list
    from mlx_parallm_amd.utils import _get_classes

    cfg = CONFIGS["odd"]
    with pytest.raises(ValueError, match="inner sizes"):
        layer_list(cfg)
    full = Model.complete_config(cfg, {k: v.shape for k, v in R.random_model(cfg, 1, 5, 9).items()})
    assert "decay_rank" not in cfg["layers"][1]["mixer"]                       # (the caller's configuration is left alone)
    model, layers = layer_list(full)
    assert model["hidden_size"] == 100 and model["rms_norm_eps"] == 3e-6 and model["streams"] == 3 and model["residual_mult"] == 0.6
    assert (model["loop_start"], model["loop_stop"], model["loop_times"]) == (1, 4, 2) and model["embed_scale"] == 2.5
    assert (model["pair_buckets"], model["pair_mul_prev"], model["pair_mul_cur"]) == (61, 1000 % 61, 77 % 61)
    assert [d["mixer"] for d in layers] == [L.MI_MIXER_GQA, L.MI_MIXER_DELTA] * 2 + [L.MI_MIXER_GQA]
    assert [(d["window"], d["keep_first"], d["rot_dims"]) for d in layers[::2]] == [(37, 3, 12), (64, 0, 10), (25, 7, 22)]
    assert [(d["decay_rank"], d["gate_rank"], d["conv"]) for d in layers[1::2]] == [(5, 9, 3), (5, 9, 2)]
    assert [d["ff"] for d in layers] == [72, 0, 0, 50, 130] and np.isclose(layers[3]["scale"], 18 ** -0.5)
    plain = layer_list(config(8, 8, [attn(1, 1, 4, 4, 0, rot=0)], 1, None, None))
    assert plain[1][0]["window"] == plain[1][0]["rot_dims"] == 0 and "loop_stop" not in plain[0] and "pair_buckets" not in plain[0]
    klass, args = _get_classes(cfg)
    assert klass.__module__.endswith("temetar") and args.from_dict(cfg).num_hidden_layers == 5
    with pytest.raises(ValueError, match="mixer type"):
        args.from_dict(config(8, 8, [dict(cfg["layers"][0], type="other")]))
    with pytest.raises(ValueError, match="feed-forward kind"):
        args.from_dict(config(8, 8, [dict(attn(1, 1, 4, 4, 4), mlp={"kind": "moe", "ff": 3})]))
    with pytest.raises(ValueError, match="loop"):
        layer_list(config(8, 8, [attn(1, 1, 4, 4, 4)], 1, (0, 2, 2)))
    with pytest.raises(ValueError, match="missing"):
        Model.complete_config(cfg, {})


def test_every_description_field_exists_in_the_binding():
    from mlx_parallm_amd import _lib as L
    from mlx_parallm_amd.models.temetar import Model, layer_list

    cfg = CONFIGS["wide"]
    model, layers = layer_list(Model.complete_config(cfg, {k: v.shape for k, v in R.random_model(cfg).items()}))
    assert set(model) <= {n for n, _ in L.ModelDesc._fields_}
    assert all(set(d) <= {n for n, _ in L.LayerDesc._fields_} for d in layers)


def test_layer_structs_agree_with_the_header(tmp_path):
    import ctypes as C
    import subprocess
    from pathlib import Path

    from mlx_parallm_amd import _lib as L

    src = '#include <stdio.h>\n#include <stddef.h>\n#include "mi355_decode.h"\nint main(void){printf("%zu %zu %zu %zu %zu\\n", sizeof(mi_layer_desc), ' \
          'offsetof(mi_layer_desc, out_gate), offsetof(mi_layer_desc, gate_rank), offsetof(mi_model_desc, norm_offset), ' \
          'offsetof(mi_model_desc, loop_times));return 0;}\n'
    (tmp_path / "p.c").write_text(src)
    inc = Path(__file__).resolve().parent.parent / "include"
    subprocess.run(["gcc", "-I", str(inc), str(tmp_path / "p.c"), "-o", str(tmp_path / "p")], check=True)
    out = subprocess.run([str(tmp_path / "p")], capture_output=True, text=True, check=True).stdout.split()
    assert [int(x) for x in out] == [C.sizeof(L.LayerDesc), L.LayerDesc.out_gate.offset, L.LayerDesc.gate_rank.offset,
                                     L.ModelDesc.norm_offset.offset, L.ModelDesc.loop_times.offset]


def test_block_bytes_count_every_run_of_a_layer():
    from mlx_parallm_amd import _lib as L
    from mlx_parallm_amd.engine import Engine
    from mlx_parallm_amd.models.temetar import Model, layer_list

    eng = Engine.__new__(Engine)
    cfg = config(8, 8, [attn(4, 2, 20, 40, 8), delta(1, 1, 4, 4, 2), attn(1, 1, 144, 128, 8)], 2, (0, 2, 3))
    model, layers = layer_list(Model.complete_config(cfg, {k: v.shape for k, v in R.random_model(cfg).items()}))
    eng.act_dtype, eng.desc, eng.layer_descs, eng._h, eng._kvs = "bfloat16", L.ModelDesc(), [], None, []
    eng.desc.arch = L.MI_ARCH_LAYERS
    for k, v in model.items():
        setattr(eng.desc, k, v)
    for f in layers:
        d = L.LayerDesc()
        for k, v in f.items():
            setattr(d, k, v)
        eng.layer_descs.append(d)
    assert eng.layer_runs() == R.layer_runs(cfg) == [0, 1, 0, 1, 0, 1, 2]
    assert eng.kv_block_bytes(16) == (3 * 2 * (32 + 64) + (160 + 128)) * 16 * 2


def test_plain_model_round_trips_through_a_checkpoint(tmp_path):
    from safetensors.torch import load_file

    cfg = config(48, 40, [attn(2, 1, 8, 8, 5, 2, ff=24), delta(2, 1, 4, 6, 3, 16)], 2, (0, 1, 2))
    w = R.random_model(cfg, 5)
    R.save_model(tmp_path, cfg, w)
    back = R.as_f64(load_file(str(tmp_path / "model.safetensors")))
    t = [1, 5, 7, 9, 2, 3, 4]
    assert json.loads((tmp_path / "config.json").read_text()) == cfg
    assert np.array_equal(R.forward(cfg, R.as_f64(w), t), R.forward(cfg, back, t))
