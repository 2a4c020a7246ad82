"""Beronex on the CPU: the plain implementation's mechanisms, the configuration reader, the ABI fields of the design."""
import json
import math

import numpy as np
import pytest

from oracle import ref_beronex as R
from tests.beronex_models import CONFIGS, attn, config, dense, latent, light, moe, yarn


def test_gelu_and_the_clamped_unit():
    z = np.array([-40.0, -1.0, 0.0, 0.5, 3.0, 40.0])
    exact = np.array([0.5 * x * (1 + math.erf(x / math.sqrt(2))) for x in z])
    assert np.allclose(R.gelu_tanh(z), exact, atol=1e-3) and R.gelu_tanh(np.array(40.0)) == 40.0
    g, u = np.array([-9.0, 0.3, 5.0, 5.0]), np.array([0.2, 9.0, -9.0, 0.1])
    want = [g_ / (1 + np.exp(-1.702 * g_)) * (u_ + 1) for g_, u_ in ((-9.0, 0.2), (0.3, 2.0), (2.0, -2.0), (2.0, 0.1))]
    assert np.allclose(R.clamped_unit(g, u, 2.0), want)


def test_rotation_of_neighbours_and_of_halves():
    rng = np.random.default_rng(1)
    x, rot = rng.standard_normal((5, 2, 10)), {"base": 100.0, "dims": 6}
    y, z = R.rotate(x, np.arange(5), rot, True), R.rotate(x, np.arange(5), rot, False)
    assert np.array_equal(y[..., 6:], x[..., 6:]) and np.allclose(y[0], x[0]) and np.allclose(z[0], x[0])
    a = 3 * 100.0 ** (-2 / 6)
    assert np.allclose(y[3, 1, 2], x[3, 1, 2] * np.cos(a) - x[3, 1, 3] * np.sin(a))
    assert np.allclose(y[3, 1, 3], x[3, 1, 3] * np.cos(a) + x[3, 1, 2] * np.sin(a))
    assert np.allclose(z[3, 1, 1], x[3, 1, 1] * np.cos(a) - x[3, 1, 4] * np.sin(a))
    order = [0, 2, 4, 1, 3, 5, 6, 7, 8, 9]                     # halves of the reordered head = neighbours of the head
    assert np.allclose(R.rotate(x[..., order], np.arange(5), rot, False), y[..., order])


def test_stretched_frequencies():
    rot = {"base": 10000.0, "dims": 32, "scaling": yarn(4.0, 2048, 32.0, 1.0)}
    f, gain = R.frequencies(rot)
    plain = 10000.0 ** (-np.arange(16) / 16)
    assert np.isclose(gain, 0.1 * math.log(4.0) + 1)
    turns = 2048 * plain / (2 * math.pi)
    assert np.allclose(f[turns > 40], plain[turns > 40]) and np.allclose(f[turns < 0.5], plain[turns < 0.5] / 4)
    between = (turns < 20) & (turns > 2)
    assert between.any() and (f[between] < plain[between]).all() and (f[between] > plain[between] / 4).all()
    # both ends of the ramp in the same pair: a step; a context so short that every pair is stretched
    f, _ = R.frequencies({"base": 10000.0, "dims": 8, "scaling": yarn(2.0, 1, 1.0, 1.0)})
    assert np.allclose(f[1:], 10000.0 ** (-np.arange(1, 4) / 4) / 2) and np.isclose(f[0], 1.0)
    assert R.frequencies({"base": 9.0, "dims": 4})[1] == 1.0


def test_norm_behind_the_rotation_sees_its_gain():
    x, rot = np.random.default_rng(2).standard_normal((6, 1, 8)), {"base": 50.0, "dims": 4, "scaling": yarn(64.0)}
    y, gain = R.rotated_rms(x, rot, 1e-6), R.frequencies(rot)[1]
    n = np.sqrt((gain ** 2 * (x[..., :4] ** 2).sum(-1) + (x[..., 4:] ** 2).sum(-1)) / 8 + 1e-6)
    assert np.allclose(y[..., 4:], x[..., 4:] / n[..., None]) and np.allclose((y * y).mean(-1), 1.0, atol=1e-5)
    assert not np.allclose(y, R.rotate(R.rms(x, 1e-6), np.arange(6), rot, True), atol=0.05)


def test_window():
    assert R.visible(6, 3)[4].tolist() == [0, 0, 1, 1, 1, 0]
    assert np.array_equal(R.visible(4, 1), np.eye(4, dtype=bool)) and np.array_equal(R.visible(4), np.tril(np.ones((4, 4), bool)))


def test_decayed_sums_are_attention_without_a_softmax():
    rng = np.random.default_rng(3)
    q, k, v, g = rng.standard_normal((9, 3, 4)), rng.standard_normal((9, 3, 4)), rng.standard_normal((9, 3, 5)), [0.0, 0.7, 1.0]
    o, s = R.decayed_sums(q, k, v, g)
    for h in range(3):
        d = np.arange(9)[:, None] - np.arange(9)[None, :]
        w = np.where(d >= 0, np.power(g[h], np.maximum(d, 0)), 0.0)
        assert np.allclose(o[:, h], (q[:, h] @ k[:, h].T * w) @ v[:, h])
    a, mid = R.decayed_sums(q[:4], k[:4], v[:4], g)
    b, end = R.decayed_sums(q[4:], k[4:], v[4:], g, mid)
    assert np.allclose(np.concatenate([a, b]), o) and np.allclose(end, s)


def test_router_weights_are_a_softmax_over_the_chosen():
    z = np.array([0.1, 2.0, -1.0, 1.5])
    assert [e for e, _ in R.route(z, 2)] == [1, 3] and np.isclose(R.route(z, 2)[0][1], 1 / (1 + np.exp(-0.5)))
    assert np.isclose(sum(g for _, g in R.route(z, 4)), 1.0) and R.route(z, 1) == [(1, 1.0)]
    assert np.isclose(R.route_margin(z, 2), 1.4) and R.route_margin(z, 4) == np.inf


def test_another_layers_keys_and_values_are_read_as_they_are():
    cfg = config(40, 50, [attn(2, 1, 8, 8, 4), attn(2, 1, 8, 8, 9, kv_from=0)])
    w = R.random_model(cfg, 3)
    assert not any(k in w for k in ("l1.mix.k", "l1.mix.v"))
    h = np.random.default_rng(0).standard_normal((12, 40))
    y, kv = R.attention(h, R.as_f64(w), "l0.mix.", cfg["layers"][0]["mixer"], 1e-5)
    y1, kv1 = R.attention(h, R.as_f64(w), "l1.mix.", cfg["layers"][1]["mixer"], 1e-5, kv)
    assert kv1 is kv and not np.allclose(y, y1)


def test_later_tokens_do_not_change_logits():
    cfg, layers = CONFIGS["odd"], []
    w, t = R.random_model(cfg, 3), np.random.default_rng(0).integers(0, 50, 30)
    a = R.forward(cfg, w, t)
    assert np.allclose(a[:11], R.forward(cfg, w, t[:11], layers)) and len(layers) == 7


def test_configuration_becomes_layer_descriptions():
    from mlx_parallm_amd import _lib as L
    from mlx_parallm_amd.models.beronex import layer_list
    from mlx_parallm_amd.utils import _get_classes

    cfg = CONFIGS["odd"]
    model, d = layer_list(cfg)
    assert model["hidden_size"] == 100 and model["vocab_size"] == 333 and model["rms_norm_eps"] == 3e-6 and model["embed_scale"] == 1.7
    assert model["block_form"] == L.MI_BLOCK_SANDWICH and model["norm_kind"] == L.MI_NORM_VECTOR
    assert [x["mixer"] for x in d] == [L.MI_MIXER_LATENT, L.MI_MIXER_GQA, L.MI_MIXER_LIGHTNING, L.MI_MIXER_GQA, L.MI_MIXER_LIGHTNING, L.MI_MIXER_LATENT, L.MI_MIXER_GQA]
    assert [x["kv_from"] for x in d] == [-1, -1, -1, 1, -1, -1, -1] and [x.get("window") for x in d] == [None, 37, None, 64, None, None, 0]
    assert (d[0]["q_rank"], d[0]["kv_rank"], d[0]["rot_dims"], d[0]["rot_pairs"]) == (37, 45, 6, L.MI_ROT_HALVES)
    assert (d[1]["rot_dims"], d[1]["rot_pairs"], d[1]["rot_factor"], d[1]["rot_original"]) == (12, L.MI_ROT_PAIRS, 8.0, 64.0)
    assert "rot_factor" not in d[6] and d[6]["rot_base"] == 300.0 and d[2]["decay"] == cfg["layers"][2]["mixer"]["decay"]
    assert [x.get("ff", 0) for x in d] == [72, 40, 0, 50, 24, 70, 0] and [x.get("act") for x in d[:2]] == [L.MI_ACT_GEGLU, L.MI_ACT_CLAMPED]
    assert (d[4]["experts"], d[4]["top"], d[4]["act_limit"], d[4]["router_bias"], d[4]["groups"]) == (5, 2, 0.8, 1, 1)
    plain = layer_list(config(8, 8, [attn(1, 1, 4, 4, 0, rot=0)]))[1][0]
    assert plain["window"] == 0 and "rot_dims" not in plain
    klass, args = _get_classes(cfg)
    assert klass.__module__.endswith("beronex") and args.from_dict(cfg).num_hidden_layers == 7
    with pytest.raises(ValueError, match="mixer type"):
        args.from_dict(config(8, 8, [dict(cfg["layers"][0], type="other")]))
    with pytest.raises(ValueError, match="feed-forward kind"):
        args.from_dict(config(8, 8, [dict(cfg["layers"][0], mlp={"kind": "other", "ff": 3})]))
    with pytest.raises(ValueError, match="decays"):
        args.from_dict(config(8, 8, [light(2, 4, 4, [0.5])]))
    bad = latent(1, 4, 4, 4, 4, 4)
    bad["mixer"]["rot"]["dims"] = 2
    with pytest.raises(ValueError, match="rot_dim"):
        args.from_dict(config(8, 8, [bad]))


def test_layer_struct_agrees_with_the_header(tmp_path):
    import ctypes as C
    import subprocess
    from pathlib import Path

    from mlx_parallm_amd import _lib as L
    from mlx_parallm_amd.models.beronex import layer_list

    model, layers = layer_list(CONFIGS["wide"])
    assert set(model) <= {n for n, _ in L.ModelDesc._fields_} and all(set(d) <= {n for n, _ in L.LayerDesc._fields_} for d in layers)
    names = ["rot_pairs", "rot_slow", "qk_norm", "q_rank", "act_limit", "router_bias", "decay"]
    src = '#include <stdio.h>\n#include <stddef.h>\n#include "mi355_decode.h"\nint main(void){printf("%zu", sizeof(mi_layer_desc));' + \
          "".join(f'printf(" %zu", offsetof(mi_layer_desc, {n}));' for n in names) + "return 0;}\n"
    (tmp_path / "p.c").write_text(src)
    inc = Path(__file__).resolve().parent.parent / "include"
    subprocess.run(["gcc", "-I", str(inc), str(tmp_path / "p.c"), "-o", str(tmp_path / "p")], check=True)
    out = subprocess.run([str(tmp_path / "p")], capture_output=True, text=True, check=True).stdout.split()
    assert [int(x) for x in out] == [C.sizeof(L.LayerDesc)] + [getattr(L.LayerDesc, n).offset for n in names]


def test_block_bytes_count_the_rotated_part_and_no_shared_keys():
    from mlx_parallm_amd import _lib as L
    from mlx_parallm_amd.engine import Engine
    from mlx_parallm_amd.models.beronex import layer_list

    eng = Engine.__new__(Engine)
    model, layers = layer_list(config(8, 8, [latent(2, 8, 8, 8, 8, 60), attn(4, 2, 20, 40, 8), light(1, 4, 4), attn(4, 2, 20, 40, 9, kv_from=1),
                                             latent(2, 8, 16, 8, 8, 48), attn(1, 1, 144, 128, 8)]))
    eng.act_dtype, eng.desc, eng.layer_descs, eng._h, eng._kvs = "bfloat16", L.ModelDesc(), [], None, []
    eng.desc.arch = L.MI_ARCH_LAYERS
    for f in layers:
        d = L.LayerDesc()
        for k, v in f.items():
            if k != "decay":
                setattr(d, k, v)
        eng.layer_descs.append(d)
    # 60 -> 64 beside 8: 128; 48 beside 16: 64
    assert eng.kv_block_bytes(16) == (128 + 2 * (32 + 64) + 64 + 160 + 128) * 16 * 2


def test_plain_model_round_trips_through_a_checkpoint(tmp_path):
    from safetensors.torch import load_file

    cfg = config(48, 40, [attn(2, 1, 8, 8, 5, mlp=moe(3, 2, 8)), light(2, 4, 6, None, dense(16)), latent(2, 4, 4, 4, 6, 8)])
    w = R.random_model(cfg, 5)
    R.save_model(tmp_path, cfg, w)
    back = R.as_f64(load_file(str(tmp_path / "model.safetensors")))
    t = [1, 5, 7, 9, 2, 3, 4]
    assert json.loads((tmp_path / "config.json").read_text()) == cfg
    assert np.array_equal(R.forward(cfg, R.as_f64(w), t), R.forward(cfg, back, t))
