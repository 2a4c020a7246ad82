"""Dolurax on the CPU: the plain implementation's mechanisms, the configuration reader, the ABI fields of the design."""
import json

import numpy as np
import pytest

from oracle import ref_dolurax as R
from tests.dolurax_models import CONFIGS, attn, config, layer, moe


def test_layer_norm_and_rms_against_torch():
    import torch

    rng = np.random.default_rng(0)
    x, w, b = rng.standard_normal((5, 12)), rng.standard_normal(12), rng.standard_normal(12)
    t = torch.from_numpy(x)
    want = torch.nn.functional.layer_norm(t, (12,), torch.from_numpy(w), torch.from_numpy(b), 1e-3).numpy()
    assert np.allclose(R.layer_norm(x, w, b, 1e-3), want)
    assert np.allclose(R.rms(x, 0.0), x / np.sqrt((x * x).mean(-1, keepdims=True)))


def test_cap_slopes_and_visibility():
    assert R.cap(3.0, None) == 3.0 and np.isclose(R.cap(1e6, 5.0), 5.0) and np.isclose(R.cap(0.01, 5.0), 0.01, atol=1e-6)
    assert np.allclose(R.slopes(4), [0.25, 1 / 16, 1 / 64, 1 / 256]) and np.isclose(R.slopes(3)[0], 2 ** (-8 / 3))
    v = R.visible(7, 3)
    assert v[2].tolist() == [1, 1, 1, 0, 0, 0, 0] and v[3].tolist() == [0, 0, 0, 1, 0, 0, 0] and v[5].tolist() == [0, 0, 0, 1, 1, 1, 0]
    assert np.array_equal(R.visible(5, None), np.tril(np.ones((5, 5), bool))) and np.array_equal(R.visible(4, 1), np.eye(4, dtype=bool))


def test_distance_bias_is_outside_the_cap():
    q, k = np.full((3, 2), 9.0), np.full((3, 2), 9.0)
    s = R.scores(q, k, 1.0, 2.0, 0.5)
    assert np.allclose(s[2], [2.0 - 1.0, 2.0 - 0.5, 2.0])


def test_values_are_mixed_behind_the_first_mixing_layer_only():
    v, f = np.ones((2, 3)), np.full((2, 3), 5.0)
    assert np.allclose(R.mix_values(v, f, 0.25), 2.0) and R.mix_values(v, None, 0.25) is v


def test_router_keeps_groups_then_experts():
    z = np.log(np.array([0.30, 0.01, 0.20, 0.19, 0.02, 0.28]))
    r = {"experts": 6, "top": 2, "groups": {"count": 3, "keep": 1}}
    assert [e for e, _ in R.route(z, r)] == [0, 1]                          # the best group is (0, 1), its second expert is weak
    assert [e for e, _ in R.route(z, {**r, "groups": {"count": 3, "keep": 2}})] == [0, 5]
    assert [e for e, _ in R.route(z, {"experts": 6, "top": 3})] == [0, 5, 2]
    g = dict(R.route(z, {"experts": 6, "top": 3}))
    assert np.isclose(sum(g.values()), 1) and np.isclose(g[0] / g[5], 0.30 / 0.28)


def test_later_tokens_and_other_chunks_do_not_change_logits():
    cfg = config(40, 50, [layer(attn(2, 1, 8, 8, 6), moe(4, 2, 8, 2, 1, 8)), layer(attn(2, 1, 8, 8, 6))])
    w = R.random_model(cfg, 3)
    t = np.random.default_rng(0).integers(0, 50, 14)
    a = R.forward(cfg, w, t)
    assert np.allclose(a[:5], R.forward(cfg, w, t[:5]))
    other = t.copy()
    other[:6] = (other[:6] + 1) % 50                                        # the whole first chunk
    b = R.forward(cfg, w, other)
    assert np.allclose(a[6:], b[6:]) and not np.allclose(a[5], b[5])


def test_configuration_becomes_layer_descriptions():
    from mlx_parallm_amd import _lib as L
    from mlx_parallm_amd.models.dolurax import layer_list
    from mlx_parallm_amd.utils import _get_classes

    cfg = CONFIGS["odd"]
    model, layers = layer_list(cfg)
    assert model["hidden_size"] == 100 and model["rms_norm_eps"] == 3e-6 and model["norm_kind"] == L.MI_NORM_LAYER
    assert model["logit_scale"] == 0.5 and model["logit_softcap"] == 25.0
    assert all(d["mixer"] == L.MI_MIXER_GQA for d in layers)
    assert [d["chunk"] for d in layers] == [37, 64, 0, 10, 50] and [d["v_mix"] for d in layers] == [0, 1, 1, 1, 1]
    assert [d["softcap"] for d in layers] == [20.0, 20.0, 0.0, 20.0, 20.0]
    assert [d.get("ff", 0) for d in layers] == [40, 24, 0, 33, 48] and [d.get("shared_ff", 0) for d in layers] == [72, 16, 0, 0, 130]
    assert (layers[0]["experts"], layers[0]["top"], layers[0]["groups"], layers[0]["keep"]) == (6, 3, 3, 2)
    assert layer_list(CONFIGS["generic"])[0]["logit_softcap"] == 0.0
    one = layer(attn(1, 1, 4, 4, 4), {"kind": "moe", "expert": {"ff": 4}, "router": {"experts": 4, "top": 2}})
    assert layer_list(config(8, 8, [one]))[1][0]["groups"] == 1
    klass, args = _get_classes(cfg)
    assert klass.__module__.endswith("dolurax") and args.from_dict(cfg).num_hidden_layers == 5
    with pytest.raises(ValueError, match="mixer type"):
        args.from_dict(config(8, 8, [dict(one, type="other")]))
    with pytest.raises(ValueError, match="feed-forward kind"):
        args.from_dict(config(8, 8, [layer(attn(1, 1, 4, 4, 4), {"kind": "dense", "ff": 3})]))


def test_every_description_field_exists_in_the_binding():
    from mlx_parallm_amd import _lib as L
    from mlx_parallm_amd.models.dolurax import layer_list

    model, layers = layer_list(CONFIGS["wide"])
    assert set(model) <= {n for n, _ in L.ModelDesc._fields_}
    assert all(set(d) <= {n for n, _ in L.LayerDesc._fields_} for d in layers)


def test_block_bytes_count_padded_keys_and_values():
    from mlx_parallm_amd import _lib as L
    from mlx_parallm_amd.engine import Engine
    from mlx_parallm_amd.models.dolurax import layer_list

    eng = Engine.__new__(Engine)
    eng.act_dtype, eng.desc = "bfloat16", L.ModelDesc()
    eng.desc.arch = L.MI_ARCH_LAYERS
    cfg = config(8, 8, [layer(attn(4, 2, 20, 40, 8)), layer(attn(1, 1, 144, 128, 8))])
    eng.layer_descs = []
    for f in layer_list(cfg)[1]:
        d = L.LayerDesc()
        for k, v in f.items():
            setattr(d, k, v)
        eng.layer_descs.append(d)
    eng._h, eng._kvs = None, []
    assert eng.kv_block_bytes(16) == (2 * (32 + 64) + (160 + 128)) * 16 * 2


def test_plain_model_round_trips_through_a_checkpoint(tmp_path):
    from safetensors.torch import load_file

    cfg = config(48, 40, [layer(attn(2, 1, 8, 8, 5), moe(4, 2, 24, 2, 1, 8)), layer(attn(2, 1, 8, 8, 5))])
    w = R.random_model(cfg, 5)
    R.save_model(tmp_path, cfg, w)
    back = R.as_f64(load_file(str(tmp_path / "model.safetensors")))
    t = [1, 5, 7, 9, 2, 3, 4]
    assert json.loads((tmp_path / "config.json").read_text()) == cfg
    assert np.array_equal(R.forward(cfg, R.as_f64(w), t), R.forward(cfg, back, t))
