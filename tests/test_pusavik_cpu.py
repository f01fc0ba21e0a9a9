"""The layer-list decoder without a GPU: configuration, registry, order of layers, the plain implementation itself."""
import json

import numpy as np
import pytest

from fusekit_amd import registry
from fusekit_amd.checkpoint import layer_config_from_json, layer_config_to_json, save_layer_checkpoint
from fusekit_amd.layer_decoder import LayerWeights, pad, random_tensors, tensor_shapes
from oracle import pusavik as plain
from pusavik_helpers import configs, lat, model, moe, ssm


@pytest.mark.parametrize("name", sorted(configs()))
def test_config_round_trip(name):
    c = configs()[name]
    j = json.loads(json.dumps(layer_config_to_json(c)))
    assert registry.family_of(j).name == "layer-list" and registry.vocab_of(j) == c.vocab
    back = layer_config_from_json(j, {})
    assert back == c and tensor_shapes(back) == tensor_shapes(c)


def test_query_rank_from_the_tensor_and_optional_keys():
    c = model([(lat(q_rank=72), moe(identity=0))])
    j = layer_config_to_json(c)
    del j["layers"][0]["mixer"]["q_rank"], j["layers"][0]["mlp"]["router"]["identity"]
    assert layer_config_from_json(j, {"l0.mix.dq": (72, 72)}) == c
    assert not layer_config_from_json(j, {"l0.mix.dq": (72, 72)}).looped
    j["layers"][0]["type"] = "other"
    with pytest.raises(ValueError, match="unknown mixer"):
        layer_config_from_json(j, {})
    j = layer_config_to_json(c)
    j["layers"][0]["mlp"]["kind"] = "dense"
    with pytest.raises(ValueError, match="unknown feed-forward"):
        layer_config_from_json(j, {})


def test_registry_knows_the_other_families():
    assert registry.family_of({"model_type": "deepseek_v2", "hidden_size": 8, "vocab_size": 9}).name == "moe"
    assert registry.family_of({"model_type": "qwen3", "hidden_size": 8, "vocab_size": 9}).name == "dense"
    with pytest.raises(ValueError, match="no model"):
        registry.family_of({"architecture": "Unheard"})


def test_order_of_layer_runs():
    c = model([(lat(), None)] * 5, loop_start=1, loop_stop=3, loop_times=2)
    assert c.runs() == [(0, None), (1, 0), (2, None), (1, 1), (2, None), (3, None), (4, None)]
    assert c.runs() == plain.layer_runs(layer_config_to_json(c))
    c = model([(lat(), None), (ssm(), None)], loop_start=0, loop_stop=2, loop_times=2)
    assert c.runs() == [(0, 0), (1, None), (0, 1), (1, None)] == plain.layer_runs(layer_config_to_json(c))
    assert model([(lat(), None)] * 2).runs() == [(0, None), (1, None)]


def test_checkpoint_files(tmp_path):
    from fusekit_amd.checkpoint import SafetensorsFile
    c = configs()["mixed"]
    t = random_tensors(c, 3)
    save_layer_checkpoint(str(tmp_path), c, t)
    f = SafetensorsFile(str(tmp_path / "model.safetensors"))
    assert {n: tuple(v["shape"]) for n, v in f.tensors.items()} == tensor_shapes(c)
    data, dtype, shape = f.raw("l0.mix.uq")
    assert dtype == "BF16" and np.array_equal(np.frombuffer(data.tobytes(), np.uint16).reshape(shape), t["l0.mix.uq"])


def test_padded_widths():
    m = lat(dim=24, rot_dim=12, vdim=20, kv_rank=40)
    assert (m.dim_ld, m.rot_ld, m.vdim_ld, m.hs, m.rank_ld, m.ldc) == (32, 32, 32, 64, 64, 96)
    assert pad(1) == 64 and pad(64) == 64 and pad(65) == 128
    assert np.allclose(LayerWeights.rot_freq(lat(rot_dim=4, rot_base=100.0)), [1.0, 0.1])


# ---- the plain implementation against closed forms ----

def test_plain_window_and_sink():
    s = np.array([0.3, -1.0, 2.0])
    p = plain.sink_softmax(s, 0.5)
    assert np.allclose(p, np.exp(s) / (np.exp(s).sum() + np.exp(0.5)))
    assert [plain.window_sees(9, j, 3) for j in (6, 7, 9, 10)] == [False, True, True, False]


def test_plain_recurrence_is_the_decayed_sum():
    r = np.random.Generator(np.random.PCG64(0))
    T, H, P, N = 7, 2, 3, 4
    x, B, C, dt = r.standard_normal((T, H, P)), r.standard_normal((T, H, N)), r.standard_normal((T, H, N)), r.random((T, H))
    A, D = r.standard_normal(H), r.standard_normal(H)
    y = plain.ssd_recurrence(x, B, C, dt, A, D)
    t, h = 6, 1
    want = sum(np.exp(-np.exp(A[h]) * dt[s + 1:t + 1, h].sum()) * dt[s, h] * (C[t, h] @ B[s, h]) * x[s, h] for s in range(t + 1)) + D[h] * x[t, h]
    assert np.allclose(y[t, h], want)


def test_plain_convolution_and_router():
    x, w = np.arange(8.0).reshape(4, 2), np.array([[1.0, 10.0, 100.0], [0.0, 0.0, 1.0]])
    y = plain.causal_conv(x, w, np.array([0.5, 0.0]))
    assert np.allclose(y[:, 0], [0.5, 200.5, 420.5, 642.5]) and np.allclose(y[:, 1], x[:, 1])
    idx, wt = plain.route(np.log(np.array([0.1, 0.2, 0.3, 0.4])), np.array([0.5, 0.0, 0.0, -0.3]), 2)
    assert list(idx) == [0, 2] and np.allclose(wt, [0.25, 0.75])


def test_plain_rotation():
    v = np.arange(1.0, 7.0)[None]
    out = plain.rotate_half(v, [3], 100.0, 4)
    a0, a1 = 3.0, 3.0 * 100.0 ** -0.5
    assert np.allclose(out[0], [1 * np.cos(a0) - 3 * np.sin(a0), 2 * np.cos(a1) - 4 * np.sin(a1),
                                3 * np.cos(a0) + 1 * np.sin(a0), 4 * np.cos(a1) + 2 * np.sin(a1), 5, 6])
