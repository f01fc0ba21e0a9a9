"""The joint layers without a GPU: configuration, layouts, and the plain implementation against closed forms."""
import json

import numpy as np
import pytest

from fumotar_helpers import att, configs, delta, lru, mlp, model, stretch
from fusekit_amd import registry
from fusekit_amd.checkpoint import SafetensorsFile, layer_config_from_json, layer_config_to_json, save_layer_checkpoint
from fusekit_amd.joint_layers import Columns, spread
from fusekit_amd.layer_decoder import Experts, Layer, random_tensors, small_joint_config, tensor_shapes
from oracle import fumotar as plain

NAMES = sorted(configs())


@pytest.mark.parametrize("name", NAMES + ["small"])
def test_config_round_trip(name):
    c = small_joint_config() if name == "small" else configs()[name]
    j = json.loads(json.dumps(layer_config_to_json(c)))
    assert registry.family_of(j).name == "layer-list" and registry.vocab_of(j) == c.vocab
    back = layer_config_from_json(j, {}, capacity=c.capacity)
    assert back == c and tensor_shapes(back) == tensor_shapes(c)


def test_ranks_from_the_tensors_and_refused_configs():
    c = configs()["no_loop"]
    j = layer_config_to_json(c)
    m = j["layers"][0]["mixer"]
    del m["decay_rank"], m["gate_rank"]
    shapes = tensor_shapes(c)
    assert layer_config_from_json(j, shapes, capacity=c.capacity) == c
    for change, text in ((lambda x: x["layers"][2]["mixer"].update(vdim=8), "widths must agree"), (lambda x: x["layers"][2]["mlp"].update(kind="gated"), "feed-forward"),
                         (lambda x: x["layers"][1]["mixer"].update(blocks=3), "multiple of blocks"), (lambda x: x["layers"][0].update(type="other"), "mixer type"),
                         (lambda x: x.update(architecture="Other"), "architecture")):
        bad = json.loads(json.dumps(layer_config_to_json(c)))
        change(bad)
        with pytest.raises(ValueError, match=text):
            layer_config_from_json(bad, shapes)
    with pytest.raises(ValueError, match="feed-forward"):
        Layer(att(), Experts(experts=2, identity=0, top=1, ff=8))


def test_tensors_of_a_checkpoint(tmp_path):
    c = configs()["mixed"]
    t = random_tensors(c, 3)
    save_layer_checkpoint(str(tmp_path), c, t)
    f = SafetensorsFile(str(tmp_path / "model.safetensors"))
    shapes = {n: tuple(v["shape"]) for n, v in f.tensors.items()}
    assert shapes == tensor_shapes(c)
    assert "head" not in shapes and shapes["bigram"] == (62, 72) and shapes["loop.in"] == (72, 144) and shapes["l0.norm1.b"] == (72,)
    assert shapes["l1.mix.a2"] == (80, 12) and shapes["l2.mix.ra"] == (3, 30, 30) and "l3.mlp.up" not in shapes


@pytest.mark.parametrize("name", NAMES)
def test_columns_of_a_joint_row(name):
    for l in configs()[name].layers:
        m, c = l.mixer, Columns(l.mixer, l.mlp)
        assert c.width % 64 == 0 and c.out % 64 == 0 and c.ko % 64 == 0
        assert c.out + dict(m.parts())[m.out_part] == c.up   # the mixer's result lies directly ahead of `up`
        assert c.rows - c.width == (m.heads if m.kind == "channel_delta" else 0)


def test_parts_of_a_long_sum():
    from fusekit_amd.joint_layers import out_parts
    for n, k in ((72, 192), (2048, 10240), (4096, 20480), (1024, 64 * 7)):
        for rows in (1, 8, 9, 32, 33, 64, 500, 2048):
            p = out_parts(rows, n, k)
            assert k % (64 * p) == 0 and (p == 1 or k // p >= 512) and (rows > 8 or p == 1)
    assert out_parts(16, 2048, 10240) == 8 and out_parts(2048, 4096, 20480) == 1


def test_spread_rows():
    a = np.arange(12).reshape(6, 2)
    s = spread(a, 2, 4)
    assert s.shape == (8, 2) and np.array_equal(s[:3], a[:3]) and np.array_equal(s[4:7], a[3:]) and not s[3].any() and not s[7].any()


def test_rotation_tables():
    for m in (att(), att(rot_dims=24, rot_scaling=stretch()), att(rot_dims=2, rot_scaling=stretch(slow=12.0)), att(rot_dims=0)):
        j = layer_config_to_json(model([(m, None)]))["layers"][0]["mixer"]["rot"]
        f, mag = plain.rot_frequencies(j)
        g, mine = m.rotation()
        assert np.allclose(f, g, rtol=1e-14) and np.isclose(mag, mine)
    # far beyond both bounds every frequency is divided, far below none is
    m = att(dim=64, rot_dims=64, rot_base=1e4, rot_scaling=stretch(original=1e12, fast=2e11, slow=1e11))
    assert np.allclose(m.rotation()[0][-4:] * 3.0, 1e4 ** (-2.0 * np.arange(28, 32) / 64)) and m.rotation()[0][0] == 1.0


# ---- the plain implementation against closed forms ----

def test_plain_delta_rule_writes_and_reads_back():
    """With no decay and step size 1 a key reads back the last value written under it."""
    K = np.eye(4)
    v = np.arange(1.0, 7.0)[:, None, None] * np.ones((6, 1, 3))
    k = K[[0, 1, 2, 0, 3, 1]][:, None]
    o = plain.delta_recurrence(k, k, v, np.ones((6, 1)), np.zeros((6, 1, 4)))
    assert np.allclose(o[:, 0], v[:, 0])
    q = K[[0, 0, 0, 0, 0, 1]][:, None]
    o = plain.delta_recurrence(q, k, v, np.ones((6, 1)), np.zeros((6, 1, 4)))
    assert np.allclose(o[:, 0, 0], [1, 1, 1, 4, 4, 6])
    # channel 0 decays by half a token, the others not at all
    g = np.zeros((6, 1, 4))
    g[:, :, 0] = np.log(0.5)
    o = plain.delta_recurrence(q, k, v, np.ones((6, 1)), g)
    assert np.allclose(o[:, 0, 0], [1, 0.5, 0.25, 4, 2, 6])


def test_plain_linear_recurrence_is_the_decayed_sum():
    r = np.random.Generator(np.random.PCG64(0))
    u, rr, ii, lam = r.standard_normal((7, 3)), r.random((7, 3)), r.random((7, 3)), r.standard_normal(3)
    a = np.exp(-8.0 * rr * np.log1p(np.exp(lam)))
    want = sum(np.prod(a[s + 1:], 0) * np.sqrt(1 - a[s] ** 2) * ii[s] * u[s] for s in range(7))
    assert np.allclose(plain.gated_recurrence(u, rr, ii, lam)[-1], want)


def test_plain_rows_of_the_pair_table():
    assert plain.bigram_rows([3, 4, 3], 7, 2, 11) == [11, (21 + 8) % 11, (28 + 6) % 11]
    x = np.array([[1.0, 2.0, 6.0]])
    assert np.allclose(plain.layer_norm(x, np.ones(3), np.array([0.0, 0.0, 1.0]), 0.0), (x - 3) / np.sqrt(14 / 3) + [0, 0, 1])
    assert np.allclose(plain.relu2(np.array([-2.0, 3.0])), [0, 9])


def test_plain_attention_values_are_raw_keys():
    """One visible key: the output is its projection, whatever norms and rotations do."""
    c = model([(att(heads=4, kv_heads=2, dim=8, rot_dims=8), mlp())])
    j, t = layer_config_to_json(c), random_tensors(c, 1)
    from fusekit_amd.layer_decoder import bf16_to_f32
    w = {n: bf16_to_f32(a).astype(np.float64) for n, a in t.items()}
    h = np.random.Generator(np.random.PCG64(1)).standard_normal((1, 72))
    got = plain.attention(h, w, "l0.mix.", j["layers"][0]["mixer"], 1e-5)
    v = (w["l0.mix.k"] @ h[0]).reshape(2, 8)[[0, 0, 1, 1]].reshape(-1)
    assert np.allclose(got[0], w["l0.mix.o"] @ v)


def test_the_recurrent_state_does_not_limit_a_sequence():
    assert model([(lru(), None), (delta(), mlp())]).max_positions is None and configs()["mixed"].max_positions == 512
