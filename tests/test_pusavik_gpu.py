"""The layer-list decoder on the GPU against the plain implementation: whole models in every way a sequence can be cut."""
import json
import os
import subprocess
import sys

import numpy as np
import pytest

from pusavik_helpers import (Model, assert_close_bf16, assert_close_f32, configs, lat, model, moe, rng, row_error, ssm, tokens)

pytestmark = pytest.mark.gpu
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
NAMES = sorted(configs())


@pytest.mark.parametrize("name", NAMES)
def test_whole_decoded_and_portions_f32(fk, name):
    m = Model(configs()[name], seed=NAMES.index(name))
    t = tokens(m.cfg, 150)
    ref = m.plain(t)
    assert_close_f32(m.run(t), ref)                        # one portion
    assert_close_f32(m.run(t, [1]), ref)                   # token after token
    assert_close_f32(m.run(t, [3, 2, 70, 1, 1, 2, 31, 2]), ref)
    assert_close_f32(m.run(t, [100, 1]), ref)              # a prompt, then decoding


@pytest.mark.parametrize("name", NAMES)
def test_whole_decoded_and_portions_bf16(fk, name):
    m = Model(configs()[name], seed=NAMES.index(name), act=16)
    t = tokens(m.cfg, 150)
    ref = m.plain(t)
    forced = name == "all_experts"
    for cuts in (None, [1], [3, 2, 70, 1, 1, 2, 31, 2], [100, 1], [64]):
        assert_close_bf16(m.run(t, cuts), ref, forced)


@pytest.mark.parametrize("name", ["mixed", "long_window", "all_experts"])
def test_forms_agree_bf16(fk, name):
    """Row forms, tiles and the fused decode launches are the same function up to rounding."""
    c = configs()[name]
    t = tokens(c, 140, 5)
    a = Model(c, seed=7, act=16)
    assert a.rt.fused
    rows = Model(c, seed=7, act=16, tiled=False, fuse=False, tensors=a.tensors)
    plainlist = Model(c, seed=7, act=16, fuse=False, tensors=a.tensors)
    assert not rows.rt.fused and not plainlist.rt.fused
    ref = a.plain(t)
    for m in (a, rows, plainlist):
        assert_close_bf16(m.run(t), ref, name == "all_experts")
        assert_close_bf16(m.run(t, [90, 1]), ref, name == "all_experts")


@pytest.mark.parametrize("act", [32, 16])
def test_passes_shorter_than_the_portion_and_rings_that_wrap(fk, act):
    """rows_per_pass 70: several passes per portion, rings of window + 69 rows written over several times."""
    c = configs()["long_window"]
    m = Model(c, seed=2, act=act, rows_per_pass=70)
    t = tokens(c, 420, 3)
    ref = m.plain(t)
    check = assert_close_f32 if act == 32 else assert_close_bf16
    check(m.run(t), ref)
    check(m.run(t, [70, 70, 33, 2]), ref)
    check(m.run(t, [389, 1]), ref)
    check(m.run(t, [7]), ref)


@pytest.mark.parametrize("act", [32, 16])
def test_long_decoding(fk, act):
    m = Model(configs()["mixed"], seed=4, act=act)
    t = tokens(m.cfg, 330, 6)
    (assert_close_f32 if act == 32 else assert_close_bf16)(m.run(t, [2, 1]), m.plain(t))


@pytest.mark.parametrize("act", [32, 16])
def test_a_state_used_again_is_a_fresh_one(fk, act):
    m = Model(configs()["mixed"], seed=5, act=act)
    a, b = tokens(m.cfg, 120, 8), tokens(m.cfg, 90, 9)
    fresh = m.run(b, [40, 1])
    m.run(a, [100, 1])
    assert np.array_equal(m.run(b, [40, 1]), fresh)
    m.run(a, [2, 1])
    assert np.array_equal(m.run(b, [40, 1]), fresh)
    assert row_error(m.run(b[:1]), m.plain(b[:1])).max() < (3e-5 if act == 32 else 0.08)


def test_wanted_places(fk):
    m = Model(configs()["mixed"], seed=6)
    t = tokens(m.cfg, 200, 2)
    ref = m.plain(t)
    m.rt.reset()
    assert m.rt.step(t[:90]).shape == (0, m.cfg.vocab)
    assert_close_f32(m.rt.step(t[90:], [5, 0, 109, 5]), ref[[95, 90, 199, 95]])
    m.rt.reset()
    assert_close_f32(m.rt.step(t, range(200)), ref)     # more than one group of head rows
    for bad in ([], [-1], [m.cfg.vocab]):
        with pytest.raises(ValueError):
            m.rt.step(bad)


def spiked(c, seed, act, gain):
    """A model whose attention is sharp: queries and keys scaled so that single keys stand out."""
    from fusekit_amd.layer_decoder import bf16_to_f32, f32_to_bf16, random_tensors
    t = random_tensors(c, seed)
    for n in t:
        if n.endswith((".mix.uk", ".mix.uq")):
            t[n] = f32_to_bf16(bf16_to_f32(t[n]) * gain)
    return Model(c, act=act, tensors=t)


@pytest.mark.parametrize("window", [2, 63, 64, 65, 127, 129])
def test_window_edges_in_prompts_and_decoding(fk, window):
    """Sharp attention: a window one token off changes the logits far beyond the limit (checked on the plain side)."""
    c = model([(lat(heads=2, dim=32, rot_dim=16, vdim=32, kv_rank=64, window=window), None)], width=64)
    m = spiked(c, 11, 32, 3.0)
    t = tokens(c, 200, 12)
    ref = m.plain(t)
    off = dict(m.json)
    from oracle import pusavik as plain
    for d in (-1, 1):
        off["layers"] = [dict(m.json["layers"][0], mixer=dict(m.json["layers"][0]["mixer"], mask=dict(size=window + d)))]
        assert row_error(plain.forward(off, m.w, t)[0], ref).max() > 20 * 3e-5
    for cuts in (None, [1], [130, 1], [2], [66, 63, 2]):
        assert_close_f32(m.run(t, cuts), ref)
    b = spiked(c, 11, 16, 3.0)
    for cuts in (None, [1], [130, 1], [66, 63, 2]):
        e = row_error(b.run(t, cuts), ref)
        assert np.median(e) < 0.03 and e.max() < 0.25, e.max()


def test_greedy_generation_through_the_scheduler(fk):
    m = Model(configs()["mixed"], seed=3)
    p = tokens(m.cfg, 37, 4)
    seq = list(p)
    for _ in range(20):
        seq.append(int(np.argmax(m.plain(seq)[-1])))
    toks, _, steps = m.rt.generate(p, 20)
    assert toks == seq[37:] and steps == 19
    assert m.rt.generate(p, 20)[0] == toks                  # a second sequence starts from nothing
    assert m.rt.generate(p[:1], 3)[0] == m.rt.generate(p[:1], 3)[0]
    b = Model(m.cfg, act=16, tensors=m.tensors)
    got = b.rt.generate(p, 70)[0]                           # more than one chunk, fed back on the GPU
    b.rt.reset()
    logits = b.rt.step(p, [len(p) - 1])
    for k, tok in enumerate(got):
        assert tok == int(np.argmax(logits[-1])), k
        logits = b.rt.step([tok], [0])


def test_replays_repeat_bit_for_bit(fk):
    m = Model(configs()["all_experts"], seed=9, act=16)
    t = tokens(m.cfg, 80, 2)
    first = m.run(t, [70, 1])
    for _ in range(3):
        assert np.array_equal(m.run(t, [70, 1]), first)


def test_command_line_artifact_and_trace(fk, tmp_path, capsys, monkeypatch):
    from fusekit_amd import __main__ as cli
    d = str(tmp_path / "m")

    def run(*argv):
        monkeypatch.setattr(sys, "argv", ["fusekit_amd", *argv])
        assert cli.main() == 0
        return capsys.readouterr().out

    run("export-random", "--out", d, "--pusavik", "--hidden", "96", "--heads", "2", "--inter", "56", "--vocab", "300")
    ids = "5,17,290,3,3,8"
    a = json.loads(run("generate", "--model", d, "--ids", ids, "--max-tokens", "12"))["tokens"]
    assert len(a) == 12
    f = json.loads(run("generate", "--model", d, "--ids", ids, "--max-tokens", "12", "--dtype", "float32"))["tokens"]
    assert len(f) == 12
    run("patch", "--model", d)
    art = json.loads(run("generate", "--model", d, "--artifact", d + "/.fusekit", "--ids", ids, "--max-tokens", "12"))["tokens"]
    assert len(art) == 12 and art[0] < 300
    out = run("bench", d, "--tokens", "8", "--ids", ids, "--dump-tokens", "--per-kernel")
    assert f"tokens={a[:8]}" in out

    # the trace runner: the same logits as the runtime's own steps
    from fusekit_amd import registry
    fam = registry.family_of(registry.read_config(d))
    rt = fam.runtime(*fam.load(d, 64, 32))
    seq = [int(t) for t in ids.split(",")]
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": seq[:4], "want": [1, 3]}], "end": []},
             {"step": 1, "entries": [{"id": "a", "tokens": seq[4:5], "want": []}], "end": []},
             {"step": 2, "entries": [{"id": "a", "tokens": seq[5:], "want": [0]}], "end": ["a"]},
             {"step": 3, "entries": [{"id": "b", "tokens": seq[:4], "want": [3]}], "end": ["b"]}]
    odir = tmp_path / "out"
    odir.mkdir()
    r = subprocess.run([os.path.join(ROOT, "bin", "trace_run"), "--model", d, "--dtype", "float32", "--out", str(odir), "--max-tokens", "64"],
                       input="".join(json.dumps(s) + "\n" for s in steps), capture_output=True, text=True, timeout=100)
    assert r.returncode == 0, r.stderr
    assert [l for l in r.stdout.splitlines() if l.startswith("done")] == [f"done {i}" for i in range(4)]
    rt.reset()
    want = rt.step(seq[:4], [1, 3])
    got = np.fromfile(odir / "0.f32", "<f4").reshape(2, 300)
    assert np.array_equal(got, want)
    assert not (odir / "1.f32").exists()
    rt.step(seq[4:5])
    assert np.array_equal(np.fromfile(odir / "2.f32", "<f4"), rt.step(seq[5:], [0])[0])
    assert np.array_equal(np.fromfile(odir / "3.f32", "<f4"), want[1])


def test_trace_runner_with_another_family(fk, tmp_path):
    from fusekit_amd.checkpoint import save_mlx_checkpoint
    from fusekit_amd.decoder import DecoderConfig, DecoderRuntime, DecoderWeights
    cfg = DecoderConfig(n_layers=2, hidden=256, n_heads=4, n_kv=2, head_dim=64, inter=512, vocab=500, capacity=64, qk_norm=True, swiglu_variant=1)
    w = DecoderWeights.random_init(cfg, seed=1)
    d = tmp_path / "dense"
    save_mlx_checkpoint(str(d), cfg, w)
    line = json.dumps({"step": 0, "entries": [{"id": "x", "tokens": [3, 14, 15], "want": [0, 2]}], "end": ["x"]}) + "\n"
    cmd = [os.path.join(ROOT, "bin", "trace_run"), "--model", str(d), "--out", str(tmp_path), "--max-tokens", "64"]
    r = subprocess.run(cmd, input=line, capture_output=True, text=True, timeout=100)
    assert r.returncode == 0, r.stderr
    rt = DecoderRuntime(cfg, w)
    rt.reset()
    assert np.array_equal(np.fromfile(tmp_path / "0.f32", "<f4").reshape(2, 500), rt.step([3, 14, 15], [0, 2]))
    assert subprocess.run(cmd + ["--dtype", "float32"], input=line, capture_output=True, text=True, timeout=100).returncode == 3
