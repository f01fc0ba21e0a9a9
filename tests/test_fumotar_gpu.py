"""The joint layers on the GPU against the plain implementation: whole models in every way a sequence can be cut."""
import json
import os
import subprocess
import sys

import numpy as np
import pytest

from fumotar_helpers import F32_LIMIT, Model, assert_close_bf16, assert_close_f32, att, configs, delta, lru, mlp, model
from oracle import fumotar as plain
from pusavik_helpers import row_error, tokens

pytestmark = pytest.mark.gpu
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
NAMES = sorted(configs())
CUTS = (None, [1], [3, 2, 70, 1, 1, 2, 31, 2], [100, 1], [64])


@pytest.mark.parametrize("name", NAMES)
def test_whole_decoded_and_portions_f32(fk, name):
    m = Model(configs()[name], seed=NAMES.index(name))
    t = tokens(m.cfg, 150)
    ref = m.plain(t)
    for cuts in CUTS:
        assert_close_f32(m.run(t, cuts), ref)


@pytest.mark.parametrize("name", NAMES)
def test_whole_decoded_and_portions_bf16(fk, name):
    m = Model(configs()[name], seed=NAMES.index(name), act=16)
    assert m.rt.fused
    t = tokens(m.cfg, 150)
    ref = m.plain(t)
    for cuts in CUTS + ([2], [16, 17, 1]):
        assert_close_bf16(m.run(t, cuts), ref)


@pytest.mark.parametrize("name", NAMES)
def test_forms_agree_bf16(fk, name):
    """Row forms, tiles and the fused launches of one token are the same function up to rounding."""
    c = configs()[name]
    t = tokens(c, 140, 5)
    a = Model(c, seed=7, act=16)
    ref = a.plain(t)
    for over in ({}, dict(tiled=False, fuse=False), dict(fuse=False)):
        m = Model(c, act=16, tensors=a.tensors, **over)
        assert m.rt.fused == (not over)
        assert_close_bf16(m.run(t), ref)
        assert_close_bf16(m.run(t, [90, 1]), ref)


@pytest.mark.parametrize("act", [32, 16])
def test_passes_shorter_than_the_portion(fk, act):
    """rows_per_pass 70: several passes per portion, whole ones replayed as a graph, into a cache they fill to the last row."""
    m = Model(configs()["mixed"], seed=2, act=act, rows_per_pass=70, capacity=420)
    t = tokens(m.cfg, 420, 3)
    ref = m.plain(t)
    check = assert_close_f32 if act == 32 else assert_close_bf16
    for cuts in (None, [70, 70, 33, 2], [389, 1], [7]):
        check(m.run(t, cuts), ref)
    with pytest.raises(ValueError, match="420 positions"):
        m.rt.step(t[:1])
    with pytest.raises(ValueError, match="420 positions"):
        m.rt.reset() or m.rt.step(t + t[:1])


@pytest.mark.parametrize("act", [32, 16])
def test_long_decoding(fk, act):
    m = Model(configs()["mixed"], seed=4, act=act)
    t = tokens(m.cfg, 400, 6)
    (assert_close_f32 if act == 32 else assert_close_bf16)(m.run(t, [2, 1]), m.plain(t))


@pytest.mark.parametrize("act", [32, 16])
def test_a_state_used_again_is_a_fresh_one(fk, act):
    m = Model(configs()["loop_all"], seed=5, act=act)
    a, b = tokens(m.cfg, 120, 8), tokens(m.cfg, 90, 9)
    fresh = m.run(b, [40, 1])
    for cuts in ([100, 1], [2, 1]):
        m.run(a, cuts)
        assert np.array_equal(m.run(b, [40, 1]), fresh)
    first = m.run(b[:1])
    assert row_error(first, m.plain(b[:1])).max() < (F32_LIMIT if act == 32 else 0.06)
    m.run(a, [1])
    assert np.array_equal(m.run(b[:1]), first)                 # no token before the first, whatever ran


def test_wanted_places(fk):
    m = Model(configs()["mixed"], seed=6)
    t = tokens(m.cfg, 200, 2)
    ref = m.plain(t)
    m.rt.reset()
    assert m.rt.step(t[:90]).shape == (0, m.cfg.vocab)
    assert_close_f32(m.rt.step(t[90:], [5, 0, 109, 5]), ref[[95, 90, 199, 95]])


def edited(c, seed, act, change):
    """A model whose tensors were changed to make one mechanism show."""
    from fusekit_amd.layer_decoder import bf16_to_f32, f32_to_bf16, random_tensors
    t = random_tensors(c, seed)
    for n in t:
        v = change(n, bf16_to_f32(t[n]))
        if v is not None:
            t[n] = f32_to_bf16(v)
    return Model(c, act=act, tensors=t)


@pytest.mark.parametrize("dim,heads,kv", [(24, 4, 2), (64, 2, 1), (128, 2, 2)])
def test_single_far_keys_decide(fk, dim, heads, kv):
    """Unrotated sharp attention over repeating tokens: every position's logits hang on the few earlier places of a token.
    That dropping one of them shows is checked on the plain side."""
    c = model([(att(dim=dim, heads=heads, kv_heads=kv, rot_dims=0, scale=8.0 * dim ** -0.5), None)], width=64, vocab=40)
    gain = lambda n, v: 2.0 * v if n.endswith(("q.norm", "k.norm", "mix.o")) else None
    m = edited(c, 11, 32, gain)
    t = tokens(c, 300, 12)
    t[200:] = t[:100]                                            # what was seen 200 positions ago
    ref = m.plain(t)
    gone = m.plain(t[:40] + [(x + 1) % c.vocab for x in t[40:42]] + t[42:])
    assert row_error(gone, ref)[242:].max() > 20 * F32_LIMIT
    for cuts in (None, [1], [199, 1], [64, 2], [63, 65, 1]):
        assert_close_f32(m.run(t, cuts), ref)
    b = edited(c, 11, 16, gain)
    for cuts in (None, [1], [199, 1], [64, 2]):
        assert_close_bf16(b.run(t, cuts), ref, 0.15)


@pytest.mark.parametrize("heads,kv,dim,capacity", [(5, 1, 40, 256), (8, 1, 64, 256), (12, 4, 32, 300), (4, 1, 96, 2500), (3, 3, 128, 2500), (1, 1, 8, 64 * 3), (2, 1, 160, 256)])
def test_head_groups_and_capacities(fk, heads, kv, dim, capacity):
    c = model([(att(heads=heads, kv_heads=kv, dim=dim, rot_dims=dim // 2 // 2 * 2, scale=2.0 * dim ** -0.5), mlp()), (att(heads=heads, kv_heads=kv, dim=dim, rot_dims=dim), None)],
              width=64, capacity=capacity)
    a, b = Model(c, seed=1), Model(c, seed=1, act=16)
    t = tokens(c, 190)
    ref = a.plain(t)
    for cuts in (None, [1], [130, 1], [17, 2, 70, 9]):
        assert_close_f32(a.run(t, cuts), ref)
        assert_close_bf16(b.run(t, cuts), ref)


@pytest.mark.parametrize("act", [32, 16])
def test_state_that_is_kept_for_long(fk, act):
    """Almost no decay: the first tokens still decide after hundreds; a state lost at a portion's edge would show."""
    c = model([(delta(heads=2, kv_heads=2, dim=64, vdim=64), mlp()), (lru(), mlp())], width=64)
    change = lambda n, v: v * 0 - 7.0 if n.endswith(("dt_bias", "lam")) else v * 0 - 2.0 if n.endswith("mix.b") else None
    m = edited(c, 3, act, change)
    t = tokens(c, 330, 4)
    ref = m.plain(t)
    other = m.plain([(x + 3) % c.vocab for x in t[:8]] + t[8:])
    assert row_error(other, ref)[300:].max() > 20 * F32_LIMIT
    for cuts in CUTS + ([65, 63, 64], [2]):
        (assert_close_f32 if act == 32 else assert_close_bf16)(m.run(t, cuts), ref)


@pytest.mark.parametrize("act", [32, 16])
def test_decays_that_wipe_the_state(fk, act):
    """Strong decays per channel: exponents of a whole chunk far beyond the range of a float."""
    c = model([(delta(heads=2, kv_heads=1, dim=96, vdim=64), mlp()), (lru(), mlp())], width=64)
    change = lambda n, v: np.where(np.arange(v.size).reshape(v.shape) % 5 < 2, 9.0, -6.0) if n.endswith(("dt_bias", "lam")) else v * 0 + 2.5 if n.endswith("A_log") else None
    m = edited(c, 5, act, change)
    t = tokens(c, 200, 6)
    ref = m.plain(t)
    for cuts in CUTS:
        (assert_close_f32 if act == 32 else assert_close_bf16)(m.run(t, cuts), ref)


@pytest.mark.parametrize("act", [32, 16])
def test_pairs_of_tokens_across_portions(fk, act):
    """Only the table of pairs tells one first token from another here."""
    c = model([(lru(), mlp())], width=64)
    m = edited(c, 8, act, lambda n, v: v * 4.0 if n == "bigram" else None)
    t = tokens(c, 60, 1)
    ref = m.plain(t)
    for cuts in (None, [1], [2], [3, 1, 1, 16, 17]):
        (assert_close_f32 if act == 32 else assert_close_bf16)(m.run(t, cuts), ref)


def test_other_designs_mix(fk):
    """Untied, without pairs, without join (a learned vector ahead of a pass), RMS norms: each part stands alone."""
    for over in (dict(tied=False), dict(pairs=None), dict(join=False, loop_start=0, loop_stop=2, loop_times=2), dict(layer_norm=False), dict(embed_scale=0.5)):
        c = model([(att(), mlp()), (delta(), mlp())], **over)
        a, b = Model(c, seed=1), Model(c, seed=1, act=16)
        t = tokens(c, 100)
        whole = a.run(t)
        assert np.isfinite(whole).all()
        assert_close_f32(a.run(t, [40, 1]), whole)
        for cuts in (None, [60, 1]):
            assert_close_bf16(b.run(t, cuts), whole)


def test_greedy_generation_through_the_scheduler(fk):
    m = Model(configs()["mixed"], seed=3)
    p = tokens(m.cfg, 37, 4)
    seq = list(p)
    for _ in range(20):
        seq.append(int(np.argmax(m.plain(seq)[-1])))
    toks, _, steps = m.rt.generate(p, 20)
    assert toks == seq[37:] and steps == 19
    assert m.rt.generate(p, 20)[0] == toks                  # a second sequence starts from nothing
    one = list(p[:1])
    for _ in range(6):
        one.append(int(np.argmax(m.plain(one)[-1])))
    assert m.rt.generate(p[:1], 6)[0] == one[1:]            # a prompt of one token
    b = Model(m.cfg, act=16, tensors=m.tensors)
    got = b.rt.generate(p, 70)[0]                           # more than one chunk, fed back on the GPU
    b.rt.reset()
    logits = b.rt.step(p, [len(p) - 1])
    for k, tok in enumerate(got):
        assert tok == int(np.argmax(logits[-1])), k
        logits = b.rt.step([tok], [0])
    with pytest.raises(ValueError, match="positions"):
        Model(m.cfg, act=16, tensors=m.tensors, capacity=64).rt.generate(p, 70)


def test_replays_repeat_bit_for_bit(fk):
    m = Model(configs()["loop_all"], seed=9, act=16)
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

    run("export-random", "--out", d, "--fumotar", "--hidden", "96", "--heads", "2", "--inter", "56", "--vocab", "300")
    ids = "5,17,290,3,3,8"
    a = json.loads(run("generate", "--model", d, "--ids", ids, "--max-tokens", "12"))["tokens"]
    f = json.loads(run("generate", "--model", d, "--ids", ids, "--max-tokens", "12", "--dtype", "float32"))["tokens"]
    assert len(a) == len(f) == 12
    run("patch", "--model", d)
    art = [json.loads(run("generate", "--model", d, "--artifact", d + "/.fusekit", "--ids", ids, "--max-tokens", "12"))["tokens"] for _ in range(2)]
    from fusekit_amd import registry
    fam = registry.family_of(registry.read_config(d))
    rt = fam.runtime(*fam.load(d, 64, 16))
    rt.reset()
    seq = [int(t) for t in ids.split(",")]
    for t in seq:
        logits = rt.step([t], [0])
    want = []
    for _ in range(12):                                     # the artifact feeds the prompt through the decode graph as well
        want.append(int(np.argmax(logits)))
        logits = rt.step([want[-1]], [0])
    assert art[0] == art[1] == want
    with pytest.raises(ValueError, match="1024 positions"):
        run("generate", "--model", d, "--artifact", d + "/.fusekit", "--ids", ids, "--max-tokens", "1030")
    out = run("bench", d, "--tokens", "8", "--ids", ids, "--dump-tokens", "--per-kernel")
    assert f"tokens={a[:8]}" in out

    # the trace runner: the same logits as the runtime's own steps
    rt = fam.runtime(*fam.load(d, 64, 32))
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
    assert np.array_equal(np.fromfile(odir / "0.f32", "<f4").reshape(2, 300), want)
    assert not (odir / "1.f32").exists()
    rt.step(seq[4:5])
    assert np.array_equal(np.fromfile(odir / "2.f32", "<f4"), rt.step(seq[5:], [0])[0])
    assert np.array_equal(np.fromfile(odir / "3.f32", "<f4"), want[1])
