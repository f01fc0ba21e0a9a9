"""Shared pieces of the joint layers' tests: small models with random weights beside the plain float64 implementation."""
from __future__ import annotations

import numpy as np

from oracle import fumotar as plain
from pusavik_helpers import row_error


def att(**k):
    from fusekit_amd.layer_decoder import CausalAttention
    d = dict(heads=6, kv_heads=3, dim=24, scale=0.17, rot_base=3000.0, rot_dims=16)
    d.update(k)
    return CausalAttention(**d)


def stretch(**k):
    from fusekit_amd.layer_decoder import RotaryScaling
    d = dict(factor=3.0, original=400, fast=12.0, slow=1.5)
    d.update(k)
    return RotaryScaling(**d)


def delta(**k):
    from fusekit_amd.layer_decoder import ChannelDelta
    d = dict(heads=4, kv_heads=2, dim=20, vdim=28, conv=4, decay_rank=12, gate_rank=18)
    d.update(k)
    return ChannelDelta(**d)


def lru(**k):
    from fusekit_amd.layer_decoder import RgLru
    d = dict(width=90, blocks=3, conv=3)
    d.update(k)
    return RgLru(**d)


def mlp(ff=52):
    from fusekit_amd.layer_decoder import DenseMlp
    return DenseMlp(ff)


def model(layers, **k):
    from fusekit_amd.layer_decoder import Layer, LayerConfig, PairTable
    d = dict(width=72, vocab=150, eps=1e-5, design="Fumotar", layer_norm=True, tied=True, join=True, pairs=PairTable(buckets=61, mul_prev=19, mul_cur=5), capacity=512)
    d.update(k)
    return LayerConfig(layers=[Layer(*l) for l in layers], **d)


# odd widths, one head, equal head counts, no feed-forward, no loop, loops over a part and over everything, rotation of a
# part of the head / of all / of nothing, with and without stretching, one tap, one block, ranks above and below a row of padding
def configs():
    return {
        "mixed": model([(att(rot_scaling=stretch()), mlp()), (delta(), mlp(100)), (lru(), mlp()), (att(heads=2, kv_heads=2, dim=64, rot_dims=64, scale=0.125), None)],
                       loop_start=1, loop_stop=3, loop_times=2),
        "loop_all": model([(lru(width=48, blocks=1, conv=1), mlp(64)), (att(heads=3, kv_heads=1, dim=40, rot_dims=40, rot_scaling=stretch(factor=2.0, original=64, fast=4.0, slow=1.0)), mlp(30)),
                           (delta(heads=3, kv_heads=3, dim=33, vdim=64, conv=1, decay_rank=70, gate_rank=3), mlp())], width=100, loop_start=0, loop_stop=3, loop_times=3),
        "no_loop": model([(delta(heads=6, kv_heads=1, dim=64, vdim=20, conv=2), None), (lru(width=140, blocks=2, conv=5), None), (att(dim=136, heads=2, kv_heads=1, rot_dims=0), mlp(200))],
                         width=64, eps=1e-3),
        "wide": model([(delta(heads=2, kv_heads=2, dim=130, vdim=96, conv=6), mlp(300)), (att(heads=4, kv_heads=2, dim=128, rot_dims=96, scale=0.09), mlp(128)), (lru(width=256, blocks=2, conv=4), mlp(64))],
                      width=192, loop_start=2, loop_stop=3, loop_times=2),
        "delta_pair": model([(delta(heads=4, kv_heads=4, dim=128, vdim=128, conv=4, decay_rank=64, gate_rank=64), mlp(64)), (delta(heads=2, kv_heads=1, dim=96, vdim=32, conv=3), mlp())], width=128),
    }


class Model:
    """One model twice: the runtime and the plain implementation."""

    def __init__(self, cfg, seed=0, act=32, tensors=None, **over):
        import dataclasses

        from fusekit_amd.checkpoint import layer_config_to_json
        from fusekit_amd.layer_decoder import LayerRuntime, LayerWeights, bf16_to_f32, random_tensors
        self.cfg = dataclasses.replace(cfg, act=act, **over)
        self.tensors = random_tensors(cfg, seed) if tensors is None else tensors
        self.json = layer_config_to_json(cfg)
        self.w = {n: bf16_to_f32(a).astype(np.float64) for n, a in self.tensors.items()}
        self.rt = LayerRuntime(self.cfg, LayerWeights.from_tensors(self.cfg, lambda n: self.tensors[n]))
        self.rt.reset()

    def plain(self, tokens):
        return plain.forward(self.json, self.w, tokens)[0]

    def run(self, tokens, cuts=None):
        """Logits of every position, the sequence cut into portions of the given sizes (the last repeats)."""
        self.rt.reset()
        out, at, k = [], 0, 0
        while at < len(tokens):
            n = len(tokens) - at if cuts is None else min(cuts[min(k, len(cuts) - 1)], len(tokens) - at)
            out.append(self.rt.step(tokens[at:at + n], range(n)))
            at += n
            k += 1
        return np.concatenate(out)


# 32-bit runs differ from the float64 statement by rounding only
F32_LIMIT = 3e-5


def assert_close_f32(got, ref):
    e = row_error(got, ref)
    assert e.max() <= F32_LIMIT, (e.max(), int(e.argmax()))


def assert_close_bf16(got, ref, limit=0.06):
    """bf16 matrices, activations and caches: nothing in these layers chooses, so no position is an exception."""
    e = row_error(got, ref)
    assert np.median(e) <= limit / 3 and e.max() <= limit, (np.median(e), e.max(), int(e.argmax()))
