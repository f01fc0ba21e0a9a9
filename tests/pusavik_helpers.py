"""Shared pieces of the layer-list decoder's tests: small models with random weights, the plain float64 implementation
beside them, and error measures."""
from __future__ import annotations

import numpy as np

from oracle import pusavik as plain


def rng(seed):
    return np.random.Generator(np.random.PCG64(seed))


def bf16_round(a):
    from fusekit_amd.layer_decoder import bf16_to_f32, f32_to_bf16
    return bf16_to_f32(f32_to_bf16(a))


def lat(**k):
    from fusekit_amd.layer_decoder import LatentAttention
    d = dict(heads=3, dim=24, rot_dim=12, vdim=20, kv_rank=40, q_rank=56, window=21, scale=0.21, rot_base=5000.0)
    d.update(k)
    d.setdefault("rot_dims", d["rot_dim"])
    return LatentAttention(**d)


def ssm(**k):
    from fusekit_amd.layer_decoder import Mamba2
    d = dict(heads=6, vdim=12, state=24, groups=3, conv=4, norm_groups=2)
    d.update(k)
    return Mamba2(**d)


def moe(**k):
    from fusekit_amd.layer_decoder import Experts
    d = dict(experts=5, identity=2, top=3, ff=40)
    d.update(k)
    return Experts(**d)


def model(layers, **k):
    from fusekit_amd.layer_decoder import Layer, LayerConfig
    d = dict(width=72, vocab=150, eps=1e-5, embed_scale=1.7)
    d.update(k)
    return LayerConfig(layers=[Layer(*l) for l in layers], **d)


# several shapes: odd widths, one head, one group, no feed-forward, no identities, every expert chosen, no loop, a loop over
# each kind of layer, windows below and above a tile, forms that the matrix-core kernels do not take
def configs():
    return {
        "mixed": model([(lat(), moe()), (ssm(), moe()), (lat(window=70), None), (ssm(conv=2, norm_groups=1), moe(identity=0, top=1))],
                       loop_start=1, loop_stop=3, loop_times=2),
        "all_experts": model([(ssm(heads=4, vdim=16, state=32, groups=1, norm_groups=4), moe(experts=3, identity=1, top=4, ff=64)),
                              (lat(heads=17, dim=32, rot_dim=32, vdim=32, kv_rank=64, q_rank=64, window=33), moe(experts=4, identity=0, top=4))], width=128),
        "loop_first": model([(lat(window=1), moe(top=2)), (ssm(conv=1), None)], width=100, loop_start=0, loop_stop=2, loop_times=3),
        "wide": model([(lat(heads=2, dim=264, rot_dim=16, vdim=40, kv_rank=584, q_rank=24, window=64), moe()),
                       (ssm(heads=2, vdim=22, state=130, groups=2, conv=5, norm_groups=2), moe(ff=100))], width=64),
        "long_window": model([(lat(heads=4, dim=64, rot_dim=64, vdim=64, kv_rank=128, window=200), moe(experts=9, top=2)),
                              (ssm(heads=8, vdim=32, state=64, groups=2, norm_groups=8), moe(experts=9, top=2)), (lat(window=64), moe())],
                             width=192, loop_start=2, loop_stop=3, loop_times=2),
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


def tokens(cfg, n, seed=1):
    return rng(seed).integers(0, cfg.vocab, n).tolist()


def row_error(got, ref):
    """Per position: RMS difference over the spread of the reference logits."""
    d = got.astype(np.float64) - ref
    d -= d.mean(-1, keepdims=True)
    return np.sqrt((d * d).mean(-1)) / ref.std()


# 32-bit runs differ from the float64 statement by rounding only
F32_LIMIT = 3e-5


def assert_close_f32(got, ref):
    e = row_error(got, ref)
    assert e.max() <= F32_LIMIT, (e.max(), int(e.argmax()))


def assert_close_bf16(got, ref, forced=False):
    """bf16 activations: a close call of a router may choose another expert at a few positions (never when every expert is
    chosen anyway: `forced`)."""
    e = row_error(got, ref)
    assert np.median(e) <= 0.03, np.median(e)
    assert np.quantile(e, 1.0 if forced else 0.9) <= 0.08, np.sort(e)[-5:]
