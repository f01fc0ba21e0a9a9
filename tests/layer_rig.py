"""Runs one dispatch family of the layer-list decoder on given arrays."""
import numpy as np

from pusavik_helpers import bf16_round


def pad(n, to=64):
    return -(-n // to) * to


class Rig:
    """Uploads operands in an activation width, runs one family, reads results back."""

    def __init__(self, act):
        from fusekit_amd import native
        from fusekit_amd.layer_decoder import bf16_to_f32, f32_to_bf16
        from fusekit_amd.runtime import Dispatch, Dispatcher, arg
        self.native, self.act, self.e = native, act, act // 8
        self.to16, self.from16, self.Dispatch, self.arg = f32_to_bf16, bf16_to_f32, Dispatch, arg
        self.d = Dispatcher()

    def up(self, a):
        """An activation array; returns (buffer, the values the device holds)."""
        a = np.asarray(a, np.float32)
        if self.act == 32:
            return self.native.DeviceBuffer.from_numpy(a), a.astype(np.float64)
        return self.native.DeviceBuffer.from_numpy(self.to16(a)), bf16_round(a).astype(np.float64)

    def w16(self, a):
        return self.native.DeviceBuffer.from_numpy(self.to16(a)), bf16_round(a).astype(np.float64)

    def raw(self, a):
        return self.native.DeviceBuffer.from_numpy(np.ascontiguousarray(a))

    def zeros(self, n, e=None):
        return self.native.zeros(n * (self.e if e is None else e))

    def down(self, b, shape):
        if self.act == 32:
            return b.to_numpy(np.float32, shape).astype(np.float64)
        return self.from16(b.to_numpy(np.uint16, shape)).astype(np.float64)

    def run(self, kernel, bufs, **p):
        self.native.sync()
        self.d.dispatch_kernel(self.Dispatch("fusekit_" + kernel + "_f0", [b if isinstance(b, tuple) else self.arg(b) for b in bufs], dict(p, act=self.act)))
        self.native.sync()

    def close(self, got, ref, tol=None):
        err = np.abs(got - ref).max() / max(np.abs(ref).max(), 1e-30)
        limit = tol or (2e-6 if self.act == 32 else 6e-3)
        assert err <= limit, err


def padded(a, ld):
    out = np.zeros(a.shape[:-1] + (ld,), a.dtype)
    out[..., :a.shape[-1]] = a
    return out
