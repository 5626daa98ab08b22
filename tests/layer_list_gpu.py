"""What the GPU tests of the layer-list decoders (Girirax, Bonatar) share: operands on the device, packed sequences, tolerances."""
import ctypes as C

import numpy as np
import pytest

BF16, F32, I32, U8 = 2, 3, 4, 5
TYPES = pytest.mark.parametrize("dtype", [BF16, F32], ids=["bf16", "f32"])
#            rms and largest error relative to the rms of the expected values
TOL = {BF16: (6e-3, 6e-2), F32: (3e-6, 5e-5)}


def near(got, want, dtype, factor=1.0):
    got, want = np.asarray(got, np.float64), np.asarray(want, np.float64)
    assert got.shape == want.shape
    scale = np.sqrt(np.mean(want ** 2)) + 1e-30
    rms, err = np.sqrt(np.mean((got - want) ** 2)) / scale, np.abs(got - want)
    worst = (err / (scale + (0.15 * np.abs(want) if dtype == BF16 else 0))).max()   # large values round coarsely
    assert rms <= TOL[dtype][0] * factor and worst <= TOL[dtype][1] * factor, (rms, worst)


def put(arena, dtype, a):
    """a on the device, and the values it has there."""
    t = arena.alloc(np.shape(a), dtype).write_float(np.asarray(a, np.float32))
    return t, t.read_float().astype(np.float64)


def ints(arena, a):
    return arena.alloc(np.shape(a), I32).write(np.asarray(a, np.int32))


def ok(status):
    assert status == 0, status


class Seqs:
    """gd_backend_packed_seqs of runs [(slot, start, new rows)]."""

    def __init__(self, gda, arena, runs, kv=True):
        n = [r[2] for r in runs]
        cu = np.concatenate([[0], np.cumsum(n)])
        held = np.concatenate([[0], np.cumsum([r[1] + r[2] for r in runs])])
        self.views = [ints(arena, np.repeat(np.arange(len(runs)), n)).view(), ints(arena, cu).view(),
                      ints(arena, [r[0] for r in runs]).view(), ints(arena, [r[1] for r in runs]).view(),
                      ints(arena, held).view()]
        p = [C.pointer(v) for v in self.views]
        self.c = gda.PackedSeqs(p[0], p[1], p[2], p[3], max(n), p[4] if kv else None, int(held[-1]) if kv else 0)
        self.rows, self.cu = int(cu[-1]), cu

    def ref(self):
        return C.byref(self.c)


DTYPES = pytest.mark.parametrize("compute", ["bfloat16", "float32"])
#                   rms of the logits' difference over the rms of the logits
LOGIT_TOL = {"bfloat16": 4e-2, "float32": 2e-5}


def decoder(D, folder, compute, **kw):
    m = D.Model(folder)
    try:
        return m.decoder(compute=compute, **kw)
    finally:
        m.close()


def logits_near(got, want, compute, factor=1.0):
    d = got - want
    d = d - d.mean(-1, keepdims=True)
    err = np.sqrt((d ** 2).mean(-1)) / np.sqrt((want ** 2).mean())
    tol = LOGIT_TOL[compute] * factor
    # 16-bit rounding has a long tail (a position where a branch is small in front of its norm); 32-bit has none
    assert err.max() <= tol * (4 if compute == "bfloat16" else 1), (float(err.max()), int(err.argmax()))
    assert np.sum(err > tol) <= max(1, 0.05 * len(err)), float(np.mean(err > tol))
