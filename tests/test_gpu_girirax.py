"""Girirax decoders on the GPU against the plain model of oracle/layer_list.py: every mechanism alone in BF16 and in
32-bit, then whole decoders through portions, batches, slots, decoding and generation."""
import ctypes as C
import os
import subprocess

import numpy as np
import pytest

import girirax_models as G
from layer_list_gpu import (BF16, DTYPES, F32, I32, TYPES, U8, Seqs, decoder as _decoder, ints as _ints,
                            logits_near as _logits_near, near as _near, ok as _ok, put as _put)

pytestmark = pytest.mark.gpu
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
@pytest.fixture()
def arena(backend):
    buf = backend.buffer(256 << 20)
    yield buf
    backend.free(buf)


@pytest.fixture(scope="module")
def L():
    from oracle import layer_list
    return layer_list


# ---- projections ------------------------------------------------------------------------------------------

@TYPES
@pytest.mark.parametrize("M,N,K", [(1, 48, 64), (3, 100, 40), (5, 33, 21), (17, 256, 96), (64, 904, 256), (128, 512, 128),
                                   (300, 640, 192), (1, 4096, 1024), (130, 130, 72), (9, 2048, 2048)])
def test_projections_of_both_types(backend, gda, arena, dtype, M, N, K):
    rng = np.random.default_rng(M * 7 + N + K)
    x, xv = _put(arena, dtype, rng.standard_normal((M, K)))
    w, wv = _put(arena, dtype, rng.standard_normal((N, K)) / np.sqrt(K))
    b, bv = _put(arena, dtype, rng.standard_normal(N))
    y = arena.alloc((M, N), dtype)
    backend.matmul_nt(x, w, y)
    _near(y.read_float(), xv @ wv.T, dtype)
    backend.fused_linear(x, w, b, None, None, y, True, 1, 0)
    _near(y.read_float(), xv @ wv.T + bv, dtype)
    wide = arena.alloc((M, N), F32)
    backend.matmul_nt(x, w, wide)                       # F32 results
    _near(wide.read_float(), xv @ wv.T, F32, factor=3)
    if N % 2 == 0:
        half = arena.alloc((M, N // 2), dtype)
        u = xv @ wv.T + bv
        value, gate = u[:, :N // 2], u[:, N // 2:]
        for kind, act in ((1, gate / (1 + np.exp(-gate))),
                          (2, 0.5 * gate * (1 + np.tanh(np.sqrt(2 / np.pi) * (gate + 0.044715 * gate ** 3))))):
            backend.fused_linear(x, w, b, None, None, half, True, 1, 0, epilogue=kind)
            _near(half.read_float(), value * act, dtype)


def test_big_tiles_and_unsupported_forms(backend, gda, arena):
    """Enough 256 x 256 tiles for every compute unit, with ragged edges, plain and gated; and what BF16 does not have."""
    rng = np.random.default_rng(5)
    M, N, K = 4100, 4104, 128
    x, xv = _put(arena, BF16, rng.standard_normal((M, K)))
    w, wv = _put(arena, BF16, rng.standard_normal((N, K)) / np.sqrt(K))
    y, half = arena.alloc((M, N), BF16), arena.alloc((M, N // 2), BF16)
    want = xv @ wv.T
    backend.matmul_nt(x, w, y)
    assert backend.linear_last_kernel() == "tile"
    _near(y.read_float(), want, BF16)
    backend.fused_linear(x, w, None, None, None, half, True, 0, 0, epilogue=2)
    gate = want[:, N // 2:]
    _near(half.read_float(), want[:, :N // 2] * 0.5 * gate * (1 + np.tanh(np.sqrt(2 / np.pi) * (gate + 0.044715 * gate ** 3))),
          BF16)
    for kw in (dict(w_is_nk=False, bias_mode=0, prologue=0), dict(w_is_nk=True, bias_mode=0, prologue=2, eps=1e-5)):
        with pytest.raises(gda.GdError) as e:
            nw = arena.alloc((K,), BF16) if kw["prologue"] == 2 else None
            wt = w if kw["w_is_nk"] else arena.alloc((K, N), BF16)
            backend.fused_linear(x, wt, None, None, nw, y, **kw)
        assert e.value.status == gda.UNSUPPORTED
    f = {t: arena.alloc(s, 1) for t, s in (("x", (4, 64)), ("w", (32, 64)), ("y", (4, 16)))}
    with pytest.raises(gda.GdError) as e:
        backend.fused_linear(f["x"], f["w"], None, None, None, f["y"], True, 0, 0, epilogue=2)   # gelu gate in F16
    assert e.value.status == gda.UNSUPPORTED


# ---- residual stream --------------------------------------------------------------------------------------

@TYPES
@pytest.mark.parametrize("N,W", [(1, 64), (5, 36), (9, 2048), (3, 9000), (2, 1)])
def test_residual_stream(backend, gda, arena, dtype, N, W):
    rng = np.random.default_rng(N + W)
    table, tv = _put(arena, dtype, rng.standard_normal((11, W)))
    ids = rng.integers(0, 11, N)
    x, copy = arena.alloc((N, W), F32), arena.alloc((N, W), dtype)
    _ok(backend.call("gd_backend_residual_embed", table.view(), _ints(arena, ids).view(), x.view(), copy.view(), 3.5))
    _near(x.read_float(), tv[ids] * 3.5, F32)
    _near(copy.read_float(), tv[ids] * 3.5, dtype)
    u, uv = _put(arena, dtype, rng.standard_normal((N, W)) * 7)
    w, wv = _put(arena, F32, rng.uniform(0.5, 1.5, W))
    want = tv[ids] * 3.5 + 0.7 * uv / np.sqrt((uv ** 2).mean(1, keepdims=True) + 0.3) * wv
    _ok(backend.call("gd_backend_residual_norm_add", u.view(), w.view(), x.view(), copy.view(), 0.3, 0.7))
    _near(x.read_float(), want, F32)
    _near(copy.read_float(), want, dtype)
    rows = rng.integers(0, N, 3)
    out = arena.alloc((3, W), dtype)
    _ok(backend.call("gd_backend_residual_norm_rows", x.view(), _ints(arena, rows).view(), w.view(), out.view(), 0.3))
    xv = x.read_float().astype(np.float64)
    _near(out.read_float(), (xv / np.sqrt((xv ** 2).mean(1, keepdims=True) + 0.3) * wv)[rows], dtype)


# ---- convolution ------------------------------------------------------------------------------------------

@TYPES
@pytest.mark.parametrize("C_,K", [(20, 4), (300, 3), (7, 1), (64, 2), (16, 7)])
def test_convolution_in_portions_and_used_slots(backend, gda, arena, L, dtype, C_, K):
    """Three sequences in portions of 1, 2 and more tokens, packed unequally; slots that held something before."""
    rng = np.random.default_rng(C_ + K)
    lens, slots = [23, 11, 17], [2, 0, 3]
    u = [rng.standard_normal((n, C_ + 5)) for n in lens]
    taps, bias = rng.standard_normal((C_, K)), rng.standard_normal(C_)
    tt, _ = _put(arena, F32, taps)
    bt, _ = _put(arena, F32, bias)
    ring, _ = _put(arena, dtype, rng.standard_normal((4, K, C_)) * 100)   # what earlier sequences left
    got = [np.zeros((n, C_)) for n in lens]
    values = [None] * 3
    at = [0, 0, 0]
    for cut in ([1, 2, 9], [2, 1, 1], [1, 1, 1], [7, 3, 2], [12, 4, 4]):
        n = [min(c, lens[s] - at[s]) for s, c in enumerate(cut)]
        live = [s for s in range(3) if n[s] > 0]
        sq = Seqs(gda, arena, [(slots[s], at[s], n[s]) for s in live])
        x, xv = _put(arena, dtype, np.concatenate([u[s][at[s]:at[s] + n[s]] for s in live]))
        out = arena.alloc((sq.rows, C_), dtype)
        m = x.matrix(cols=C_)
        m.offset += 3 * x.itemsize                      # pitched: columns 3 .. of wider rows
        _ok(backend.call("gd_backend_causal_conv_silu", m, tt.view(), bt.view(), ring.view(), out.view(), sq.ref()))
        o = out.read_float()
        for k, s in enumerate(live):
            got[s][at[s]:at[s] + n[s]] = o[sq.cu[k]:sq.cu[k + 1]]
            part = xv[sq.cu[k]:sq.cu[k + 1], 3:3 + C_]
            values[s] = part if values[s] is None else np.concatenate([values[s], part])
            at[s] += n[s]
    for s in range(3):
        T = at[s]
        _near(got[s][:T], L.silu(L.causal_conv(values[s], taps.astype(np.float32).astype(np.float64), bias)), dtype)


# ---- recurrence -------------------------------------------------------------------------------------------

def _ssm_reference(L, xbc, dt, m, bias, a_log, d):
    H, P, N, Gn = m
    T, inner = xbc.shape[0], H * P
    return L.ssd_scan(xbc[:, :inner].reshape(T, H, P), xbc[:, inner:inner + Gn * N].reshape(T, Gn, N),
                      xbc[:, inner + Gn * N:].reshape(T, Gn, N), L.softplus(dt + bias), a_log, d)


@TYPES
@pytest.mark.parametrize("H,P,N,Gn", [(4, 16, 16, 2), (3, 20, 40, 3), (2, 64, 128, 1), (2, 72, 256, 1), (5, 7, 9, 1),
                                      (1, 1, 1, 1), (2, 48, 32, 2), (4, 128, 64, 1), (1, 40, 400, 1)])
def test_recurrence_in_portions(backend, gda, arena, L, dtype, H, P, N, Gn):
    """Portions on both sides of the chunked form and of its 64-token chunks, packed with other sequences; the first
    portion starts from a slot full of another sequence's state."""
    rng = np.random.default_rng(H * P + N)
    lens = [150, 75]
    inner = H * P
    raw = [rng.standard_normal((n, inner + 2 * Gn * N)) / np.array([1.0] * inner + [N ** 0.25] * (2 * Gn * N)) for n in lens]
    dts = [rng.standard_normal((n, H)) for n in lens]
    bias, a_log, d = rng.uniform(-4, -1, H), rng.uniform(-1, 2, H), rng.standard_normal(H)
    small = [_put(arena, F32, v) for v in (bias, a_log, d)]
    a_log = small[1][1]
    st, _ = _put(arena, F32, rng.standard_normal((3, H, N, P)) * 50)
    args = gda.SsmArgs(H, P, N, Gn)
    slots, at = [2, 0], [0, 0]
    got, xs, ds = [[], []], [[], []], [[], []]
    for cut in ([1, 66], [65, 2], [2, 1], [17, 6], [64, 0], [1, 0]):
        live = [s for s in range(2) if cut[s] > 0]
        sq = Seqs(gda, arena, [(slots[s], at[s], cut[s]) for s in live])
        x, xv = _put(arena, dtype, np.concatenate([raw[s][at[s]:at[s] + cut[s]] for s in live]))
        dt, dv = _put(arena, dtype, np.concatenate([dts[s][at[s]:at[s] + cut[s]] for s in live]))
        y = arena.alloc((sq.rows, inner), dtype)
        _ok(backend.call("gd_backend_ssm_scan", x.view(), dt.matrix(), small[0][0].view(), small[1][0].view(),
                         small[2][0].view(), st.view(), y.view(), sq.ref(), C.byref(args)))
        o = y.read_float()
        for k, s in enumerate(live):
            sl = slice(sq.cu[k], sq.cu[k + 1])
            got[s].append(o[sl]); xs[s].append(xv[sl]); ds[s].append(dv[sl])
            at[s] += cut[s]
    assert at == lens
    for s in range(2):
        want = _ssm_reference(L, np.concatenate(xs[s]), np.concatenate(ds[s]), (H, P, N, Gn), small[0][1], a_log, small[2][1])
        _near(np.concatenate(got[s]), want.reshape(lens[s], inner), dtype, factor=1 if dtype == BF16 else 4)
    assert np.all(np.isfinite(st.read_float()))


@pytest.mark.parametrize("decay", ["slow", "fast"])
def test_recurrence_carries_one_early_token_through_chunks(backend, gda, arena, L, decay):
    """One token with a large step at the start of a prompt and small ones behind it: its trace is what the output is
    made of hundreds of tokens later (slow decay), or must be gone (fast decay).  The chunked form and token by token."""
    H, P, N, T = 2, 32, 64, 300
    rng = np.random.default_rng(9)
    x = rng.standard_normal((T, H * P + 2 * N)) * 0.05
    x[2] = rng.standard_normal(H * P + 2 * N) * 2
    x[:, H * P + N:] = x[2, H * P:H * P + N] / 4                    # every C asks for that token's B
    dt = np.full((T, H), -6.0)
    dt[2] = 3.0
    small = [_put(arena, F32, v)[0] for v in (np.zeros(H), np.full(H, -4.0 if decay == "slow" else 3.0), np.zeros(H))]
    xt, xv = _put(arena, BF16, x)
    dtt, dv = _put(arena, BF16, dt)
    st = arena.alloc((1, H, N, P), F32).write(np.zeros((1, H, N, P)))
    y = arena.alloc((T, H * P), BF16)
    args = gda.SsmArgs(H, P, N, 1)
    want = _ssm_reference(L, xv, dv, (H, P, N, 1), np.zeros(H), small[1].read(), np.zeros(H)).reshape(T, H * P)
    sq = Seqs(gda, arena, [(0, 0, T)])
    _ok(backend.call("gd_backend_ssm_scan", xt.view(), dtt.matrix(), small[0].view(), small[1].view(), small[2].view(),
                     st.view(), y.view(), sq.ref(), C.byref(args)))
    _near(y.read_float()[200:], want[200:], BF16, factor=2)
    left = st.read()
    outs = []
    for t in range(T):
        sq = Seqs(gda, arena, [(0, t, 1)])
        _ok(backend.call("gd_backend_ssm_scan", xt.rows(t, 1).view(), dtt.rows(t, 1).matrix(), small[0].view(),
                         small[1].view(), small[2].view(), st.view(), y.rows(t, 1).view(), sq.ref(), C.byref(args)))
    _near(y.read_float()[200:], want[200:], BF16, factor=2)
    _near(left, st.read(), F32, factor=30)                          # 16-bit parts against plain F32


@TYPES
@pytest.mark.parametrize("H,P,N,Gn,K", [(4, 16, 16, 2, 4), (3, 20, 40, 3, 3), (2, 64, 128, 1, 4), (5, 7, 9, 5, 1), (2, 40, 300, 1, 7)])
def test_fused_convolution_and_recurrence_step(backend, gda, arena, dtype, H, P, N, Gn, K):
    """One launch of a decode step against the two operators: same results, rings and states, from the first token on."""
    rng = np.random.default_rng(N)
    ch, B = H * P + 2 * Gn * N, 3
    small = [_put(arena, F32, v)[0] for v in (rng.uniform(-3, -1, H), rng.uniform(-1, 1, H), rng.standard_normal(H))]
    taps, bias = _put(arena, F32, rng.standard_normal((ch, K)) * 0.5)[0], _put(arena, F32, rng.standard_normal(ch) * 0.1)[0]
    args = gda.SsmArgs(H, P, N, Gn)
    junk = rng.standard_normal((4, K, ch)) * 9, rng.standard_normal((4, H, N, P)) * 9
    sides = [(_put(arena, dtype, junk[0])[0], _put(arena, F32, junk[1])[0], arena.alloc((B, H * P), dtype)) for _ in range(2)]
    conv = arena.alloc((B, ch), dtype)
    for t in range(6):
        start = [t, t + 1 if t else 0, 0]
        sq = Seqs(gda, arena, [(2, start[0], 1), (0, t, 1), (3, start[2], 1)])
        x = _put(arena, dtype, rng.standard_normal((B, ch + H)))[0]
        xm, dt = x.matrix(cols=ch), x.matrix(cols=H)
        dt.offset += ch * x.itemsize
        rest = [v.view() for v in small]
        ring, st, y = sides[0]
        _ok(backend.call("gd_backend_causal_conv_silu", xm, taps.view(), bias.view(), ring.view(), conv.view(), sq.ref()))
        _ok(backend.call("gd_backend_ssm_scan", conv.view(), dt, *rest, st.view(), y.view(), sq.ref(), C.byref(args)))
        ring, st, y = sides[1]
        _ok(backend.call("gd_backend_conv_ssm_step", xm, taps.view(), bias.view(), ring.view(), dt, *rest, st.view(), y.view(),
                         sq.ref(), C.byref(args)))
        for a, b in zip(*sides):
            _near(a.read_float(), b.read_float(), dtype)


@TYPES
@pytest.mark.parametrize("inner,parts", [(64, 1), (96, 4), (4096, 2), (30, 3), (5000, 1)])
def test_gate_then_group_norm(backend, gda, arena, L, dtype, inner, parts):
    rng = np.random.default_rng(inner)
    y, yv = _put(arena, dtype, rng.standard_normal((6, inner)) * np.linspace(0.2, 5, inner))
    z, zv = _put(arena, dtype, rng.standard_normal((6, inner + 3)))
    w, wv = _put(arena, F32, rng.uniform(0.5, 1.5, inner))
    out = arena.alloc((6, inner), dtype)
    m = z.matrix(cols=inner)
    _ok(backend.call("gd_backend_gated_group_norm", y.view(), m, w.view(), out.view(), parts, 0.02))
    _near(out.read_float(), L.gated_group_norm(yv, zv[:, :inner], wv, parts, 0.02), dtype)


# ---- latent attention -------------------------------------------------------------------------------------

class Latent:
    """One latent attention layer at operator level: random projections, a cache with used slots, and the plain result."""

    def __init__(self, gda, backend, arena, L, dtype, H, D, R, V, KV, QR=24, slots=3, tmax=320, seed=0, base=500.0):
        self.gda, self.be, self.arena, self.L, self.dtype = gda, backend, arena, L, dtype
        self.H, self.D, self.R, self.V, self.KV, self.QR, self.tmax, self.base = H, D, R, V, KV, QR, tmax, base
        self.rng = rng = np.random.default_rng(seed + H * D + KV)
        self.args = gda.LatentArgs(H, D, R, V, QR, KV, 0.9 * (D + R) ** -0.5, 0.01)
        self.qn, self.qnv = _put(arena, F32, rng.uniform(0.5, 1.5, QR))
        self.kn, self.knv = _put(arena, F32, rng.uniform(0.5, 1.5, KV))
        self.freq = arena.alloc((R // 2,), F32).write(base ** (-2.0 * np.arange(R // 2) / R))
        ukv = rng.standard_normal((H * (D + V), KV)) / np.sqrt(KV)
        self.ukv, self.ukvv = _put(arena, dtype, ukv)
        ukt = self.ukvv[:H * D].reshape(H, D, KV).transpose(0, 2, 1).reshape(H * KV, D)
        self.ukt, _ = _put(arena, dtype, ukt)
        pitch = gda.lib().gd_backend_latent_pitch(KV, R)
        self.cache, _ = _put(arena, dtype, rng.standard_normal((slots, tmax, pitch)) * 30)  # an earlier sequence's rows
        self.c = [np.zeros((0, KV))] * slots    # plain latents and rotated key parts of every slot
        self.kr = [np.zeros((0, R))] * slots

    def run(self, runs, q=None, kv=True, proj=None):
        """runs [(slot, start, n)]: prepare, then attend over queries q [rows, H, D + R]; returns (got, expected)."""
        H, D, R, V, KV, QR = self.H, self.D, self.R, self.V, self.KV, self.QR
        sq = Seqs(self.gda, self.arena, runs, kv)
        N = sq.rows
        if proj is None:
            proj = self.rng.standard_normal((N, QR + KV + R + H * V))
        p, pv = _put(self.arena, self.dtype, proj)
        if q is None:
            q = self.rng.standard_normal((N, H, D + R))
        qt, qv = _put(self.arena, self.dtype, q.reshape(N, -1))
        ang, cq = self.arena.alloc((N, R), F32), self.arena.alloc((N, QR), self.dtype)
        out = self.arena.alloc((N, H * V), self.dtype).write_float(np.zeros((N, H * V)))
        pm, gm = p.matrix(cols=QR + KV + R), p.matrix(cols=H * V)
        gm.offset += (QR + KV + R) * p.itemsize
        _ok(self.be.call("gd_backend_latent_prepare", pm, self.qn.view(), self.kn.view(), self.freq.view(), ang.view(),
                         cq.view(), self.cache.view(), sq.ref(), C.byref(self.args)))
        need = self.gda.lib().gd_backend_latent_work_bytes(self.be.handle, C.byref(self.args), N, sq.c.max_new,
                                                           sq.c.kv_total, self.tmax, self.dtype)
        work = self.arena.alloc((need,), U8)
        _ok(self.be.call("gd_backend_latent_attend", qt.view(), self.ukt.view(), self.ukv.view(), gm, ang.view(),
                         self.cache.view(), work.view(), out.view(), sq.ref(), C.byref(self.args)))
        _near(cq.read_float(), self.L.rms_norm(pv[:, :QR], self.qnv, 0.01), self.dtype)
        want = np.zeros((N, H, V))
        gate = self.L.sigmoid(pv[:, QR + KV + R:])
        stored = self.cache.read_float().astype(np.float64)
        uk, uv = self.ukvv[:H * D].reshape(H, D, KV), self.ukvv[H * D:].reshape(H, V, KV)
        for k, (slot, start, n) in enumerate(runs):
            rows = slice(sq.cu[k], sq.cu[k + 1])
            pos = np.arange(start, start + n)
            c = self.L.rms_norm(pv[rows, QR:QR + KV], self.knv, 0.01)
            kr = self.L.rotate_half(pv[rows, None, QR + KV:QR + KV + R], pos, self.base, R)[:, 0]
            _near(stored[slot, start:start + n, :KV], c, self.dtype)
            _near(stored[slot, start:start + n, KV:KV + R], kr, self.dtype, factor=1 if self.dtype == BF16 else 10)
            # the attention is compared over what the cache holds
            held = stored[slot, :start + n]
            qh = qv[rows].reshape(n, H, D + R)
            qr = self.L.rotate_half(qh[..., D:], pos, self.base, R)
            kh = np.einsum("jc,hdc->jhd", held[:, :KV], uk)
            vh = np.einsum("jc,hvc->jhv", held[:, :KV], uv)
            s = (np.einsum("ihd,jhd->hij", qh[..., :D], kh) + np.einsum("ihr,jr->hij", qr, held[:, KV:KV + R])) * self.args.scale
            s = np.where(np.arange(start + n)[None, None, :] <= pos[None, :, None], s, -np.inf)
            s = np.exp(s - s.max(-1, keepdims=True))
            want[rows] = np.einsum("hij,jhv->ihv", s / s.sum(-1, keepdims=True), vh)
        return out.read_float(), want.reshape(N, H * V) * gate


LATENT_SIZES = [(4, 24, 8, 16, 48), (3, 72, 24, 56, 112), (16, 128, 64, 128, 512), (17, 32, 16, 40, 64), (2, 20, 6, 10, 21),
                (1, 8, 2, 8, 16), (20, 128, 32, 96, 256), (5, 192, 64, 128, 192), (1, 1, 2, 1, 1),
                (40, 16, 8, 8, 32), (18, 16, 16, 16, 640)]


@TYPES
@pytest.mark.parametrize("sizes", LATENT_SIZES, ids=lambda s: "x".join(map(str, s)))
def test_latent_attention_of_prompts_portions_and_steps(backend, gda, arena, L, dtype, sizes):
    """Portions on both sides of the expanded form, of its 128-row and 64-key blocks and of the decode form's pieces, in
    batches of unequal sequences, into slots that are already full of something else."""
    la = Latent(gda, backend, arena, L, dtype, *sizes)
    for runs in ([(1, 0, 70), (0, 0, 1)], [(1, 70, 1), (0, 1, 1), (2, 0, 1)], [(0, 2, 2), (1, 71, 33)],
                 [(1, 104, 31), (2, 1, 160), (0, 4, 64)], [(1, 135, 1), (0, 68, 1), (2, 161, 1)], [(1, 136, 1)],
                 [(0, 0, 40)], [(0, 40, 1), (2, 162, 1)]):
        got, want = la.run(runs)
        _near(got, want, dtype, factor=1.5 if dtype == BF16 else 10)
    got, want = la.run([(2, 163, 40)], kv=False)      # without the expanded form's tables
    _near(got, want, dtype, factor=1.5 if dtype == BF16 else 10)


@pytest.mark.parametrize("sizes", [(4, 72, 24, 56, 112), (16, 128, 64, 128, 512)], ids=lambda s: "x".join(map(str, s)))
@pytest.mark.parametrize("form", ["expanded", "absorbed"])
def test_every_key_is_seen_by_the_rows_behind_it_and_by_no_other(backend, gda, arena, L, sizes, form):
    """A single key whose score stands out by far, at the edges of blocks and pieces and at both ends: rows behind it
    must return its value, rows in front of it must not."""
    la = Latent(gda, backend, arena, L, BF16, *sizes, seed=3)
    H, D, R, V, KV, QR = la.H, la.D, la.R, la.V, la.KV, la.QR
    T = 300
    proj = la.rng.standard_normal((T, QR + KV + R + H * V)) * 0.5
    proj[:, QR + KV:QR + KV + R] = 0                      # no rotated part: the latents decide
    uk = la.ukvv[:H * D].reshape(H, D, KV)
    for key in (0, 1, 62, 63, 64, 127, 128, 191, 255, 256, 299):
        c = la.L.rms_norm(proj[key, QR:QR + KV], la.knv, 0.01)
        k = np.einsum("hdc,c->hd", uk, c)
        q = np.zeros((T, H, D + R))
        q[:, :, :D] = 14.0 * k / (k ** 2).sum(-1, keepdims=True) / la.args.scale    # score of `key`: 14
        if form == "expanded":
            got, want = la.run([(1, 0, T)], q=q, proj=proj)
        else:
            rows = sorted({max(key - 1, 0), key, min(key + 1, T - 1), T - 1})
            la.run([(1, 0, T)], proj=proj)
            got, want = [], []
            for r in rows:
                g, w = la.run([(1, r, 1)], q=q[r:r + 1], proj=proj[r:r + 1])
                got.append(g), want.append(w)
            got, want = np.concatenate(got), np.concatenate(want)
        _near(got, want, BF16, factor=2)


# ---- decoders ---------------------------------------------------------------------------------------------

MODELS = {
    "mixed": G.config([G.mamba(), G.latent(), (G.mamba(heads=2, vdim=24, state=24, groups=1, norm_groups=3, conv=2), 40),
                       (G.latent(heads=3, dim=16, rot_dim=16, vdim=32, q_rank=24, kv_rank=32, scale=0.31, base=777.0), None)]),
    "recurrent": G.config([(G.mamba(heads=6, vdim=8, state=8, groups=3, norm_groups=1, conv=3), None), G.mamba(groups=4, norm_groups=4)],
                          vocab=70, width=40, eps=1e-3, residual_mult=1.0, embedding_scale=1.0),
    "attention": G.config([G.latent(heads=1, dim=8, rot_dim=8, vdim=8, q_rank=16, kv_rank=16), (G.latent(rot_dim=2, dim=30), 64)],
                          vocab=101, width=48, ff=200, residual_mult=0.3, embedding_scale=7.0),
    "odd": G.config([G.latent(heads=3, dim=10, rot_dim=6, vdim=7, q_rank=9, kv_rank=13),
                     G.mamba(heads=3, vdim=5, state=6, groups=1, norm_groups=5, conv=1)], vocab=37, width=30, ff=22),
    "wide": G.config([G.mamba(heads=4, vdim=64, state=128, groups=1, norm_groups=1),
                      G.latent(heads=8, dim=64, rot_dim=32, vdim=64, q_rank=96, kv_rank=256)], width=256, ff=512),
}
@pytest.fixture(scope="module")
def D(gda):
    from gradients_c_amd import decoder
    return decoder


@pytest.fixture(scope="module")
def models(tmp_path_factory, L):
    """name -> (folder, tokens [3][T], plain logits [3][T, vocab])"""
    made = {}

    def get(name, T=90):
        if (name, T) not in made:
            cfg = MODELS[name]
            t = G.weights(cfg, 11)
            rng = np.random.default_rng(12)
            tokens = [rng.integers(0, cfg["vocab"], n) for n in (T, T // 2 + 1, T // 3)]
            folder = G.save(str(tmp_path_factory.mktemp(name)), cfg, t)
            made[name, T] = (folder, tokens, [L.forward(cfg, t, k) for k in tokens], cfg, t)
        return made[name, T]
    return get


@DTYPES
@pytest.mark.parametrize("name", list(MODELS))
def test_prompt_portions_and_decoding_agree_with_the_plain_model(D, models, name, compute):
    folder, tokens, want, cfg, _ = models(name)
    d = _decoder(D, folder, compute, max_seq=100, batch=3)
    try:
        t, w = tokens[0], want[0]
        slot = d.acquire()
        _logits_near(d.extend({slot: t}), w, compute)                       # the whole prompt
        d.release(slot)
        for cut in (2, 3, 17, 33, 64):                                        # portions, in a slot that was used
            slot = d.acquire()
            got = [d.extend({slot: t[a:a + cut]}) for a in range(0, len(t), cut)]
            _logits_near(np.concatenate(got), w, compute)
            d.release(slot)
        slot = d.acquire()
        got = [d.extend({slot: t[:40]}, want=[])] + [d.extend({slot: [k]}) for k in t[40:]]
        _logits_near(np.concatenate(got[1:]), w[40:], compute)               # a prompt, then token by token
        d.release(slot)
        slot = d.acquire()
        got = np.concatenate([d.extend({slot: [k]}) for k in t[:30]])        # token by token from the first
        _logits_near(got, w[:30], compute)
    finally:
        d.close()


@DTYPES
@pytest.mark.parametrize("name", ["mixed", "wide"])
def test_batches_of_unequal_requests(D, models, name, compute):
    """Requests that start, continue and end at different times share steps; each must give what it gives alone."""
    folder, tokens, want, cfg, _ = models(name)
    d = _decoder(D, folder, compute, max_seq=100, batch=4)
    try:
        a, b, c = d.acquire(), d.acquire(), d.acquire()
        at, got = {a: 0, b: 0, c: 0}, {a: [], b: [], c: []}
        req = {a: 0, b: 1, c: 2}
        plan = [{a: 40}, {a: 1, b: 20}, {b: 1, c: 2, a: 1}, {c: 27, a: 33, b: 1}, {a: 1, b: 1, c: 1}, {b: 5, a: 2}]
        for step in plan:
            runs = {s: tokens[req[s]][at[s]:at[s] + n] for s, n in step.items()}
            out = d.extend(runs)
            k = 0
            for s, r in runs.items():
                got[s].append(out[k:k + len(r)])
                k += len(r)
                at[s] += len(r)
        for s in (a, b, c):
            g = np.concatenate(got[s])
            _logits_near(g, want[req[s]][:len(g)], compute)
        d.release(b)                                                          # a slot is freed and used again
        b = d.acquire()
        out = d.extend({a: tokens[0][at[a]:at[a] + 1], b: tokens[2][:25]})
        _logits_near(out[1:], want[2][:25], compute)
        _logits_near(out[:1], want[0][at[a]:at[a] + 1], compute)
        # only wanted places, in any order
        out = d.extend({b: tokens[2][25:29]}, want=[3, 0])
        _logits_near(out, want[2][[28, 25]], compute)
    finally:
        d.close()


@DTYPES
def test_prefill_step_and_resident_session(D, models, compute):
    """The calls every model of the library has: packed prefill of all rows, steps with host tokens, and the resident
    session whose greedy tokens feed themselves through a replayed graph."""
    folder, tokens, want, cfg, _ = models("mixed")
    prompts = [t[:12 + 5 * i] for i, t in enumerate(tokens)]
    cu = np.concatenate([[0], np.cumsum([len(p) for p in prompts])])
    d = _decoder(D, folder, compute, max_seq=64, batch=3)
    try:
        logits, nxt, gap = d.prefill(np.concatenate(prompts), cu)
        for i, p in enumerate(prompts):
            _logits_near(logits[i:i + 1].astype(np.float64), want[i][len(p) - 1:len(p)], compute, factor=1 if compute == "bfloat16" else 50)
        for k in range(3):
            step = [tokens[i][len(p) + k] for i, p in enumerate(prompts)]
            logits, nxt, gap = d.step(step)
            for i, p in enumerate(prompts):
                _logits_near(logits[i:i + 1].astype(np.float64), want[i][len(p) + k:len(p) + k + 1], compute,
                             factor=1 if compute == "bfloat16" else 50)
        d.prefill(np.concatenate(prompts), cu)
        first = nxt
        by_step = []
        cur = first
        for _ in range(12):
            _, cur, _ = d.step(cur)
            by_step.append(cur.copy())
        d.prefill(np.concatenate(prompts), cu)
        ids, gaps, _ = d.run_resident(first, 12)
        for k in range(12):
            same = ids[k] == by_step[k]
            if not same.all():
                assert gaps[k][~same].max() < 1e-2
                break
    finally:
        d.close()


def _greedy(L, cfg, weights, prompt, n):
    seq, gaps = list(prompt), []
    for _ in range(n):
        row = L.forward(cfg, weights, seq)[-1]
        top = np.sort(row)[-2:]
        gaps.append(top[1] - top[0])
        seq.append(int(row.argmax()))
    return seq[len(prompt):], gaps


def test_greedy_generation_through_the_entry_point(D, L, models):
    folder, tokens, _, cfg, w = models("mixed")
    prompts = [tokens[0][:9], tokens[1][:5], tokens[2][:14]]
    cu = np.concatenate([[0], np.cumsum([len(p) for p in prompts])])
    d = _decoder(D, folder, "float32", max_seq=60, batch=3)
    try:
        out = d.generate(np.concatenate(prompts), cu, 20)
        sampled = d.generate(np.concatenate(prompts), cu, 20, temperature=0.8, rng_state=5)
        again = d.generate(np.concatenate(prompts), cu, 20, temperature=0.8, rng_state=5)
    finally:
        d.close()
    for p, got in zip(prompts, out):
        want, gaps = _greedy(L, cfg, w, p, 20)
        assert len(got) == 20
        for k in range(20):
            if got[k] != want[k]:
                assert gaps[k] < 1e-3, (k, gaps[k])
                break
    assert all((a == b).all() for a, b in zip(sampled, again))
    assert any(len(a) != len(b) or (a != b).any() for a, b in zip(sampled, out))


@DTYPES
def test_the_inference_program_opens_a_model_folder(D, models, compute):
    folder, tokens, _, _, _ = models("mixed")
    prompt = tokens[0][:11]
    exe = os.path.join(ROOT, "gradients.c_amd", "gpt_lm_infer")

    def run(*args):
        r = subprocess.run([exe, "--checkpoint", folder, "--dtype", compute, *args], capture_output=True, timeout=60)
        return r.returncode, r.stdout.decode(), r.stderr.decode()
    ids = ",".join(str(int(t)) for t in prompt)
    d = _decoder(D, folder, compute, max_seq=40, batch=1)
    try:
        greedy = d.generate(prompt, [0, len(prompt)], 12)[0].tolist()
        sampled = d.generate(prompt, [0, len(prompt)], 12, 0.9, 0.02, 1.2, 0.0, -1,
                             D.lib().gd_gpt_generation_rng(5, 1, 0))[0].tolist()
    finally:
        d.close()
    line = lambda out: [int(v) for v in next(l for l in out.splitlines() if l.startswith("ids:"))[4:].split()]
    rc, out, err = run("--token-ids", ids, "--max-new-tokens", "12")
    assert rc == 0, (rc, err)
    assert line(out) == greedy and "architecture=Girirax" in out and "prompt_tokens=11" in out
    rc, out, err = run("--token-ids", ids, "--max-new-tokens", "12", "--temperature", "0.9", "--min-p", "0.02",
                       "--repetition-penalty", "1.2", "--seed", "5")
    assert rc == 0 and line(out) == sampled
    stop = greedy[5]
    rc, out, err = run("--token-ids", ids, "--max-new-tokens", "12", "--stop-token", str(stop))
    assert rc == 0 and line(out) == greedy[:greedy.index(stop)]
    rc, out, err = run("--token-ids", "1,2,1000000")
    assert rc == 1 and "vocabulary" in err
    rc, out, err = run("--token-ids", "1,two")
    assert rc == 1 and "list" in err
    assert run("--token-ids", "1", "--prompt", "x")[0] == 2


@DTYPES
def test_long_decoding(D, L, tmp_path, compute):
    """Hundreds of single tokens behind a short prompt: the state is carried, the cache grows over several pieces."""
    cfg = G.config([G.mamba(), G.latent()], vocab=64, width=48, ff=64)
    w = G.weights(cfg, 21)
    t = np.random.default_rng(22).integers(0, 64, 420)
    want = L.forward(cfg, w, t)
    d = _decoder(D, G.save(str(tmp_path), cfg, w), compute, max_seq=420)
    try:
        slot = d.acquire()
        d.extend({slot: t[:5]}, want=[])
        got = np.concatenate([d.extend({slot: [k]}) for k in t[5:]])
        _logits_near(got, want[5:], compute)
    finally:
        d.close()


def test_long_prompt_in_one_step_and_in_portions(D, L, tmp_path):
    cfg = G.config([G.mamba(heads=2, vdim=32, state=32, groups=1), G.latent(heads=2, dim=32, rot_dim=32, vdim=32, kv_rank=64)], vocab=64, width=64)
    w = G.weights(cfg, 31)
    t = np.random.default_rng(32).integers(0, 64, 700)
    want = L.forward(cfg, w, t)
    d = _decoder(D, G.save(str(tmp_path), cfg, w), "bfloat16", max_seq=704, batch=2)
    try:
        _logits_near(d.extend({d.acquire(): t}), want, "bfloat16")
        slot = d.acquire()
        got = [d.extend({slot: t[a:b]}) for a, b in ((0, 255), (255, 257), (257, 258), (258, 640), (640, 700))]
        _logits_near(np.concatenate(got), want, "bfloat16")
    finally:
        d.close()


def test_trace_run_replays_steps(models, tmp_path):
    import json
    folder, tokens, want, cfg, _ = models("mixed")
    t = [int(k) for k in tokens[0][:50]]
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": t[:30], "want": [4, 29]}], "end": []},
             {"step": 1, "entries": [{"id": "a", "tokens": t[30:31], "want": []}], "end": []},
             {"step": 2, "entries": [{"id": "a", "tokens": t[31:50], "want": [18]}], "end": ["a"]},
             {"step": 3, "entries": [{"id": "b", "tokens": t[:3], "want": [2]}], "end": ["b"]}]
    r = subprocess.run([os.path.join(ROOT, "bin", "trace_run"), "--model", folder, "--dtype", "float32", "--out",
                        str(tmp_path), "--max-tokens", "50"], input="".join(json.dumps(s) + "\n" for s in steps),
                       capture_output=True, text=True, timeout=100)
    assert r.returncode == 0, r.stderr
    assert r.stdout.split("\n")[:4] == ["done 0", "done 1", "done 2", "done 3"]
    for step, places in ((0, [4, 29]), (2, [49]), (3, [2])):
        got = np.fromfile(os.path.join(str(tmp_path), "%d.f32" % step), np.float32).reshape(-1, cfg["vocab"])
        _logits_near(got, want[0][places], "float32")
    assert not os.path.exists(os.path.join(str(tmp_path), "1.f32"))
