"""Bonatar decoders on the GPU against the plain model of oracle/layer_list.py: every mechanism alone in BF16 and in
32-bit, then whole decoders through portions, batches, slots, decoding and generation."""
import ctypes as C
import os
import subprocess

import numpy as np
import pytest

import bonatar_models as B
from layer_list_gpu import BF16, DTYPES, F32, I32, TYPES, U8, Seqs, decoder, ints, logits_near, near, ok, put

pytestmark = pytest.mark.gpu
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))


@pytest.fixture()
def arena(backend):
    buf = backend.buffer(384 << 20)
    yield buf
    backend.free(buf)


@pytest.fixture(scope="module")
def L():
    from oracle import layer_list
    return layer_list


# ---- projections ------------------------------------------------------------------------------------------

def _clamped(value, gate, limit, alpha=1.702):
    g = np.minimum(gate, limit)
    return g / (1 + np.exp(-alpha * g)) * (np.clip(value, -limit, limit) + 1)


@TYPES
@pytest.mark.parametrize("M,N,K", [(1, 48, 64), (3, 100, 40), (5, 34, 21), (17, 256, 96), (9, 2048, 2048), (20, 4096, 1024),
                                   (128, 512, 128), (300, 640, 192), (130, 130, 72), (257, 528, 256), (700, 8192, 128)])
def test_square_relu_and_clamped_gate_epilogues(backend, arena, dtype, M, N, K):
    """Every kernel family: few rows, large weights, tiles with whole and ragged edges."""
    rng = np.random.default_rng(M * 7 + N + K)
    x, xv = put(arena, dtype, rng.standard_normal((M, K)))
    w, wv = put(arena, dtype, rng.standard_normal((N, K)) / np.sqrt(K))
    b, bv = put(arena, dtype, rng.standard_normal(N))
    y, half = arena.alloc((M, N), dtype), arena.alloc((M, N // 2), dtype)
    u = xv @ wv.T
    backend.fused_linear(x, w, None, None, None, y, True, 0, 0, epilogue=3)
    near(y.read_float(), np.maximum(u, 0) ** 2, dtype, factor=2)
    backend.fused_linear(x, w, b, None, None, y, True, 1, 0, epilogue=3)
    near(y.read_float(), np.maximum(u + bv, 0) ** 2, dtype, factor=2)
    for limit, alpha in ((0.8, 1.702), (3.0, 0.5)):
        backend.fused_linear(x, w, None, None, None, half, True, 0, 0, epilogue=4, gate_limit=limit, gate_alpha=alpha)
        near(half.read_float(), _clamped(u[:, :N // 2], u[:, N // 2:], limit, alpha), dtype, factor=1.5)


@pytest.mark.parametrize("M,N,K", [(200, 264, 64), (1000, 528, 128), (4200, 2064, 192), (129, 288, 40), (300, 257, 64)])
def test_a_few_columns_behind_whole_tiles(backend, arena, M, N, K):
    """Stacked projections whose last part is narrow: its columns come from another kernel, into the same pitched rows."""
    rng = np.random.default_rng(N)
    x, xv = put(arena, BF16, rng.standard_normal((M, K)))
    w, wv = put(arena, BF16, rng.standard_normal((N, K)) / np.sqrt(K))
    pitch = (N + 7) // 8 * 8 + 8
    y = arena.alloc((M, pitch), BF16).write_float(np.full((M, pitch), 7.0))
    m = y.matrix(cols=N)
    ok(backend.call("gd_backend_matmul_nt", x.matrix(), w.matrix(), m))
    got = y.read_float()
    near(got[:, :N], xv @ wv.T, BF16)
    assert (got[:, N:] == 7.0).all()


def test_forms_that_half_precision_does_not_have(backend, gda, arena):
    x, w, y = arena.alloc((4, 64), 1), arena.alloc((32, 64), 1), arena.alloc((4, 32), 1)
    for epilogue, out in ((3, y), (4, arena.alloc((4, 16), 1))):
        with pytest.raises(gda.GdError) as e:
            backend.fused_linear(x, w, None, None, None, out, True, 0, 0, epilogue=epilogue, gate_limit=1.0, gate_alpha=1.0)
        assert e.value.status == gda.UNSUPPORTED


# ---- residual stream --------------------------------------------------------------------------------------

@TYPES
@pytest.mark.parametrize("N,W,top", [(1, 64, 1), (5, 36, 3), (9, 2048, 2), (3, 9000, 2), (2, 1, 1), (70, 200, 4),
                                     (1030, 512, 2), (1500, 2048, 1)])
def test_add_and_norm(backend, gda, arena, dtype, N, W, top):
    """A branch, routed rows, both or neither; the norm for the next sublayer, packed for its experts or not."""
    rng = np.random.default_rng(N + W)
    x, xv = put(arena, F32, rng.standard_normal((N, W)) * 3)
    u, uv = put(arena, dtype, rng.standard_normal((N, W)))
    w, wv = put(arena, F32, rng.uniform(0.5, 1.5, W))
    P = N * top + 3
    perm = rng.permutation(P)[:N * top].astype(np.int32)
    if N * top > 4:
        perm[3] = -1                                                     # a choice that leads nowhere
    r, rv = put(arena, dtype, rng.standard_normal((P, W)))
    place = ints(arena, perm)
    pv, rview = C.pointer(place.view()), C.pointer(r.view())
    routed = gda.RoutedRows(rview, pv, top, 0.3)
    out = arena.alloc((N, W), dtype)
    packed = arena.alloc((P, W), dtype)
    to_view = C.pointer(packed.view())
    to = gda.RoutedRows(to_view, pv, top, 1.0)
    sums = np.where(perm.reshape(N, top)[..., None] >= 0, rv[perm.reshape(N, top)], 0).sum(1) * 0.3
    for branch, added, normed, scattered in ((1, 0, 1, 0), (0, 0, 1, 1), (1, 1, 1, 1), (0, 1, 1, 0), (1, 1, 0, 0), (1, 0, 0, 0)):
        packed.write_float(np.full((P, W), 5.0))
        out.write_float(np.full((N, W), 5.0))
        ok(backend.call("gd_backend_residual_add_norm", u.view() if branch else None, C.byref(routed) if added else None,
                        x.view(), w.view() if normed else None, out.view() if normed else None,
                        C.byref(to) if scattered else None, 0.2))
        xv = xv + (uv if branch else 0) + (sums if added else 0)
        near(x.read_float(), xv, F32, factor=2)
        h = xv / np.sqrt((xv ** 2).mean(1, keepdims=True) + 0.2) * wv
        if normed:
            near(out.read_float(), h, dtype)
        want = np.full((P, W), 5.0)
        if scattered:
            live = perm >= 0
            want[perm[live]] = np.repeat(h, top, axis=0)[live]
        near(packed.read_float(), want, dtype)
    assert backend.call("gd_backend_residual_add_norm", u.view(), None, x.view(), w.view(), None, None, 0.2) == -1
    assert backend.call("gd_backend_residual_add_norm", None, None, x.view(), None, None, None, 0.2) == -1


# ---- attention --------------------------------------------------------------------------------------------

class Grouped:
    """One attention layer at operator level: caches with used slots, and what every slot has been given."""

    def __init__(self, gda, backend, arena, L, dtype, H, G, D, V, R, chunk, slots=3, tmax=400, seed=0, scale=None, mult=1.3,
                 base=300.0):
        self.gda, self.be, self.arena, self.L, self.dtype = gda, backend, arena, L, dtype
        self.H, self.G, self.D, self.V, self.R, self.chunk = H, G, D, V, R, chunk
        self.rng = rng = np.random.default_rng(seed + H * D + V + chunk)
        self.args = gda.GroupedArgs(H, G, D, V, R, chunk, scale or 0.9 * D ** -0.5, mult)
        self.freq = base ** (-2.0 * np.arange(R // 2) / max(R, 1))
        self.freq_dev = arena.alloc((max(R // 2, 1),), F32)
        self.freq_dev.write(self.freq if R else np.zeros(1))
        self.places = min(chunk, tmax) if chunk else tmax
        self.kc = put(arena, dtype, rng.standard_normal((slots, G, self.places, D)) * 30)[0]   # an earlier sequence's rows
        self.vc = put(arena, dtype, rng.standard_normal((slots, G, self.places, V)) * 30)[0]
        self.k, self.v = [np.zeros((0, G, D))] * slots, [np.zeros((0, G, V))] * slots          # rotated keys, values

    def proj(self, n):
        cols = (self.H + self.G) * self.D + self.G * self.V + self.H
        return self.rng.standard_normal((n, (cols + 7) // 8 * 8)) * 0.9, cols

    def run(self, runs, rows=None):
        """runs [(slot, start, n)]; rows: the projection's values; returns (got, expected)."""
        H, G, D, V, R = self.H, self.G, self.D, self.V, self.R
        sq = Seqs(self.gda, self.arena, runs, kv=False)
        N = sq.rows
        values, cols = self.proj(N)
        if rows is not None:
            values = rows
        p, pv = put(self.arena, self.dtype, values)
        out = self.arena.alloc((N, H * V), self.dtype).write_float(np.full((N, H * V), 9.0))
        need = self.gda.lib().gd_backend_grouped_work_bytes(self.be.handle, C.byref(self.args), N, sq.c.max_new, self.places, self.dtype)
        work = self.arena.alloc((need,), U8)
        ok(self.be.call("gd_backend_grouped_attend", p.matrix(cols=cols), self.freq_dev.view(), self.kc.view(), self.vc.view(),
                        work.view(), out.view(), sq.ref(), C.byref(self.args)))
        want = np.zeros((N, H, V))
        q = pv[:, :H * D].reshape(N, H, D)
        k = pv[:, H * D:(H + G) * D].reshape(N, G, D)
        v = pv[:, (H + G) * D:(H + G) * D + G * V].reshape(N, G, V)
        gate = self.L.sigmoid(pv[:, cols - H:cols])
        freq = self.freq_dev.read_float().astype(np.float64)[:R // 2]
        for i, (slot, start, n) in enumerate(runs):
            r = slice(sq.cu[i], sq.cu[i + 1])
            pos = np.arange(start, start + n)
            turn = lambda t: self.L.rotate_neighbours(t, pos, freq, self.args.rot_mult)
            self.k[slot] = np.concatenate([self.k[slot][:start], turn(k[r])])
            self.v[slot] = np.concatenate([self.v[slot][:start], v[r]])
            want[r] = self.L.chunk_attention(turn(q[r]), self.k[slot], self.v[slot], self.args.scale, self.chunk or None, start)
        return out.read_float(), (want * gate[:, :, None]).reshape(N, H * V)


#             heads, kv heads, dim, vdim, rotated dimensions, chunk
GROUPED = [(6, 3, 24, 16, 16, 20), (4, 4, 40, 72, 40, 64), (8, 2, 128, 128, 128, 100), (20, 1, 64, 32, 24, 33),
           (3, 1, 10, 7, 6, 7), (1, 1, 8, 8, 8, 1), (16, 2, 64, 128, 64, 0), (2, 2, 192, 128, 64, 90), (4, 2, 256, 64, 16, 300),
           (2, 1, 2, 1, 2, 5), (36, 2, 16, 24, 8, 130), (5, 5, 96, 96, 96, 1000), (4, 1, 136, 8, 0, 50)]


def _tolerance(dtype):
    return dict(factor=1.6 if dtype == BF16 else 12)


@TYPES
@pytest.mark.parametrize("sizes", GROUPED, ids=lambda s: "x".join(map(str, s)))
def test_attention_of_prompts_portions_and_steps(backend, gda, arena, L, dtype, sizes):
    """Prompts over several chunks, portions that end and start inside chunks and blocks, single tokens across chunk
    borders, in batches of unequal sequences, into slots that are already full of something else."""
    a = Grouped(gda, backend, arena, L, dtype, *sizes)
    for runs in ([(1, 0, 150), (0, 0, 1)], [(1, 150, 1), (0, 1, 1), (2, 0, 1)], [(0, 2, 2), (1, 151, 33)],
                 [(1, 184, 31), (2, 1, 160), (0, 4, 64)], [(1, 215, 1), (0, 68, 1), (2, 161, 1)], [(1, 216, 1)],
                 [(0, 69, 3)], [(0, 72, 1), (2, 162, 1)], [(2, 163, 130)]):
        near(*a.run(runs), dtype, **_tolerance(dtype))
    a.k[1], a.v[1] = a.k[1][:0], a.v[1][:0]
    near(*a.run([(1, 0, 9), (2, 293, 1)]), dtype, **_tolerance(dtype))   # the slot is used again
    for t in range(9, 30):
        near(*a.run([(1, t, 1), (0, 64 + t, 1)]), dtype, **_tolerance(dtype))


@TYPES
@pytest.mark.parametrize("sizes", [(6, 3, 24, 16, 24, 20), (8, 2, 128, 128, 128, 100), (4, 1, 64, 64, 0, 64), (3, 3, 10, 6, 10, 33),
                                   (2, 1, 192, 128, 192, 65)], ids=lambda s: "x".join(map(str, s)))
@pytest.mark.parametrize("form", ["prompt", "portions", "steps"])
def test_a_key_is_seen_by_its_chunk_behind_it_and_by_no_other_row(backend, gda, arena, L, dtype, sizes, form):
    """A single key whose score stands out by far, first and last of chunks and blocks: the rows of its chunk behind it
    must return its value, rows in front of it and the next chunk's must not."""
    H, G, D, V, R, chunk = sizes
    T = 3 * chunk + 5 if chunk >= 64 else 5 * chunk + 3
    keys = sorted({0, 1, chunk - 1, chunk, chunk + 1, 2 * chunk - 2, 2 * chunk - 1, 2 * chunk, 63, 64, 65, T - 1})
    rng = np.random.default_rng(chunk)
    for key in [k for k in keys if k < T]:
        arena.reset()
        a = Grouped(gda, backend, arena, L, dtype, *sizes, slots=1, tmax=T, mult=1.0, seed=key)
        rows, cols = a.proj(T)
        rows[:, H * D:(H + G) * D] *= 0.05
        target = rng.choice([-1.0, 1.0], (G, D))                        # the rotated key at `key`, up to rounding
        rows[key, H * D:(H + G) * D] = L.rotate_neighbours(target[None], np.array([-key]), a.freq, 1.0).reshape(-1)
        for t in range(T):                                              # every query asks for it with a score of 14
            q = L.rotate_neighbours(target[None], np.array([-t]), a.freq, 1.0)[0] * (14.0 / (D * a.args.scale))
            rows[t, :H * D] = np.repeat(q, H // G, axis=0).reshape(-1)
        got, want = [], []
        cuts = {"prompt": [T], "portions": [2, chunk - 1, 3, chunk, T], "steps": [max(min(keys[-1], T) - 2 * chunk, 1)] + [1] * T}[form]
        at = 0
        for n in cuts:
            n = min(n, T - at)
            if n <= 0:
                break
            g, w = a.run([(0, at, n)], rows[at:at + n])
            got.append(g), want.append(w)
            at += n
        got, want = np.concatenate(got), np.concatenate(want)
        near(got, want, dtype, factor=2.5 if dtype == BF16 else 30)


@TYPES
def test_positions_far_from_the_start(backend, gda, arena, L, dtype):
    """Angles of hundreds of thousands of turns, by portions and by steps, in the 50 places of a chunk."""
    a = Grouped(gda, backend, arena, L, dtype, 4, 2, 16, 8, 16, 50, base=3.0)
    start = 300000
    a.k[1], a.v[1] = np.zeros((start, 2, 16)), np.zeros((start, 2, 8))
    for runs in ([(1, start, 7)], [(1, start + 7, 1)], [(1, start + 8, 1)], [(1, start + 9, 60)], [(1, start + 69, 1)]):
        near(*a.run(runs), dtype, **_tolerance(dtype))


def test_slots_out_of_range_and_unfit_operands(backend, gda, arena, L):
    """Sequences with a slot or a start that does not exist leave the caches alone; operands that do not fit together
    are refused."""
    for dtype in (BF16, F32):
        a = Grouped(gda, backend, arena, L, dtype, 4, 2, 16, 16, 16, 10)
        before = a.kc.read_float().copy()
        for runs in ([(7, 0, 1), (-1, 3, 1)], [(7, 0, 4), (0, -2, 3)]):
            sq = Seqs(gda, arena, runs, kv=False)
            values, cols = a.proj(sq.rows)
            p = put(arena, dtype, values)[0]
            out, work = arena.alloc((sq.rows, 64), dtype), arena.alloc((1 << 16,), U8)
            call = lambda **kw: backend.call("gd_backend_grouped_attend", kw.get("p", p.matrix(cols=cols)), a.freq_dev.view(),
                                             kw.get("kc", a.kc).view(), a.vc.view(), work.view(), kw.get("out", out).view(),
                                             sq.ref(), C.byref(kw.get("args", a.args)))
            ok(call())
            assert (a.kc.read_float() == before).all()
        assert call(p=p.matrix(cols=cols - 1)) == -1
        assert call(kc=a.vc.rows(0, 1)) == -1
        assert call(out=arena.alloc((sq.rows, 63), dtype)) == -1
        assert call(args=gda.GroupedArgs(4, 3, 16, 16, 16, 10, 1.0, 1.0)) == -1
        assert call(args=gda.GroupedArgs(4, 2, 16, 16, 18, 10, 1.0, 1.0)) == -1


# ---- routed feed-forward ----------------------------------------------------------------------------------

class Routed:
    def __init__(self, gda, backend, arena, dtype, E, K, W, F, vocab=60, limit=0.8, seed=0, unused=()):
        self.gda, self.be, self.arena, self.dtype = gda, backend, arena, dtype
        self.E, self.K, self.W, self.F = E, K, W, F
        rng = self.rng = np.random.default_rng(seed + E * K + W)
        some = [e for e in range(E) if e not in unused]
        self.table = np.stack([rng.permutation(some)[:K] for _ in range(vocab)]).astype(np.int32)
        self.args = gda.RoutedArgs(E, K, W, F, limit, 1.702, 1.0 / K)
        self.limit = limit
        self.ug, self.ugv = put(arena, dtype, rng.standard_normal((E * 2 * F, W)) / np.sqrt(W))
        self.dn, self.dnv = put(arena, dtype, rng.standard_normal((E * W, F)) / np.sqrt(F))
        self.table_dev = ints(arena, self.table)

    def route(self, ids, more=()):
        """The tables of this layer, and of others in the same launch: views, place, first."""
        N = len(ids)
        held = []
        jobs = (self.gda.RouteJob * (1 + len(more)))()
        for j, r in enumerate((self,) + tuple(more)):
            place, first = self.arena.alloc((N * r.K,), I32), self.arena.alloc((r.E + 1,), I32)
            tiles = self.arena.alloc((2 + 2 * self.gda.lib().gd_backend_route_tiles(C.byref(r.args), N, 1),), I32)
            views = [C.pointer(t.view()) for t in (r.table_dev, place, first, tiles)]
            jobs[j] = self.gda.RouteJob(*views, C.pointer(r.args))
            held.append((place, first, tiles, views))
        ok(self.be.call("gd_backend_route_by_tables", jobs, len(jobs), ints(self.arena, ids).view(), self.dtype))
        return held

    def check_places(self, ids, place, first):
        """Every choice has a place of its own among its expert's rows."""
        place, first = place.read().reshape(len(ids), self.K), first.read()
        counts = np.zeros(self.E, int)
        seen = set()
        for n, id_ in enumerate(ids):
            for k in range(self.K):
                if not 0 <= id_ < len(self.table):
                    assert place[n, k] == -1
                    continue
                e = self.table[id_, k]
                assert first[e] <= place[n, k] < first[e + 1]
                seen.add(int(place[n, k]))
                counts[e] += 1
        assert len(seen) == counts.sum() and (np.diff(first) == counts).all() and first[0] == 0
        return place

    def run(self, ids, h):
        N, P = len(ids), len(ids) * self.K + self.gda.ROUTED_PAD
        place, first, tiles, views = self.route(ids)[0]
        at = self.check_places(ids, place, first)
        hv = put(self.arena, self.dtype, h)[1]
        packed = np.full((P, self.W), np.nan)                           # rows nobody asked for may hold anything
        for n in range(N):
            for k in range(self.K):
                if at[n, k] >= 0:
                    packed[at[n, k]] = hv[n]
        rows = self.arena.alloc((P, self.W), self.dtype).write_float(packed)
        act = self.arena.alloc((P, self.F), self.dtype).write_float(np.full((P, self.F), np.nan))
        out = self.arena.alloc((P, self.W), self.dtype)
        routes = self.gda.Routes(views[2], views[3], N)
        ok(self.be.call("gd_backend_routed_mlp", rows.view(), self.ug.view(), self.dn.view(), act.view(), out.view(),
                        C.byref(routes), C.byref(self.args)))
        got = out.read_float()
        want = np.zeros((N, self.K, self.W))
        mine = np.zeros((N, self.K, self.W))
        for n, id_ in enumerate(ids):
            for k in range(self.K):
                if at[n, k] < 0:
                    continue
                e = self.table[id_, k]
                u = self.ugv[e * 2 * self.F:(e + 1) * 2 * self.F] @ hv[n]
                a = _clamped(u[:self.F], u[self.F:], self.limit)
                want[n, k] = self.dnv[e * self.W:(e + 1) * self.W] @ a
                mine[n, k] = got[at[n, k]]
        return mine, want


@TYPES
@pytest.mark.parametrize("E,K,W,F,N", [
    (5, 2, 64, 40, 3), (7, 1, 96, 24, 40), (3, 3, 30, 21, 11), (1, 1, 8, 8, 1), (16, 2, 256, 128, 33), (4, 2, 72, 8, 300),
    (6, 2, 256, 128, 400), (3, 1, 192, 320, 500), (2, 2, 128, 256, 900), (3, 2, 256, 128, 1300), (3, 2, 136, 200, 1200), (2, 1, 320, 192, 1600), (2, 1, 512, 64, 1700), (300, 3, 64, 16, 70),
    (9, 4, 128, 200, 260)])
def test_routed_feed_forward(backend, gda, arena, dtype, E, K, W, F, N):
    """Few and many rows per expert, experts without rows, sizes on and off the tiles of every kernel."""
    r = Routed(gda, backend, arena, dtype, E, K, W, F, unused=(1,) if E > 4 else ())
    ids = r.rng.integers(0, 60, N)
    if N > 20:
        ids[5], ids[9] = -1, 60                                         # ids that do not exist have no places
        ids[10:18] = ids[10]
    got, want = r.run(ids, r.rng.standard_normal((N, W)))
    near(got, want, dtype, factor=2)


def test_routes_of_many_layers_in_one_call(backend, gda, arena):
    r = [Routed(gda, backend, arena, BF16, 3 + i % 9, 1 + i % 3, 8, 8, seed=i) for i in range(70)]
    for N in (1, 50, 3000):
        ids = r[0].rng.integers(0, 60, N)
        for layer, (place, first, _, _) in zip(r, r[0].route(ids, r[1:])):
            layer.check_places(ids, place, first)


def test_most_experts(backend, gda, arena):
    r = Routed(gda, backend, arena, BF16, 4096, 2, 8, 8, vocab=4000)
    ids = r.rng.integers(0, 4000, 5000)
    place, first, _, _ = r.route(ids)[0]
    r.check_places(ids, place, first)
    args = gda.RoutedArgs(4097, 2, 8, 8, 1.0, 1.0, 1.0)
    with pytest.raises(AssertionError):
        r.args = args
        r.route(ids)


# ---- decoders ---------------------------------------------------------------------------------------------

A = B.attention
MODELS = {
    "mixed": B.config([(A(), B.dense()), (A(heads=4, kv_heads=1, dim=32, vdim=40, rot_dims=32, chunk=33), B.moe()), 1,
                       (A(chunk=9, scaling=None), None), 1]),
    "dense": B.config([(A(heads=2, kv_heads=2, dim=16, vdim=24, rot_dims=4, chunk=50, scaling={"factor": 8.0, "original": 32, "fast": 1.0, "slow": 1.0}), B.dense(30))],
                      vocab=70, width=40, eps=1e-3, embedding_scale=1.0),
    "experts": B.config([(A(heads=1, kv_heads=1, dim=8, vdim=8, rot_dims=8, chunk=12), B.moe(experts=1, top=1, ff=16, limit=0.5, shared=None)),
                         (A(heads=8, kv_heads=4, chunk=70), B.moe(experts=9, top=4, ff=24, limit=2.0, shared=8, shared_limit=0.3)), 0],
                        vocab=101, width=48, embedding_scale=7.0),
    "odd": B.config([(A(heads=3, kv_heads=1, dim=10, vdim=7, rot_dims=6, chunk=7), B.moe(experts=3, top=3, ff=9, shared=11)), 2,
                     (A(heads=2, kv_heads=2, dim=6, vdim=5, rot_dims=2, base=50.0, chunk=1), B.dense(13))], vocab=37, width=30),
    "wide": B.config([(A(heads=20, kv_heads=1, dim=64, vdim=128, rot_dims=64, base=5e5, chunk=40), B.moe(experts=4, top=2, ff=128, shared=192)),
                      (A(heads=4, kv_heads=2, dim=128, vdim=64, rot_dims=96, chunk=64), B.dense(512))], width=256),
    "large heads": B.config([(A(heads=2, kv_heads=1, dim=192, vdim=128, rot_dims=192, chunk=30), B.dense(64)), 0], width=128),
}


@pytest.fixture(scope="module")
def D(gda):
    from gradients_c_amd import decoder as module
    return module


@pytest.fixture(scope="module")
def models(tmp_path_factory, L):
    """name -> (folder, tokens [3][T], plain logits [3][T, vocab], configuration, weights)"""
    made = {}

    def get(name, T=90):
        if (name, T) not in made:
            cfg = MODELS[name]
            t = B.weights(cfg, 11)
            rng = np.random.default_rng(12)
            tokens = [rng.integers(0, cfg["vocab"], n) for n in (T, T // 2 + 1, T // 3)]
            folder = B.save(str(tmp_path_factory.mktemp("model")), cfg, t)
            made[name, T] = (folder, tokens, [L.forward_bonatar(cfg, t, k) for k in tokens], cfg, t)
        return made[name, T]
    return get


@DTYPES
@pytest.mark.parametrize("name", list(MODELS))
def test_prompt_portions_and_decoding_agree_with_the_plain_model(D, models, name, compute):
    folder, tokens, want, cfg, _ = models(name)
    d = decoder(D, folder, compute, max_seq=100, batch=3)
    try:
        t, w = tokens[0], want[0]
        slot = d.acquire()
        logits_near(d.extend({slot: t}), w, compute)                          # the whole prompt
        d.release(slot)
        for cut in (2, 3, 17, 33, 64):                                        # portions, in a slot that was used
            slot = d.acquire()
            got = [d.extend({slot: t[a:a + cut]}) for a in range(0, len(t), cut)]
            logits_near(np.concatenate(got), w, compute)
            d.release(slot)
        slot = d.acquire()
        got = [d.extend({slot: t[:40]}, want=[])] + [d.extend({slot: [k]}) for k in t[40:]]
        logits_near(np.concatenate(got[1:]), w[40:], compute)                 # a prompt, then token by token
        d.release(slot)
        slot = d.acquire()
        got = np.concatenate([d.extend({slot: [k]}) for k in t[:45]])         # token by token from the first
        logits_near(got, w[:45], compute)
    finally:
        d.close()


@DTYPES
@pytest.mark.parametrize("name", ["mixed", "wide"])
def test_batches_of_unequal_requests(D, models, name, compute):
    """Requests that start, continue and end at different times share steps; each must give what it gives alone."""
    folder, tokens, want, cfg, _ = models(name)
    d = decoder(D, folder, compute, max_seq=100, batch=4)
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
            logits_near(g, want[req[s]][:len(g)], compute)
        d.release(b)                                                          # a slot is freed and used again
        b = d.acquire()
        out = d.extend({a: tokens[0][at[a]:at[a] + 1], b: tokens[2][:25]})
        logits_near(out[1:], want[2][:25], compute)
        logits_near(out[:1], want[0][at[a]:at[a] + 1], compute)
        out = d.extend({b: tokens[2][25:29]}, want=[3, 0])                    # only wanted places, in any order
        logits_near(out, want[2][[28, 25]], compute)
    finally:
        d.close()


@DTYPES
@pytest.mark.parametrize("name", ["mixed", "wide"])
def test_prefill_step_and_resident_session(D, models, name, compute):
    """The calls every model of the library has: packed prefill of all rows, steps with host tokens, and the resident
    session whose greedy tokens feed themselves, and their routes, through a replayed graph."""
    folder, tokens, want, cfg, _ = models(name)
    prompts = [t[:12 + 5 * i] for i, t in enumerate(tokens)]
    cu = np.concatenate([[0], np.cumsum([len(p) for p in prompts])])
    factor = 1 if compute == "bfloat16" else 50
    d = decoder(D, folder, compute, max_seq=64, batch=3)
    try:
        logits, nxt, gap = d.prefill(np.concatenate(prompts), cu)
        for i, p in enumerate(prompts):
            logits_near(logits[i:i + 1].astype(np.float64), want[i][len(p) - 1:len(p)], compute, factor=factor)
        for k in range(3):
            step = [tokens[i][len(p) + k] for i, p in enumerate(prompts)]
            logits, nxt, gap = d.step(step)
            for i, p in enumerate(prompts):
                logits_near(logits[i:i + 1].astype(np.float64), want[i][len(p) + k:len(p) + k + 1], compute, factor=factor)
        d.prefill(np.concatenate(prompts), cu)
        first = nxt
        by_step = []
        cur = first
        for _ in range(25):
            _, cur, _ = d.step(cur)
            by_step.append(cur.copy())
        d.prefill(np.concatenate(prompts), cu)
        ids, gaps, _ = d.run_resident(first, 25)
        for k in range(25):
            same = ids[k] == by_step[k]
            if not same.all():
                assert gaps[k][~same].max() < 1e-2
                break
    finally:
        d.close()


def _greedy(L, cfg, weights, prompt, n):
    seq, gaps = list(prompt), []
    for _ in range(n):
        row = L.forward_bonatar(cfg, weights, seq)[-1]
        top = np.sort(row)[-2:]
        gaps.append(top[1] - top[0])
        seq.append(int(row.argmax()))
    return seq[len(prompt):], gaps


def test_greedy_generation_through_the_entry_point(D, L, models):
    folder, tokens, _, cfg, w = models("mixed")
    prompts = [tokens[0][:9], tokens[1][:5], tokens[2][:14]]
    cu = np.concatenate([[0], np.cumsum([len(p) for p in prompts])])
    d = decoder(D, folder, "float32", max_seq=70, batch=3)
    try:
        out = d.generate(np.concatenate(prompts), cu, 40)
        sampled = d.generate(np.concatenate(prompts), cu, 20, temperature=0.8, rng_state=5)
        again = d.generate(np.concatenate(prompts), cu, 20, temperature=0.8, rng_state=5)
    finally:
        d.close()
    for p, got in zip(prompts, out):
        want, gaps = _greedy(L, cfg, w, p, 40)
        assert len(got) == 40
        for k in range(40):
            if got[k] != want[k]:
                assert gaps[k] < 1e-3, (k, gaps[k])
                break
    assert all((a == b).all() for a, b in zip(sampled, again))
    assert any((a != b[:20]).any() for a, b in zip(sampled, out))


@DTYPES
def test_the_inference_program_opens_a_model_folder(D, models, compute):
    folder, tokens, _, _, _ = models("mixed")
    prompt = tokens[0][:11]
    exe = os.path.join(ROOT, "gradients.c_amd", "gpt_lm_infer")
    d = decoder(D, folder, compute, max_seq=50, batch=1)
    try:
        greedy = d.generate(prompt, [0, len(prompt)], 30)[0].tolist()
    finally:
        d.close()
    r = subprocess.run([exe, "--checkpoint", folder, "--dtype", compute, "--token-ids", ",".join(str(int(t)) for t in prompt),
                        "--max-new-tokens", "30"], capture_output=True, timeout=60)
    out = r.stdout.decode()
    assert r.returncode == 0 and "architecture=Bonatar" in out, (r.returncode, r.stderr)
    assert [int(v) for v in next(l for l in out.splitlines() if l.startswith("ids:"))[4:].split()] == greedy


@DTYPES
def test_long_decoding(D, L, tmp_path, compute):
    """Hundreds of single tokens behind a short prompt, through many chunks of one layer and the pieces of another's."""
    cfg = B.config([(A(chunk=16), B.moe()), (A(dim=32, vdim=32, rot_dims=32, chunk=260), B.dense())], vocab=64, width=48)
    w = B.weights(cfg, 21)
    t = np.random.default_rng(22).integers(0, 64, 420)
    want = L.forward_bonatar(cfg, w, t)
    d = decoder(D, B.save(str(tmp_path), cfg, w), compute, max_seq=420)
    try:
        slot = d.acquire()
        d.extend({slot: t[:5]}, want=[])
        got = np.concatenate([d.extend({slot: [k]}) for k in t[5:]])
        logits_near(got, want[5:], compute)
    finally:
        d.close()


def test_long_prompt_in_one_step_and_in_portions(D, L, tmp_path):
    cfg = B.config([(A(heads=4, kv_heads=2, dim=32, vdim=32, rot_dims=32, chunk=300), B.moe(experts=3, ff=128)),
                    (A(heads=2, kv_heads=1, dim=64, vdim=64, rot_dims=32, chunk=128), B.dense(256))], vocab=64, width=128)
    w = B.weights(cfg, 31)
    t = np.random.default_rng(32).integers(0, 64, 1400)
    want = L.forward_bonatar(cfg, w, t)
    d = decoder(D, B.save(str(tmp_path), cfg, w), "bfloat16", max_seq=1404, batch=2)
    try:
        logits_near(d.extend({d.acquire(): t}), want, "bfloat16")
        slot = d.acquire()
        got = [d.extend({slot: t[a:b]}) for a, b in ((0, 255), (255, 257), (257, 258), (258, 640), (640, 900), (900, 1400))]
        logits_near(np.concatenate(got), want, "bfloat16")
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
        logits_near(got, want[0][places], "float32")
