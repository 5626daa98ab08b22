"""Bonatar decoders without a GPU: reading configuration and weights, shared weights, slots (against the device-less
backend), and the plain model's own mechanisms against closed forms."""
import json

import numpy as np
import pytest

import bonatar_models as B

BAD_STATE, UNSUPPORTED, INVALID = -5, -6, -1


@pytest.fixture(scope="module")
def folder(tmp_path_factory):
    cfg = B.config([(B.attention(), B.dense()), (B.attention(chunk=9), B.moe()), 1, (B.attention(kv_heads=6), None)])
    return B.save(str(tmp_path_factory.mktemp("model")), cfg, B.weights(cfg, 1)), cfg


def test_registry_names_the_architecture(host, folder):
    _, D = host
    m = D.Model(folder[0])
    assert (m.architecture, m.vocab, m.n_layers) == ("Bonatar", 150, 4)
    m.close()


@pytest.mark.parametrize("change,status", [
    (lambda c: c.pop("vocab"), BAD_STATE),
    (lambda c: c["norm"].pop("eps"), BAD_STATE),
    (lambda c: c["norm"].update(eps=-1.0), BAD_STATE),
    (lambda c: c.pop("embedding"), BAD_STATE),
    (lambda c: c["layers"][0].update(type="mamba2"), UNSUPPORTED),
    (lambda c: c["layers"][0].pop("type"), BAD_STATE),
    (lambda c: c["layers"][0].pop("mixer"), BAD_STATE),
    (lambda c: c["layers"][0]["mixer"].update(kv_heads=4), BAD_STATE),
    (lambda c: c["layers"][0]["mixer"].pop("scale"), BAD_STATE),
    (lambda c: c["layers"][0]["mixer"].pop("rot"), BAD_STATE),
    (lambda c: c["layers"][0]["mixer"]["rot"].update(dims=7), BAD_STATE),
    (lambda c: c["layers"][0]["mixer"]["rot"].update(dims=26), BAD_STATE),
    (lambda c: c["layers"][0]["mixer"]["rot"].update(base=0), BAD_STATE),
    (lambda c: c["layers"][0]["mixer"]["rot"]["scaling"].pop("slow"), BAD_STATE),
    (lambda c: c["layers"][0]["mixer"]["rot"]["scaling"].update(factor=0), BAD_STATE),
    (lambda c: c["layers"][0]["mixer"]["mask"].update(size=0), BAD_STATE),
    (lambda c: c["layers"][0]["mlp"].update(kind="other"), UNSUPPORTED),
    (lambda c: c["layers"][0]["mlp"].pop("ff"), BAD_STATE),
    (lambda c: c["layers"][3].update(mlp=B.moe(experts=2, top=3)), BAD_STATE),
    (lambda c: c["layers"][3].update(mlp=B.moe(experts=5000)), UNSUPPORTED),
    (lambda c: c["layers"][3].update(mlp=dict(B.moe(), router=None)), BAD_STATE),
    (lambda c: c["layers"][3].update(mlp=dict(B.moe(), expert={"ff": 8})), BAD_STATE),
    (lambda c: c["layers"][3].update(mlp=dict(B.moe(), shared={"limit": 8})), BAD_STATE),
    (lambda c: c["layers"][2].update(weights_of=9), BAD_STATE),
    (lambda c: c["layers"][2].update(weights_of=-1), BAD_STATE),
    (lambda c: c["layers"][2].update(weights_of="one"), BAD_STATE),
    (lambda c: c["layers"][2].update(weights_of=0), BAD_STATE),                       # of other sizes
    (lambda c: c["layers"][1].update(weights_of=2) or c["layers"][2].update(weights_of=1), BAD_STATE),   # in a circle
])
def test_configuration_errors_are_refused(host, folder, tmp_path, change, status):
    pkg, D = host
    cfg = json.loads(json.dumps(folder[1]))
    change(cfg)
    B.save(str(tmp_path), cfg, {"embed": np.zeros((2, 2), np.float32)})
    with pytest.raises(pkg.GdError) as e:
        D.Model(str(tmp_path))
    assert e.value.status == status, str(e.value)


@pytest.mark.parametrize("change", [
    lambda c: c["layers"][0]["mixer"]["rot"].pop("scaling"),
    lambda c: c["layers"][0]["mixer"].pop("mask"),
    lambda c: c["layers"][0].pop("mlp"),
    lambda c: c["layers"][2].update(weights_of=2),                                    # its own
    lambda c: c["layers"][3].update(c["layers"][1], weights_of=2),                    # through another one
])
def test_optional_parts_of_the_configuration(host, folder, tmp_path, change):
    _, D = host
    cfg = json.loads(json.dumps(folder[1]))
    change(cfg)
    B.save(str(tmp_path), cfg, {"embed": np.zeros((2, 2), np.float32)})
    D.Model(str(tmp_path)).close()


def test_weights_that_do_not_fit_are_refused(host, folder, tmp_path):
    pkg, D = host
    cfg = folder[1]
    t = B.weights(cfg, 1)
    table = t["l1.mlp.table"]
    twice, outside, below = table.copy(), table.copy(), table.copy()
    twice[7, 1] = twice[7, 0]
    outside[149, 0] = 5
    below[0, 0] = -1
    for name, array, status in (("l0.mix.g", t["l0.mix.g"][:-1], BAD_STATE), ("l1.mlp.e4.down", None, BAD_STATE),
                                ("l1.mlp.shared.gate", t["l1.mlp.shared.gate"].T, BAD_STATE), ("head", None, BAD_STATE),
                                ("l1.mlp.table", table[:, :1], BAD_STATE), ("l1.mlp.table", table.astype(np.float32), UNSUPPORTED),
                                ("l1.mlp.table", twice, BAD_STATE), ("l1.mlp.table", outside, BAD_STATE),
                                ("l1.mlp.table", below, BAD_STATE), ("l3.mix.q", np.zeros((144, 64), np.int32), UNSUPPORTED)):
        changed = dict(t)
        if array is None:
            changed.pop(name)
        else:
            changed[name] = array
        m = D.Model(B.save(str(tmp_path / "m"), cfg, changed))
        with pytest.raises(pkg.GdError) as e:
            m.decoder(max_seq=32)
        assert e.value.status == status, name
        m.close()


def test_shared_weights_are_held_once_and_caches_are_not(host, tmp_path):
    """Three runs of one layer need its weights once and three caches; caches hold a chunk, not the sequence."""
    _, D = host

    def memory(layers, max_seq):
        cfg = B.config(layers)
        m = D.Model(B.save(str(tmp_path / "m"), cfg, B.weights(cfg, 1)))
        o = D.ModelOptions(max_seq, 8, 16, 2, 0)
        mem = m.memory(o)
        m.close()
        return mem.params_bytes, mem.state_bytes
    layer = (B.attention(chunk=64), B.moe(top=1))
    one, shared = memory([layer], 640), memory([layer, 0, 0], 640)
    cache = 8 * 64 * 3 * (24 + 16) * 2
    assert one[0] == shared[0] and shared[1] - one[1] == 2 * cache
    longer = memory([layer], 6400)
    assert longer[1] - one[1] < 8 * 6400 * 8                # no cache of the longer sequence, only its records
    apart = memory([layer, layer, layer], 640)
    assert apart[0] > 2 * one[0] and apart[1] > shared[1]   # (a table of routes each)


def test_slots_and_arguments_of_extend(host, folder):
    pkg, D = host
    m = D.Model(folder[0])
    d = m.decoder(max_seq=20, batch=2, max_step_tokens=16)
    try:
        a, b = d.acquire(), d.acquire()

        def status(fn):
            with pytest.raises(pkg.GdError) as e:
                fn()
            return e.value.status
        d.extend({a: [1, 2, 3], b: [4]}, want=[])
        assert list(d.positions) == [3, 1]
        assert status(lambda: d.extend({a: list(range(18))}, want=[])) == INVALID
        d.release(a)
        assert d.acquire() == a and list(d.positions) == [0, 1]
    finally:
        d.close()
        m.close()


# ---- the plain model's mechanisms -----------------------------------------------------------------------------

def test_plain_yarn_frequencies():
    from oracle import layer_list as L
    base, dims, s = 10000.0, 64, {"factor": 8.0, "original": 4096, "fast": 32.0, "slow": 1.0}
    f, mult = L.yarn_frequencies(base, dims, s)
    raw, one = L.yarn_frequencies(base, dims, None)
    assert one == 1.0 and np.isclose(mult, 0.1 * np.log(8.0) + 1)
    turns = raw * 4096 / (2 * np.pi)
    assert np.allclose(f[turns > 40], raw[turns > 40]) and np.allclose(f[turns < 0.7], raw[turns < 0.7] / 8)
    between = (turns < 20) & (turns > 2)
    assert between.any() and np.all((f < raw)[between] & (f > raw / 8)[between])
    # both ends on one pair: a step
    f, _ = L.yarn_frequencies(base, dims, dict(s, fast=1e9, slow=1e9))
    assert np.allclose(f[1:], raw[1:] / 8) and np.isclose(f[0], raw[0])


def test_plain_rotation_and_chunks():
    from oracle import layer_list as L
    rng = np.random.default_rng(4)
    freq = np.array([1.0, 0.3])
    q, k = rng.standard_normal((9, 2, 6)), rng.standard_normal((9, 2, 6))
    pos = np.arange(9)
    rq, rk = L.rotate_neighbours(q, pos, freq, 1.0), L.rotate_neighbours(k, pos, freq, 1.0)
    sq, sk = L.rotate_neighbours(q, pos + 5, freq, 1.0), L.rotate_neighbours(k, pos + 5, freq, 1.0)
    assert np.allclose(np.einsum("ihd,jhd->hij", rq, rk), np.einsum("ihd,jhd->hij", sq, sk))
    assert np.allclose(rq[..., 4:], q[..., 4:]) and np.allclose(rq[0], q[0])
    assert np.allclose(L.rotate_neighbours(q, pos, freq, 2.0)[..., :4], 2 * rq[..., :4])
    v = rng.standard_normal((9, 1, 5))
    out = L.chunk_attention(q, np.zeros((9, 1, 6)), v, 1.0, 4)      # equal scores: running mean inside the chunk
    for i in range(9):
        assert np.allclose(out[i], v[i // 4 * 4:i + 1, 0].mean(0))
    assert np.allclose(L.chunk_attention(q, k, np.repeat(v, 2, 1), 1.0, 1), np.repeat(v, 2, 1))
    assert np.allclose(L.chunk_attention(q, k, np.repeat(v, 2, 1), 1.0, None), L.causal_attention(q, k, np.repeat(v, 2, 1), 1.0))


def test_plain_experts():
    from oracle import layer_list as L
    rng = np.random.default_rng(5)
    one = {"gate": np.eye(3), "up": np.eye(3), "down": np.eye(3)}
    h = np.array([[0.5, -2.0, 3.0]])
    g, u = np.array([0.5, -2.0, 1.0]), np.array([0.5, -1.0, 1.0])   # clamped to 1: gates above, values on both sides
    assert np.allclose(L.clamped_expert(h, one, "", 1.0), g / (1 + np.exp(-1.702 * g)) * (u + 1))
    assert np.allclose(L.square_relu_mlp(h, one), [[0.25, 0, 9.0]])
    w = {"table": np.array([[0, 2], [1, 0]])}
    for e in range(3):
        w.update({"e%d.%s" % (e, k): rng.standard_normal((3, 3)) for k in one})
    h = rng.standard_normal((2, 3))
    m = {"router": {"top": 2}, "expert": {"limit": 1.0}, "shared": None}
    y = L.table_routed_mlp(h, w, [1, 0], m)
    e = [L.clamped_expert(h, w, "e%d." % i, 1.0) for i in range(3)]
    assert np.allclose(y[0], (e[1] + e[0])[0] / 2) and np.allclose(y[1], (e[0] + e[2])[1] / 2)
