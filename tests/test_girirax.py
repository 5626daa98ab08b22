"""Girirax decoders without a GPU: reading configuration and weights, the model registry, slots and argument checks
(against the device-less backend), and the plain model's own mechanisms against closed forms."""
import ctypes as C
import json
import os
import struct
import subprocess

import numpy as np
import pytest

import girirax_models as G

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
BAD_STATE, UNSUPPORTED, IO, INVALID, BUSY = -5, -6, -9, -1, -4


@pytest.fixture(scope="module")
def folder(tmp_path_factory):
    cfg = G.config([G.mamba(), (G.latent(), None), G.latent(heads=3, kv_rank=32)])
    return G.save(str(tmp_path_factory.mktemp("model")), cfg, G.weights(cfg, 1)), cfg


def _open(D, path):
    m = D.Model(path)
    m.close()
    return m


def test_registry_names_the_architecture_of_a_path(host, folder):
    _, D = host
    m = _open(D, folder[0])
    assert (m.architecture, m.vocab, m.n_layers) == ("Girirax", 192, 3)
    golden = os.path.join(ROOT, "tests", "golden", "gpt_small_seed777.gdckpt")
    m = _open(D, golden)
    assert m.architecture == "gpt_lm" and m.n_layers >= 1


@pytest.mark.parametrize("change,status", [
    (lambda c: c.update(architecture="Other"), UNSUPPORTED),
    (lambda c: c.pop("architecture"), BAD_STATE),
    (lambda c: c.pop("vocab"), BAD_STATE),
    (lambda c: c.update(width=-4), BAD_STATE),
    (lambda c: c.update(width=12.5), BAD_STATE),
    (lambda c: c.pop("residual_mult"), BAD_STATE),
    (lambda c: c["norm"].pop("eps"), BAD_STATE),
    (lambda c: c.pop("embedding"), BAD_STATE),
    (lambda c: c.update(layers=[]), BAD_STATE),
    (lambda c: c["layers"][0].update(type="window"), UNSUPPORTED),
    (lambda c: c["layers"][0]["mixer"].update(groups=3), BAD_STATE),
    (lambda c: c["layers"][0]["mixer"].update(norm_groups=5), BAD_STATE),
    (lambda c: c["layers"][0]["mixer"].pop("state"), BAD_STATE),
    (lambda c: c["layers"][1]["mixer"].pop("scale"), BAD_STATE),
    (lambda c: c["layers"][1]["mixer"]["rot"].update(dims=4), BAD_STATE),
    (lambda c: c["layers"][1]["mixer"]["rot"].update(base=0), BAD_STATE),
    (lambda c: c["layers"][2]["mlp"].update(kind="routed"), UNSUPPORTED),
    (lambda c: c["layers"][2]["mlp"].pop("ff"), BAD_STATE),
])
def test_configuration_errors_are_refused(host, folder, tmp_path, change, status):
    pkg, D = host
    cfg = json.loads(json.dumps(folder[1]))
    change(cfg)
    G.save(str(tmp_path), cfg, {"embed": np.zeros((2, 2), np.float32)})
    with pytest.raises(pkg.GdError) as e:
        D.Model(str(tmp_path))
    assert e.value.status == status, str(e.value)


def test_missing_and_malformed_files(host, folder, tmp_path):
    pkg, D = host

    def status(path):
        with pytest.raises(pkg.GdError) as e:
            D.Model(path)
        return e.value.status
    assert status(str(tmp_path / "nowhere")) == IO
    empty = tmp_path / "empty"
    empty.mkdir()
    assert status(str(empty)) == IO
    (empty / "config.json").write_text("{not json")
    assert status(str(empty)) == BAD_STATE
    (empty / "config.json").write_text(json.dumps(folder[1]))
    assert status(str(empty)) == IO
    good = open(os.path.join(folder[0], "model.safetensors"), "rb").read()

    def weights(data):
        (empty / "model.safetensors").write_bytes(data)
        return status(str(empty))
    assert weights(b"\0\0\0") == IO
    assert weights(struct.pack("<Q", 1 << 40)) == IO
    assert weights(good[:-2]) == IO                                   # data ends early
    head = {"a": {"dtype": "BF16", "shape": [2], "data_offsets": [0, 2]}}
    text = json.dumps(head).encode()
    assert weights(struct.pack("<Q", len(text)) + text + b"\0" * 4) == BAD_STATE   # bytes do not fit the shape
    head["a"].update(dtype="I64", data_offsets=[0, 16])
    text = json.dumps(head).encode()
    assert weights(struct.pack("<Q", len(text)) + text + b"\0" * 16) == UNSUPPORTED


def test_weights_of_another_shape_are_refused_before_anything_is_written(host, folder, tmp_path):
    pkg, D = host
    cfg = folder[1]
    t = G.weights(cfg, 1)
    for name, array in (("l1.mix.uk", t["l1.mix.uk"][:-1]), ("l0.mix.conv", t["l0.mix.conv"][:, :-1]), ("embed", None)):
        changed = dict(t)
        if array is None:
            changed.pop(name)
        else:
            changed[name] = array
        m = D.Model(G.save(str(tmp_path / name), cfg, changed))
        with pytest.raises(pkg.GdError) as e:
            m.decoder(max_seq=32)
        assert e.value.status == BAD_STATE
        m.close()


def test_slots_and_arguments_of_extend(host, folder):
    pkg, D = host
    m = D.Model(folder[0])
    d = m.decoder(max_seq=20, batch=2, max_step_tokens=16)
    try:
        a, b = d.acquire(), d.acquire()
        assert {a, b} == {0, 1}

        def status(fn):
            with pytest.raises(pkg.GdError) as e:
                fn()
            return e.value.status
        assert status(d.acquire) == BUSY
        d.extend({a: [1, 2, 3], b: [4]}, want=[])
        assert list(d.positions) == [3, 1]
        assert status(lambda: d.extend({a: list(range(18))}, want=[])) == INVALID   # past max_seq
        assert status(lambda: d.extend({a: list(range(10)), b: list(range(10))}, want=[])) == INVALID  # past the step
        assert status(lambda: d.extend({2: [1]}, want=[])) == INVALID
        assert status(lambda: d.extend({a: [1]}, want=[1])) == INVALID
        d.release(a)
        assert status(lambda: d.release(a)) == INVALID
        assert d.acquire() == a and list(d.positions) == [0, 1]
    finally:
        d.close()
        m.close()
    golden = D.Model(os.path.join(ROOT, "tests", "golden", "gpt_small_seed777.gdckpt"))
    g = golden.decoder(max_seq=16, heads=4)
    try:
        with pytest.raises(pkg.GdError) as e:
            g.extend({0: [1]}, want=[])
        assert e.value.status == UNSUPPORTED
    finally:
        g.close()
        golden.close()


def test_trace_run_refuses_bad_command_lines():
    exe = os.path.join(ROOT, "gradients.c_amd", "trace_run")
    if not os.path.exists(exe):
        pytest.skip("not built")
    for args in ([], ["--model", "x"], ["--model", "x", "--dtype", "int8", "--out", ".", "--max-tokens", "4"],
                 ["--model", "x", "--dtype", "float32", "--out", ".", "--max-tokens", "0"]):
        assert subprocess.run([exe] + args, capture_output=True, stdin=subprocess.DEVNULL).returncode == 2
    r = subprocess.run([exe, "--model", "/nonexistent", "--dtype", "float32", "--out", ".", "--max-tokens", "4"],
                       capture_output=True, stdin=subprocess.DEVNULL)
    assert r.returncode == 1 and b"no such file" in r.stderr


# ---- the plain model's mechanisms -----------------------------------------------------------------------------

def test_plain_recurrence_matches_the_unrolled_sum():
    from oracle import layer_list as L
    rng = np.random.default_rng(3)
    T, H, P, N = 7, 2, 3, 4
    x, b, c = rng.standard_normal((T, H, P)), rng.standard_normal((T, 1, N)), rng.standard_normal((T, 1, N))
    dt, a_log, d = rng.uniform(0.1, 1, (T, H)), rng.uniform(-1, 1, H), rng.standard_normal(H)
    y = L.ssd_scan(x, b, c, dt, a_log, d)
    for h in range(H):
        for t in range(T):
            want = d[h] * x[t, h]
            for s in range(t + 1):
                decay = np.exp(-np.exp(a_log[h]) * dt[s + 1:t + 1, h].sum())
                want = want + decay * dt[s, h] * (c[t, 0] @ b[s, 0]) * x[s, h]
            assert np.allclose(y[t, h], want)


def test_plain_rotation_attention_norms():
    from oracle import layer_list as L
    rng = np.random.default_rng(4)
    q, k = rng.standard_normal((9, 2, 6)), rng.standard_normal((9, 2, 6))
    pos = np.arange(9)
    rq, rk = L.rotate_half(q, pos, 100.0, 6), L.rotate_half(k, pos, 100.0, 6)
    shifted = L.rotate_half(q, pos + 5, 100.0, 6), L.rotate_half(k, pos + 5, 100.0, 6)
    assert np.allclose(np.einsum("ihd,jhd->hij", rq, rk), np.einsum("ihd,jhd->hij", *shifted))
    assert np.allclose(np.linalg.norm(rq, axis=-1), np.linalg.norm(q, axis=-1)) and np.allclose(rq[0], q[0])
    v = rng.standard_normal((9, 2, 5))
    out = L.causal_attention(q, np.zeros_like(k), v, 1.0)
    assert np.allclose(out, np.cumsum(v, axis=0) / (pos + 1)[:, None, None])   # equal scores: running mean
    z, w = rng.standard_normal((3, 8)), rng.uniform(0.5, 2, 8)
    parts = L.gated_group_norm(np.ones((3, 8)), z, w, 2, 0.0) / w
    assert np.allclose((parts.reshape(3, 2, 4) ** 2).mean(-1), 1)
    u = rng.standard_normal((5, 3))
    taps = np.zeros((3, 4))
    taps[:, 1] = 1     # two tokens back
    assert np.allclose(L.causal_conv(u, taps, np.zeros(3))[2:], u[:-2])
    assert np.allclose(L.causal_conv(u, taps, np.ones(3))[:2], 1)
