"""Small Bonatar configurations with seeded random weights for the tests."""
import numpy as np

from girirax_models import rounded, save  # noqa: F401  (save: for the tests)


def attention(heads=6, kv_heads=3, dim=24, vdim=16, rot_dims=16, base=1000.0, chunk=20, scale=None, scaling="default"):
    if scaling == "default":
        scaling = {"factor": 4.0, "original": 60, "fast": 4.0, "slow": 0.5}
    rot = {"base": base, "dims": rot_dims}
    if scaling is not None:
        rot["scaling"] = scaling
    return {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale or 1.2 * dim ** -0.5, "rot": rot,
            "mask": {"size": chunk}}


def dense(ff=72):
    return {"kind": "dense", "ff": ff}


def moe(experts=5, top=2, ff=40, limit=0.9, shared=56, shared_limit=1.4):
    return {"kind": "moe", "router": {"experts": experts, "top": top}, "expert": {"ff": ff, "limit": limit},
            "shared": None if shared is None else {"ff": shared, "limit": shared_limit}}


def config(layers, vocab=150, width=64, eps=1e-5, embedding_scale=5.0):
    """layers: (attention, feed-forward or None), or the number of the layer whose weights are used."""
    listed = []
    for l in layers:
        owner = l
        while isinstance(owner, int):
            owner = layers[owner]
        entry = {"type": "attention", "mixer": owner[0], "mlp": owner[1]}
        if isinstance(l, int):
            entry["weights_of"] = l
        listed.append(entry)
    return {"architecture": "Bonatar", "vocab": vocab, "width": width, "norm": {"eps": eps},
            "embedding": {"scale": embedding_scale}, "layers": listed}


def weights(cfg, seed):
    """name -> float32 array whose values are BF16 numbers (tables: int32)."""
    rng = np.random.default_rng(seed)
    W, V, t = cfg["width"], cfg["vocab"], {}

    def mat(name, rows, cols, gain=1.0):
        t[name] = rng.standard_normal((rows, cols)) * (gain / np.sqrt(cols))

    def norm(name):
        t[name] = rng.uniform(-0.4, 0.4, W)

    def expert(name, ff):
        mat(name + "gate", ff, W)
        mat(name + "up", ff, W)
        mat(name + "down", W, ff, 1.5)
    t["embed"] = rng.standard_normal((V, W)) * 0.2
    mat("head", V, W)
    norm("final.norm")
    for i, l in enumerate(cfg["layers"]):
        if l.get("weights_of") is not None:
            continue
        p, m, f = "l%d." % i, l["mixer"], l["mlp"]
        norm(p + "norm1")
        mat(p + "mix.q", m["heads"] * m["dim"], W, 1.3)
        mat(p + "mix.k", m["kv_heads"] * m["dim"], W, 1.3)
        mat(p + "mix.v", m["kv_heads"] * m["vdim"], W)
        mat(p + "mix.g", m["heads"], W)
        mat(p + "mix.o", W, m["heads"] * m["vdim"], 1.5)
        if f is None:
            continue
        norm(p + "norm2")
        if f["kind"] == "dense":
            mat(p + "mlp.up", f["ff"], W)
            mat(p + "mlp.down", W, f["ff"])
            continue
        E, K = f["router"]["experts"], f["router"]["top"]
        for e in range(E):
            expert(p + "mlp.e%d." % e, f["expert"]["ff"])
        t[p + "mlp.table"] = np.stack([rng.permutation(E)[:K] for _ in range(V)]).astype(np.int32)
        if f["shared"] is not None:
            expert(p + "mlp.shared.", f["shared"]["ff"])
    return {k: v if v.dtype == np.int32 else rounded(v) for k, v in t.items()}
