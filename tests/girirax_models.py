"""Small Girirax configurations with seeded random weights for the tests, and the folder a decoder is opened from."""
import json
import os
import struct

import numpy as np


def _bf16(a):
    u = np.ascontiguousarray(a, np.float32).view(np.uint32)
    return ((u + 0x7FFF + ((u >> 16) & 1)) >> 16).astype(np.uint16)


def rounded(a):
    """The nearest BF16 values, as float32."""
    return (_bf16(a).astype(np.uint32) << 16).view(np.float32).reshape(np.shape(a))


def mamba(heads=4, vdim=16, state=16, groups=2, norm_groups=2, conv=4):
    return {"type": "mamba2", "mixer": {"heads": heads, "vdim": vdim, "state": state, "groups": groups,
                                        "norm_groups": norm_groups, "conv": conv}}


def latent(heads=4, dim=24, rot_dim=8, vdim=16, q_rank=40, kv_rank=48, scale=None, base=10000.0):
    return {"type": "latent_attention",
            "mixer": {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "q_rank": q_rank,
                      "kv_rank": kv_rank, "scale": scale or (dim + rot_dim) ** -0.5,
                      "rot": {"base": base, "dims": rot_dim}}}


def config(layers, vocab=192, width=64, ff=96, eps=1e-6, residual_mult=0.8, embedding_scale=3.0):
    """layers: mixers from mamba() / latent(), or (mixer, ff) with ff None for no feed-forward."""
    listed = []
    for l in layers:
        mixer, size = l if isinstance(l, tuple) else (l, ff)
        listed.append(dict(mixer, mlp=None if size is None else {"kind": "dense", "ff": size}))
    return {"architecture": "Girirax", "vocab": vocab, "width": width, "norm": {"eps": eps},
            "residual_mult": residual_mult, "embedding": {"scale": embedding_scale}, "layers": listed}


def weights(cfg, seed):
    """name -> float32 array whose values are BF16 numbers."""
    rng = np.random.default_rng(seed)
    W, t = cfg["width"], {}

    def mat(name, rows, cols):
        t[name] = rng.standard_normal((rows, cols)) / np.sqrt(cols)

    def vec(name, n, lo, hi):
        t[name] = rng.uniform(lo, hi, n)
    t["embed"] = rng.standard_normal((cfg["vocab"], W)) * 0.3
    vec("final.norm", W, 0.5, 1.5)
    for i, l in enumerate(cfg["layers"]):
        p, m = "l%d." % i, l["mixer"]
        vec(p + "norm1", W, 0.5, 1.5)
        if l["type"] == "mamba2":
            inner, ch = m["heads"] * m["vdim"], m["heads"] * m["vdim"] + 2 * m["groups"] * m["state"]
            mat(p + "mix.in", inner + ch + m["heads"], W)
            t[p + "mix.conv"] = rng.standard_normal((ch, m["conv"])) * 0.6
            vec(p + "mix.conv.b", ch, -0.2, 0.2)
            vec(p + "mix.dt_bias", m["heads"], -4, -1)
            vec(p + "mix.A_log", m["heads"], -1, 1.5)
            vec(p + "mix.D", m["heads"], 0.5, 1.5)
            vec(p + "mix.norm", inner, 0.5, 1.5)
            mat(p + "mix.o", W, inner)
        else:
            H = m["heads"]
            mat(p + "mix.dq", m["q_rank"], W)
            vec(p + "mix.dq.norm", m["q_rank"], 0.5, 1.5)
            mat(p + "mix.uq", H * (m["dim"] + m["rot_dim"]), m["q_rank"])
            mat(p + "mix.dkv", m["kv_rank"] + m["rot_dim"], W)
            vec(p + "mix.dkv.norm", m["kv_rank"], 0.5, 1.5)
            mat(p + "mix.uk", H * m["dim"], m["kv_rank"])
            mat(p + "mix.uv", H * m["vdim"], m["kv_rank"])
            mat(p + "mix.g", H * m["vdim"], W)
            mat(p + "mix.o", W, H * m["vdim"])
        if l["mlp"] is not None:
            F = l["mlp"]["ff"]
            for part, rows, cols in (("gate", F, W), ("up", F, W), ("down", W, F)):
                mat(p + "mlp." + part, rows, cols)
                vec(p + "mlp." + part + ".b", rows, -0.2, 0.2)
            vec(p + "norm2", W, 0.5, 1.5)
    return {k: rounded(v) for k, v in t.items()}


def save(folder, cfg, tensors):
    """config.json and model.safetensors (BF16; integer arrays as I32)."""
    os.makedirs(folder, exist_ok=True)
    with open(os.path.join(folder, "config.json"), "w") as f:
        json.dump(cfg, f)
    header, blob = {}, b""
    for name, a in tensors.items():
        whole = np.issubdtype(np.asarray(a).dtype, np.integer)
        raw = np.ascontiguousarray(a, np.int32).tobytes() if whole else _bf16(a).tobytes()
        header[name] = {"dtype": "I32" if whole else "BF16", "shape": list(a.shape),
                        "data_offsets": [len(blob), len(blob) + len(raw)]}
        blob += raw
    text = json.dumps(header).encode()
    with open(os.path.join(folder, "model.safetensors"), "wb") as f:
        f.write(struct.pack("<Q", len(text)) + text + blob)
    return folder
