"""Prefill and decode throughput of the decoders whose layers are listed in config.json (Girirax, Bonatar) at sizes that
resemble real layers (random weights), beside the gpt_lm decoder of the same width, depth, vocabulary and batch.

    python bench.py --girirax                 every size, Girirax and gpt_lm, one JSON line
    python bench.py --bonatar                 every size, Bonatar and gpt_lm
    python bench.py --bonatar --size 2048     one size
    python bench.py --bonatar --size 2048 --model bonatar --prefill-only     for kernel traces (one untimed pass, one timed)
    python bench.py --bonatar --size 2048 --model bonatar --decode-steps 8   few steps, for kernel traces

Girirax: half of the layers are state-space recurrences, half latent attention; the projections of a layer hold about as
many weights as those of the gpt_lm layer.  Bonatar: four query heads share keys and values; half of the layers have a
square-relu feed-forward with as many weights as gpt_lm's, half a shared expert and two routed ones that together are as
large for a token; the routed experts that a token does not use come on top.  Prefill: packed prompts of mixed lengths.
Decode: greedy resident session over caches of 1024 .. 4095 tokens that a real prefill built, positions held, graph
replays.
"""
import json
import time

import numpy as np

#        width: layers, feed-forward, vocabulary, gpt heads x size, recurrence, latent attention, decode batch; Bonatar:
#        key/value heads, chunk, number of experts
SIZES = {
    1024: dict(layers=12, ff=2816, vocab=32768, heads=8, head_dim=128, batch=64, kv_heads=2, chunk=8192, experts=16,
               ssm=dict(heads=32, vdim=64, state=128, groups=1, norm_groups=1, conv=4),
               latent=dict(heads=8, dim=128, rot_dim=64, vdim=128, q_rank=512, kv_rank=256)),
    2048: dict(layers=24, ff=5632, vocab=32768, heads=16, head_dim=128, batch=16, kv_heads=4, chunk=2048, experts=16,
               ssm=dict(heads=64, vdim=64, state=128, groups=1, norm_groups=1, conv=4),
               latent=dict(heads=16, dim=128, rot_dim=64, vdim=128, q_rank=768, kv_rank=512)),
    4096: dict(layers=8, ff=11264, vocab=32768, heads=32, head_dim=128, batch=32, kv_heads=8, chunk=8192, experts=8,
               ssm=dict(heads=128, vdim=64, state=128, groups=8, norm_groups=8, conv=4),
               latent=dict(heads=32, dim=128, rot_dim=64, vdim=128, q_rank=1536, kv_rank=512)),
}
T = 4096


def girirax_config(width):
    s = SIZES[width]
    mixers = [("mamba2", s["ssm"]),
              ("latent_attention", dict(s["latent"], scale=(s["latent"]["dim"] + s["latent"]["rot_dim"]) ** -0.5,
                                        rot={"base": 10000.0, "dims": s["latent"]["rot_dim"]}))]
    return {"architecture": "Girirax", "vocab": s["vocab"], "width": width, "norm": {"eps": 1e-5}, "residual_mult": 0.5,
            "embedding": {"scale": 8.0},
            "layers": [{"type": t, "mixer": m, "mlp": {"kind": "dense", "ff": s["ff"]}}
                       for t, m in (mixers[i % 2] for i in range(s["layers"]))]}


def bonatar_config(width):
    s = SIZES[width]
    D = s["head_dim"]
    mixer = {"heads": s["heads"], "kv_heads": s["kv_heads"], "dim": D, "vdim": D, "scale": D ** -0.5,
             "mask": {"size": s["chunk"]},
             "rot": {"base": 500000.0, "dims": D, "scaling": {"factor": 8.0, "original": 8192, "fast": 32.0, "slow": 1.0}}}
    mlps = [{"kind": "dense", "ff": s["ff"] * 3 // 2},
            {"kind": "moe", "router": {"experts": s["experts"], "top": 2}, "expert": {"ff": s["ff"] // 4, "limit": 7.0},
             "shared": {"ff": s["ff"] // 2, "limit": 7.0}}]
    return {"architecture": "Bonatar", "vocab": s["vocab"], "width": width, "norm": {"eps": 1e-5}, "embedding": {"scale": 8.0},
            "layers": [{"type": "attention", "mixer": mixer, "mlp": mlps[i % 2]} for i in range(s["layers"])]}


CONFIGS = {"girirax": girirax_config, "bonatar": bonatar_config}


def _prompts(which, batch):
    rng = np.random.default_rng(which)
    lens = rng.integers(64, 2049, batch) if which == 4 else rng.integers(1024, 4096, batch)
    return lens, np.concatenate([[0], np.cumsum(lens)]).astype(np.int32)


def _open(D, model, width, batch, step_tokens):
    s = SIZES[width]
    if model in CONFIGS:
        m = D.Model(config_json=json.dumps(CONFIGS[model](width)), seed=7)
        try:
            return m.decoder(max_seq=T, batch=batch, max_step_tokens=step_tokens)
        finally:
            m.close()
    cfg = D.gpt_config(s["vocab"], width, s["layers"], s["heads"], s["head_dim"], s["ff"], T, batch, window=0,
                       tie_lm_head=True, seed=7)
    return D.GptDecoder(cfg, max_prefill_tokens=step_tokens)


def _weights(model, width):
    """weights of the layers that a token's pass multiplies with (the LM head apart)"""
    s = SIZES[width]
    mlp = 3 * width * s["ff"]
    if model == "gpt_lm":
        return s["layers"] * (4 * width * width + mlp)
    if model == "bonatar":
        qkvo = 2 * s["heads"] * s["head_dim"] + 2 * s["kv_heads"] * s["head_dim"] + s["heads"]
        return s["layers"] * (width * qkvo + mlp)
    m, a = s["ssm"], s["latent"]
    inner = m["heads"] * m["vdim"]
    ssm = width * (3 * inner + 2 * m["groups"] * m["state"] + m["heads"])
    lat = width * (a["q_rank"] + a["kv_rank"] + a["rot_dim"] + 2 * a["heads"] * a["vdim"]) + \
        a["q_rank"] * a["heads"] * (a["dim"] + a["rot_dim"]) + a["kv_rank"] * a["heads"] * (a["dim"] + a["vdim"])
    return s["layers"] // 2 * (ssm + lat + 2 * mlp)


def _prefill(D, model, width):
    lens, cu = _prompts(4, 32)
    n = int(cu[-1])
    d = _open(D, model, width, 32, n)
    ids = np.random.default_rng(5).integers(0, SIZES[width]["vocab"], n).astype(np.int32)
    d.prefill(ids, cu, want_logits=False)
    t0 = time.perf_counter()
    d.prefill(ids, cu, want_logits=False)
    s = time.perf_counter() - t0
    d.close()
    return {"prompts": 32, "tokens": n, "ms": round(s * 1e3, 2), "tokens_per_s": round(n / s, 1),
            "projection_tflops": round(2.0 * n * _weights(model, width) / s / 1e12, 1)}


def _decode(D, model, width, steps):
    batch = SIZES[width]["batch"]
    lens, cu = _prompts(3, batch)
    n = int(cu[-1])
    d = _open(D, model, width, batch, n)
    ids = np.random.default_rng(6).integers(0, SIZES[width]["vocab"], n).astype(np.int32)
    _, first, _ = d.prefill(ids, cu, want_logits=False)
    warm = min(20, steps)
    d.resident_begin(first, warm + 3 * steps + 1, hold_positions=True)
    d.resident_run(warm)
    d.resident_sync()
    times = []
    for _ in range(3):
        t0 = time.perf_counter()
        d.resident_run(steps)
        d.resident_sync()
        times.append(time.perf_counter() - t0)
    d.resident_end()
    d.close()
    s = sorted(times)[1] / steps
    return {"batch": batch, "cached_tokens": n, "steps": steps, "ms_per_step": round(s * 1e3, 4),
            "tokens_per_s": round(batch / s, 1)}


def run(pkg, architecture, size=None, model=None, prefill_only=False, decode_only=False, steps=100):
    from . import decoder as D
    out = {}
    for width in ([size] if size else sorted(SIZES)):
        for m in ([model] if model else [architecture, "gpt_lm"]):
            r = {"layer_weights": _weights(m, width)}
            if not decode_only:
                r["prefill"] = _prefill(D, m, width)
            if not prefill_only:
                r["decode"] = _decode(D, m, width, steps)
            out.setdefault("width %d, %d layers" % (width, SIZES[width]["layers"]), {})[m] = r
    print(json.dumps({architecture: out, "dtype": {architecture: "bf16", "gpt_lm": "f16"}, "data": "synthetic",
                      "weights": "random"}))
