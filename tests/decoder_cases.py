"""Small decoder language models for the tests: configurations, random weights (bf16 values), model directories."""
import json
import os

import numpy as np


def bf16(x):
    """x rounded to the nearest bf16 value, as float32."""
    bits = np.ascontiguousarray(x, dtype=np.float32).view(np.uint32).astype(np.uint64)
    return (((bits + 0x7fff + ((bits >> 16) & 1)) >> 16) << 16).astype(np.uint32).view(np.float32)


def left(heads, kv_heads, dim, vdim, chunk, rot_dims, base=10000.0, scale=None):
    return {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "mask": {"size": chunk}, "rot": {"base": base, "dims": rot_dims},
            "scale": dim ** -0.5 if scale is None else scale}


def right(heads, dim, vdim, decay):
    assert len(decay) == heads
    return {"heads": heads, "dim": dim, "vdim": vdim, "decay": list(decay)}


def parallel(l, r, ff):
    return {"type": "parallel", "mixer": {"left": l, "right": r}, "mlp": {"kind": "dense", "ff": ff} if ff else None}


def general_delta(heads, dim, ff):
    return {"type": "general_delta", "mixer": {"heads": heads, "dim": dim}, "mlp": {"kind": "dense", "ff": ff} if ff else None}


def config(vocab, width, layers, loop=None, eps=1e-5):
    c = {"architecture": "Vabevik", "vocab": vocab, "width": width, "norm": {"eps": eps}, "layers": layers}
    if loop:
        c["loop"] = {"start": loop[0], "stop": loop[1], "times": loop[2]}
    return c


def retention(heads, dim, vdim, decay, mlp, rot_dims=None, base=10000.0):
    assert len(decay) == heads
    rot = {"base": base, "dims": dim if rot_dims is None else rot_dims}
    return {"type": "retention", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "decay": list(decay), "rot": rot}, "mlp": mlp}


def latent(heads, dim, rot_dim, vdim, q_rank, kv_rank, mlp, scaling=None, kv_from=None, base=10000.0, scale=None):
    mixer = {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "q_rank": q_rank, "kv_rank": kv_rank,
             "scale": (dim + rot_dim) ** -0.5 if scale is None else scale, "rot": {"base": base, "dims": rot_dim}}
    if scaling:
        mixer["rot"]["scaling"] = dict(zip(("factor", "original", "fast", "slow"), scaling))
    if kv_from is not None:
        mixer["kv_from"] = kv_from
    return {"type": "latent_attention", "mixer": mixer, "mlp": mlp}


def dense(ff):
    return {"kind": "dense", "ff": ff}


def moe(experts, top, ff):
    return {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top}}


def sandwich(vocab, width, layers, bigram, eps=1e-5, residual_mult=1.0, logit_scale=1.0):
    return {"architecture": "Tuzavik", "vocab": vocab, "width": width, "norm": {"eps": eps}, "layers": layers, "residual_mult": residual_mult,
            "logit_scale": logit_scale, "embedding": {"bigram": dict(zip(("buckets", "mul_prev", "mul_cur"), bigram))}}


CONFIGS = {
    # no loop, no feed-forward in one layer, one query head per key/value head, values wider than keys, a decay of one
    "plain": config(77, 96, [parallel(left(3, 3, 24, 40, 37, 8), right(2, 20, 36, [0.9, 1.0]), 72), general_delta(3, 20, 0),
                             parallel(left(4, 2, 16, 16, 64, 16), right(1, 48, 16, [0.5]), 40)]),
    # widths that are no multiple of anything, five query heads per key/value head, a loop that runs three times
    "looped": config(130, 150, [general_delta(2, 36, 90), parallel(left(5, 1, 36, 20, 50, 10), right(3, 12, 70, [0.7, 0.99, 0.0]), 61),
                                general_delta(1, 72, 33), parallel(left(6, 2, 32, 64, 21, 0), right(2, 64, 32, [0.95, 0.8]), 130)],
                     loop=(1, 3, 3), eps=3e-4),
    # heads above 128 channels, a delta head above 64, a loop over everything, run once, chunks longer than any prompt
    "wide": config(300, 264, [parallel(left(2, 1, 136, 144, 5000, 64, base=300.0), right(2, 132, 200, [0.999, 0.6]), 256), general_delta(2, 160, 200)],
                   loop=(0, 2, 1)),
    # chunks of a few positions
    "short_chunks": config(64, 64, [parallel(left(4, 2, 16, 24, 5, 4, scale=0.4), right(4, 16, 16, [0.3, 0.9, 0.97, 1.0]), 96),
                                    parallel(left(8, 2, 8, 8, 12, 8), right(1, 8, 24, [0.99]), 64)]),
    # retention alone: one head and several, values wider and narrower than keys, few or no rotated channels, decays of 0 and 1, a layer
    # without feed-forward, a prime number of buckets and factors above it
    "retention": sandwich(90, 100, [retention(1, 24, 40, [0.97], dense(70)), retention(3, 36, 20, [1.0, 0.5, 0.99], None, rot_dims=10, base=300.0),
                                    retention(2, 130, 70, [0.999, 0.2], moe(3, 1, 50), rot_dims=0)], (101, 1009, 777777), eps=3e-4, residual_mult=0.4),
    # latents shared by several layers, two of them kept, frequencies stretched and not, every expert chosen, sizes that are no multiples
    "latents": sandwich(120, 150, [latent(3, 20, 10, 28, 44, 36, dense(90), scaling=(4.0, 64, 8.0, 1.0), base=500.0),
                                   latent(5, 12, 6, 20, 24, 72, moe(5, 5, 36), scale=0.3),
                                   latent(2, 33, 10, 17, 20, 36, None, scaling=(4.0, 64, 8.0, 1.0), base=500.0, kv_from=0),
                                   latent(4, 16, 6, 24, 30, 72, dense(40), kv_from=1)], (64, 3, 5), residual_mult=0.9, logit_scale=0.3),
    # heads above 128 channels, latents above 256, many experts
    "wide_latents": sandwich(200, 264, [latent(5, 110, 60, 100, 140, 300, moe(70, 6, 130), scaling=(16.0, 100, 32.0, 2.0)), retention(2, 64, 200, [0.9, 0.98], dense(256)),
                                        latent(17, 24, 60, 140, 60, 300, dense(200), scaling=(16.0, 100, 32.0, 2.0), kv_from=0)], (37, 0, 1), logit_scale=2.0),
    # a latent and a key part beyond what the matrix cores take
    "long_latents": sandwich(64, 96, [latent(2, 24, 80, 40, 32, 560, dense(64)), latent(3, 16, 80, 16, 16, 560, moe(9, 2, 72), kv_from=0)], (11, 6, 7),
                             residual_mult=0.8),
    # both mixers, both feed-forwards
    "mixed": sandwich(160, 160, [latent(4, 16, 8, 24, 48, 40, moe(6, 2, 48)), retention(4, 16, 24, [0.9, 0.99, 0.999, 0.8], dense(128)),
                                 latent(6, 24, 8, 8, 32, 40, moe(12, 3, 64), kv_from=0)], (211, 29, 53), residual_mult=0.6, logit_scale=0.7),
}
PARALLEL = sorted(name for name, c in CONFIGS.items() if c["architecture"] == "Vabevik")
SANDWICH = sorted(name for name, c in CONFIGS.items() if c["architecture"] == "Tuzavik")


def weights(cfg, seed=0, sharp=3.0):
    """Random weights; queries and keys of the attention scaled so that single keys stand out (`sharp`)."""
    rng = np.random.default_rng(seed)
    out = {}

    def linear(name, n, k, gain=1.0):
        out[name] = bf16(rng.standard_normal((n, k)) * gain * k ** -0.5)

    def vector(name, n, mean=1.0, std=0.2):
        out[name] = bf16(mean + std * rng.standard_normal(n))

    if cfg["architecture"] == "Tuzavik":
        sandwich_weights(cfg, rng, sharp, out, linear, vector)
        return out
    width = cfg["width"]
    out["embed"] = bf16(rng.standard_normal((cfg["vocab"], width)))
    linear("head", cfg["vocab"], width)
    vector("final.norm", width)
    if cfg.get("loop"):
        out["loop.step"] = bf16(0.5 * rng.standard_normal((cfg["loop"]["times"], width)))
    for i, layer in enumerate(cfg["layers"]):
        base, m = f"l{i}.", layer["mixer"]
        vector(base + "norm1", width)
        if layer["type"] == "parallel":
            l, r = m["left"], m["right"]
            linear(base + "mix.left.q", l["heads"] * l["dim"], width, sharp)
            linear(base + "mix.left.k", l["kv_heads"] * l["dim"], width, sharp)
            linear(base + "mix.left.v", l["kv_heads"] * l["vdim"], width)
            linear(base + "mix.left.o", width, l["heads"] * l["vdim"])
            vector(base + "mix.left.out", width)
            for name, n in (("q", r["heads"] * r["dim"]), ("k", r["heads"] * r["dim"]), ("v", r["heads"] * r["vdim"]), ("g", r["heads"] * r["vdim"])):
                linear(base + "mix.right." + name, n, width)
            linear(base + "mix.right.o", width, r["heads"] * r["vdim"])
            vector(base + "mix.right.norm", r["heads"] * r["vdim"])
            vector(base + "mix.right.out", width)
        else:
            every = m["heads"] * m["dim"]
            for name in ("r", "k", "v", "a", "g"):
                linear(base + "mix." + name, every, width)
            rank = 8 + 5 * i
            linear(base + "mix.w1", rank, width)
            linear(base + "mix.w2", every, rank, 2.0)
            vector(base + "mix.w0", every, -2.0, 2.0)          # decays from slow to fast
            vector(base + "mix.a.b", every, 0.0, 1.0)
            vector(base + "mix.norm", every)
            linear(base + "mix.o", width, every)
        if layer["mlp"]:
            ff = layer["mlp"]["ff"]
            linear(base + "mlp.gate", ff, width)
            linear(base + "mlp.up", ff, width)
            linear(base + "mlp.down", width, ff)
    return out


CODE = 8                                                   # channels of the stream that the routers read


def sandwich_weights(cfg, rng, sharp, out, linear, vector):
    """Tuzavik's.  The last CODE channels of the stream hold a code of the token that no layer adds to, and routers read only
    them: an expert's rank never rests on rounding, whatever the rest of the stream does."""
    width, vocab = cfg["width"], cfg["vocab"]
    out["embed"] = bf16(rng.standard_normal((vocab, width)))
    out["bigram"] = bf16(rng.standard_normal((cfg["embedding"]["bigram"]["buckets"] + 1, width)))
    out["bigram"][:, -CODE:] = 0
    linear("head", vocab, width)
    vector("final.norm", width, 0.0)
    routers = {}
    for i, layer in enumerate(cfg["layers"]):
        base, m, mlp = f"l{i}.", layer["mixer"], layer["mlp"]
        for name in ("norm1", "norm1b") + (("norm2", "norm2b") if mlp else ()):
            vector(base + name, width, 0.0)
            if name.endswith("b"):
                out[base + name][-CODE:] = -1
        if layer["type"] == "retention":
            for name, n in (("q", m["heads"] * m["dim"]), ("k", m["heads"] * m["dim"]), ("v", m["heads"] * m["vdim"]), ("g", m["heads"] * m["vdim"])):
                linear(base + "mix." + name, n, width)
            linear(base + "mix.o", width, m["heads"] * m["vdim"])
        else:
            linear(base + "mix.dq", m["q_rank"], width)
            vector(base + "mix.dq.norm", m["q_rank"])
            linear(base + "mix.uq", m["heads"] * (m["dim"] + m["rot_dim"]), m["q_rank"], sharp)
            if "kv_from" not in m:
                linear(base + "mix.dkv", m["kv_rank"] + m["rot_dim"], width)
                vector(base + "mix.dkv.norm", m["kv_rank"])
            linear(base + "mix.uk", m["heads"] * m["dim"], m["kv_rank"])
            linear(base + "mix.uv", m["heads"] * m["vdim"], m["kv_rank"])
            linear(base + "mix.o", width, m["heads"] * m["vdim"])
        if mlp is None:
            continue
        for part in [""] if mlp["kind"] == "dense" else [f"e{e}." for e in range(mlp["router"]["experts"])]:
            ff = mlp["ff"] if mlp["kind"] == "dense" else mlp["expert"]["ff"]
            linear(base + "mlp." + part + "gate", ff, width)
            linear(base + "mlp." + part + "up", ff, width)
            linear(base + "mlp." + part + "down", width, ff)
        if mlp["kind"] == "moe":
            router = np.zeros((mlp["router"]["experts"], width), np.float32)
            router[:, -CODE:] = rng.standard_normal((len(router), CODE))
            out[base + "mlp.router"] = bf16(router)
            routers[base] = (bf16(router), mlp["router"]["top"])
    for token in range(vocab):
        while True:
            code = bf16(rng.standard_normal(CODE))
            out["embed"][token, -CODE:] = code
            gaps = [1.0]
            for base, (router, top) in routers.items():
                z = np.sort(router[:, -CODE:] @ ((1 + out[base + "norm2"][-CODE:]) * code))[::-1]
                if top < len(z):
                    gaps.append((z[top - 1] - z[top]) / np.abs(z).max())
            if min(gaps) > 0.05:
                break


def write_model(directory, cfg, tensors):
    import torch
    from safetensors.torch import save_file
    with open(os.path.join(directory, "config.json"), "w") as f:
        json.dump(cfg, f)
    save_file({name: torch.from_numpy(t.copy()).to(torch.bfloat16) for name, t in tensors.items()}, os.path.join(directory, "model.safetensors"))


def tokens_of(cfg, count, seed=1):
    return np.random.default_rng(seed).integers(0, cfg["vocab"], count).astype(np.int32)


def error(got, want):
    """Largest row error: rms of the difference over the rms of the wanted rows, means taken off."""
    got, want = np.asarray(got, np.float64), np.asarray(want, np.float64)
    d = got - want
    d -= d.mean(axis=-1, keepdims=True)
    scale = np.sqrt(np.mean((want - want.mean(axis=-1, keepdims=True)) ** 2))
    return float(np.sqrt(np.mean(d * d, axis=-1)).max() / scale)
