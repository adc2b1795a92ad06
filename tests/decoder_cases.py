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
}


def weights(cfg, seed=0, sharp=3.0):
    """Random weights; queries and keys of the attention scaled so that single keys stand out (`sharp`)."""
    rng = np.random.default_rng(seed)
    out = {}

    def linear(name, n, k, gain=1.0):
        out[name] = bf16(rng.standard_normal((n, k)) * gain * k ** -0.5)

    def vector(name, n, mean=1.0, std=0.2):
        out[name] = bf16(mean + std * rng.standard_normal(n))

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
