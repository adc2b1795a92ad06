"""Plain, slow implementation of the decoder language models (numpy, float64): one function per mechanism, whole
sequences only, nothing cached and nothing shared with the product.

`forward(config, weights, tokens)` gives the logits of every position; `config` is the dictionary of a model's
config.json and `weights` maps tensor names to arrays.
"""
import numpy as np

F = np.float64


def silu(z):
    return z * sigmoid(z)


def sigmoid(z):
    e = np.exp(-np.abs(z))
    return np.where(z >= 0, 1.0 / (1.0 + e), e / (1.0 + e))


def rms_norm(x, w, eps):
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps) * w


def rotate(x, first_position, dims, base):
    """x [tokens][heads][dim]: channels i and i + dims/2 of the first `dims` turn by position * base^(-2i/dims)."""
    half = dims // 2
    if half == 0:
        return x.copy()
    p = first_position + np.arange(x.shape[0], dtype=F)
    angle = p[:, None] * np.power(F(base), -2.0 * np.arange(half, dtype=F) / dims)[None, :]
    c, s = np.cos(angle)[:, None, :], np.sin(angle)[:, None, :]
    u, v = x[..., :half], x[..., half:dims]
    return np.concatenate([u * c - v * s, v * c + u * s, x[..., dims:]], axis=-1)


def chunk_visible(n, size):
    """[query][key]: the keys of the query's own block of `size` positions, up to itself."""
    i = np.arange(n)
    return (i[None, :] <= i[:, None]) & (i[None, :] // size == i[:, None] // size)


def softmax_attention(q, k, v, scale, visible):
    """q [n][H][d], k [n][G][d], v [n][G][e] -> [n][H][e]; query head h reads key/value head h // (H / G)."""
    n, heads, _ = q.shape
    group = heads // k.shape[1]
    out = np.zeros((n, heads, v.shape[2]), F)
    for h in range(heads):
        score = (q[:, h] @ k[:, h // group].T) * scale
        score = np.where(visible, score, -np.inf)
        p = np.exp(score - score.max(axis=1, keepdims=True))
        out[:, h] = (p / p.sum(axis=1, keepdims=True)) @ v[:, h // group]
    return out


def decayed_linear_attention(q, k, v, decay):
    """S <- decay_h S + k v^T; o = S^T q.  q, k [n][H][d], v [n][H][e] -> ([n][H][e], final state [H][d][e])."""
    n, heads, d = q.shape
    state = np.zeros((heads, d, v.shape[2]), F)
    out = np.zeros((n, heads, v.shape[2]), F)
    for t in range(n):
        for h in range(heads):
            state[h] = decay[h] * state[h] + np.outer(k[t, h], v[t, h])
            out[t, h] = state[h].T @ q[t, h]
    return out, state


def generalized_delta(r, w, k, v, a, unit_eps=1e-6):
    """u = k / |k|; S <- diag(w) S - (a u)(u^T S) + k v^T with the old S in both terms; o = S^T r.  All [n][H][d]."""
    n, heads, d = r.shape
    state = np.zeros((heads, d, d), F)
    out = np.zeros((n, heads, d), F)
    for t in range(n):
        for h in range(heads):
            u = k[t, h] / np.sqrt(np.sum(k[t, h] ** 2) + unit_eps)
            old = state[h]
            state[h] = w[t, h][:, None] * old - np.outer(a[t, h] * u, u @ old) + np.outer(k[t, h], v[t, h])
            out[t, h] = state[h].T @ r[t, h]
    return out, state


def delta_decay(h, w1, w2, w0):
    return np.exp(-np.exp(-0.5) * sigmoid(np.tanh(h @ w1.T) @ w2.T + w0))


def mix_parallel(h, spec, weight, eps):
    n = h.shape[0]
    left, right = spec["left"], spec["right"]

    def heads(x, count):
        return x.reshape(n, count, -1)

    rot = left["rot"]
    q = rotate(heads(h @ weight("left.q").T, left["heads"]), 0, rot["dims"], rot["base"])
    k = rotate(heads(h @ weight("left.k").T, left["kv_heads"]), 0, rot["dims"], rot["base"])
    v = heads(h @ weight("left.v").T, left["kv_heads"])
    o = softmax_attention(q, k, v, left["scale"], chunk_visible(n, left["mask"]["size"]))
    a = o.reshape(n, -1) @ weight("left.o").T

    q = heads(silu(h @ weight("right.q").T), right["heads"])
    k = heads(silu(h @ weight("right.k").T), right["heads"])
    v = heads(silu(h @ weight("right.v").T), right["heads"])
    o, _ = decayed_linear_attention(q, k, v, right["decay"])
    o = rms_norm(o.reshape(n, -1), weight("right.norm"), eps) * sigmoid(h @ weight("right.g").T)
    b = o @ weight("right.o").T
    return 0.5 * (rms_norm(a, weight("left.out"), eps) + rms_norm(b, weight("right.out"), eps))


def mix_general_delta(h, spec, weight, eps):
    n = h.shape[0]

    def heads(x):
        return x.reshape(n, spec["heads"], spec["dim"])

    w = delta_decay(h, weight("w1"), weight("w2"), weight("w0"))
    a = sigmoid(h @ weight("a").T + weight("a.b"))
    o, _ = generalized_delta(heads(h @ weight("r").T), heads(w), heads(h @ weight("k").T), heads(h @ weight("v").T), heads(a))
    o = rms_norm(o, 1.0, eps).reshape(n, -1) * weight("norm") * sigmoid(h @ weight("g").T)
    return o @ weight("o").T


def gated_mlp(h, gate, up, down):
    return (silu(h @ gate.T) * (h @ up.T)) @ down.T


def layer_runs(config):
    """(layer, pass of the loop or None, whether it opens that pass) in the order in which they run."""
    loop = config.get("loop")
    count = len(config["layers"])
    if not loop:
        return [(i, None, False) for i in range(count)]
    runs = [(i, None, False) for i in range(loop["start"])]
    for t in range(loop["times"]):
        runs += [(i, t, i == loop["start"]) for i in range(loop["start"], loop["stop"])]
    return runs + [(i, None, False) for i in range(loop["stop"], count)]


def rotate_neighbours(x, first_position, frequencies, magnitude=1.0):
    """x [tokens][heads][dim]: channels 2i and 2i + 1 turn by position * frequencies[i], times `magnitude`."""
    n = 2 * len(frequencies)
    p = first_position + np.arange(x.shape[0], dtype=F)
    angle = (p[:, None] * np.asarray(frequencies, F)[None, :])[:, None, :]
    c, s = np.cos(angle) * magnitude, np.sin(angle) * magnitude
    out = x.copy()
    u, v = x[..., 0:n:2], x[..., 1:n:2]
    out[..., 0:n:2], out[..., 1:n:2] = u * c - v * s, v * c + u * s
    return out


def yarn(dims, base, scaling):
    """(frequencies, magnitude): slow pairs are stretched by `factor`, fast ones stay, a ramp between."""
    f = np.power(F(base), -2.0 * np.arange(dims // 2, dtype=F) / dims)
    if scaling is None:
        return f, 1.0

    def pair_that_turns(times):
        return dims * np.log(scaling["original"] / (2 * np.pi * times)) / (2 * np.log(base))

    lo = max(np.floor(pair_that_turns(scaling["fast"])), 0)
    hi = min(np.ceil(pair_that_turns(scaling["slow"])), dims - 1)
    ramp = np.clip((np.arange(dims // 2) - lo) / max(hi - lo, 0.001), 0, 1)
    return f / scaling["factor"] * ramp + f * (1 - ramp), 0.1 * np.log(scaling["factor"]) + 1


def retention(q, k, v, decay, rot):
    """q, k [n][H][d] turned in halves, k scaled by d^(-1/2), then linear attention with a decay per head."""
    dims, base = (rot["dims"], rot["base"]) if rot else (0, 1.0)
    q, k = rotate(q, 0, dims, base), rotate(k, 0, dims, base) * q.shape[2] ** -0.5
    return decayed_linear_attention(q, k, v, decay)[0]


def mix_retention(h, spec, weight, eps, shared, index):
    n, heads = h.shape[0], spec["heads"]
    split = lambda name: (h @ weight(name).T).reshape(n, heads, -1)
    o = retention(split("q"), split("k"), split("v"), spec["decay"], spec.get("rot"))
    o = rms_norm(o, 1.0, eps).reshape(n, -1) * silu(h @ weight("g").T)
    return o @ weight("o").T


def latent_of(h, spec, down, norm, eps):
    """What a latent layer keeps of each token: the normed latent and the turned key part that all heads share."""
    kept = h @ down.T
    rank = spec["kv_rank"]
    frequencies, magnitude = yarn(spec["rot_dim"], spec["rot"]["base"], spec["rot"].get("scaling"))
    return rms_norm(kept[:, :rank], norm, eps), rotate_neighbours(kept[:, None, rank:], 0, frequencies, magnitude)[:, 0]


def latent_attention(q, latent, key_part, up_k, up_v, spec):
    """q [n][H][dim + rot_dim] as projected; each head's keys and values are made from the latent -> [n][H][vdim]."""
    n, heads, dim = q.shape[0], spec["heads"], spec["dim"]
    frequencies, magnitude = yarn(spec["rot_dim"], spec["rot"]["base"], spec["rot"].get("scaling"))
    q = np.concatenate([q[..., :dim], rotate_neighbours(q[..., dim:], 0, frequencies, magnitude)], axis=-1)
    k = (latent @ up_k.T).reshape(n, heads, dim)
    k = np.concatenate([k, np.broadcast_to(key_part[:, None, :], (n, heads, key_part.shape[1]))], axis=-1)
    v = (latent @ up_v.T).reshape(n, heads, spec["vdim"])
    return softmax_attention(q, k, v, spec["scale"], np.tril(np.ones((n, n), bool)))


def mix_latent(h, spec, weight, eps, shared, index):
    """`shared` maps a layer to what it keeps; a layer with 'kv_from' reads another's."""
    n = h.shape[0]
    source = spec.get("kv_from")
    if source is None:
        source = index
        shared[index] = latent_of(h, spec, weight("dkv"), weight("dkv.norm"), eps)
    q = rms_norm(h @ weight("dq").T, weight("dq.norm"), eps) @ weight("uq").T
    o = latent_attention(q.reshape(n, spec["heads"], -1), *shared[source], weight("uk"), weight("uv"), spec)
    return o.reshape(n, -1) @ weight("o").T


def sigmoid_experts(h, router, experts, top):
    """Each token's `top` experts of the highest sigmoid(router), weighted with it; `experts` is a list of functions."""
    score = sigmoid(h @ router.T)
    out = np.zeros((h.shape[0], experts[0](h[:1]).shape[1]), F)
    for t in range(h.shape[0]):
        for e in np.argsort(-score[t], kind="stable")[:top]:
            out[t] += score[t, e] * experts[e](h[t:t + 1])[0]
    return out


def feed_forward(h, spec, weight):
    if spec["kind"] == "dense":
        return gated_mlp(h, weight("gate"), weight("up"), weight("down"))
    experts = [lambda x, e=e: gated_mlp(x, *(weight(f"e{e}.{name}") for name in ("gate", "up", "down"))) for e in range(spec["router"]["experts"])]
    return sigmoid_experts(h, weight("router"), experts, spec["router"]["top"])


def bigram_rows(tokens, spec):
    rows = [spec["buckets"]]
    for before, token in zip(tokens[:-1], tokens[1:]):
        rows.append((int(before) * spec["mul_prev"] + int(token) * spec["mul_cur"]) % spec["buckets"])
    return np.array(rows)


def forward_tuzavik(config, weights, tokens, streams=None):
    eps, m = config["norm"]["eps"], config["residual_mult"]
    tokens = np.asarray(tokens)
    norm = lambda x, name: rms_norm(x, 1.0 + weights[name], eps)
    x = weights["embed"][tokens] + weights["bigram"][bigram_rows(tokens, config["embedding"]["bigram"])]
    shared = {}
    for index, layer in enumerate(config["layers"]):
        base = f"l{index}."
        mix = {"retention": mix_retention, "latent_attention": mix_latent}[layer["type"]]
        y = mix(norm(x, base + "norm1"), layer["mixer"], lambda name: weights[f"{base}mix.{name}"], eps, shared, index)
        x = x + m * norm(y, base + "norm1b")
        if layer["mlp"] is not None:
            y = feed_forward(norm(x, base + "norm2"), layer["mlp"], lambda name: weights[f"{base}mlp.{name}"])
            x = x + m * norm(y, base + "norm2b")
        if streams is not None:
            streams.append(x)
    return norm(x, "final.norm") @ weights["head"].T * config["logit_scale"]


MIXERS = {"parallel": mix_parallel, "general_delta": mix_general_delta}


def forward(config, weights, tokens, streams=None):
    """Logits [tokens][vocab]; `streams` (a list) receives the residual stream behind every layer run."""
    weights = {name: np.asarray(t, dtype=F) for name, t in weights.items()}
    if config["architecture"] == "Tuzavik":
        return forward_tuzavik(config, weights, tokens, streams)
    eps = config["norm"]["eps"]
    x = weights["embed"][np.asarray(tokens)]
    for index, turn, opens in layer_runs(config):
        layer = config["layers"][index]
        if opens:
            x = x + weights["loop.step"][turn]
        h = rms_norm(x, weights[f"l{index}.norm1"], eps)
        y = MIXERS[layer["type"]](h, layer["mixer"], lambda name: weights[f"l{index}.mix.{name}"], eps)
        if layer["mlp"] is not None:
            y = y + gated_mlp(h, *(weights[f"l{index}.mlp.{name}"] for name in ("gate", "up", "down")))
        x = x + y
        if streams is not None:
            streams.append(x)
    return rms_norm(x, weights["final.norm"], eps) @ weights["head"].T
