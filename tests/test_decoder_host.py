"""CPU checks of the decoder language models: exports and structures of the C ABI, config.json reading, argument validation
without a device, and the plain implementation's mechanisms against closed forms."""
import copy
import ctypes as C
import importlib
import json
import os
import re
import subprocess

import numpy as np
import pytest

import decoder_cases as cases
import decoder_oracle as plain

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))


@pytest.fixture(scope="module")
def decoder():
    return importlib.import_module("qingming-qwen3-tts_amd.decoder")


def test_header_symbols_are_exported(decoder):
    text = re.sub(r"/\*.*?\*/", "", open(os.path.join(ROOT, "include", "qm_decoder.h")).read(), flags=re.S)
    names = sorted(set(re.findall(r"\b(qm_[a-z0-9_]+)\s*\(", text)))
    for name in names:
        assert hasattr(decoder.lib(), name), name
    assert sorted(decoder.EXPORTS) == names


def test_structures_have_the_headers_layout(decoder, tmp_path):
    structures = {"qm_residual_term": decoder.ResidualTerm, "qm_residual_norm": decoder.ResidualNorm, "qm_gated_norm": decoder.GatedNorm,
                  "qm_decoder_linear": decoder.DecoderLinear, "qm_attention_partials": decoder.AttentionPartials,
                  "qm_chunk_attention": decoder.ChunkAttention, "qm_decay_attention": decoder.DecayAttention, "qm_general_delta": decoder.GeneralDelta,
                  "qm_latent_rows": decoder.LatentRows, "qm_latent_attention": decoder.LatentAttention, "qm_experts": decoder.Experts}
    lines = [f'printf("{c} %zu\\n", sizeof({c}));' for c in structures]
    fields = [(c, name) for c, s in structures.items() for name, _ in s._fields_]
    lines += [f'printf("{c}.{name} %zu\\n", offsetof({c}, {name}));' for c, name in fields]
    source = os.path.join(str(tmp_path), "layout.c")
    with open(source, "w") as f:
        f.write('#include <stddef.h>\n#include <stdio.h>\n#include "qm_decoder.h"\nint main(void) {\n' + "\n".join(lines) + "\nreturn 0; }\n")
    program = os.path.join(str(tmp_path), "layout")
    subprocess.run(["gcc", "-I", os.path.join(ROOT, "include"), source, "-o", program], check=True)
    got = dict(line.split() for line in subprocess.run([program], check=True, capture_output=True, text=True).stdout.splitlines())
    for c, s in structures.items():
        assert int(got[c]) == C.sizeof(s), c
    for c, name in fields:
        assert int(got[f"{c}.{name}"]) == getattr(structures[c], name).offset, (c, name)


def test_registry_and_configurations(decoder, tmp_path):
    assert decoder.architectures() == ["Vabevik", "Tuzavik"]
    path = os.path.join(str(tmp_path), "config.json")

    def check(cfg):
        with open(path, "w") as f:
            f.write(cfg if isinstance(cfg, str) else json.dumps(cfg))
        decoder.check_config(path)

    for cfg in cases.CONFIGS.values():
        check(cfg)
    base = cases.CONFIGS["looped"]
    no_loop = copy.deepcopy(base)
    no_loop["loop"] = None
    check(no_loop)

    def broken(change):
        cfg = copy.deepcopy(base)
        change(cfg)
        with pytest.raises(decoder.DecoderError) as e:
            check(cfg)
        assert e.value.code == -7

    broken(lambda c: c.update(architecture="SomethingElse"))
    broken(lambda c: c.pop("architecture"))
    broken(lambda c: c.pop("norm"))
    broken(lambda c: c.update(layers=[]))
    broken(lambda c: c.update(width=0))
    broken(lambda c: c.update(vocab=2.5))
    broken(lambda c: c["loop"].update(stop=9))
    broken(lambda c: c["loop"].update(times=0))
    broken(lambda c: c["layers"][0].update(type="other"))
    broken(lambda c: c["layers"][0]["mlp"].update(kind="other"))
    broken(lambda c: c["layers"][1]["mixer"]["left"].update(kv_heads=2))
    broken(lambda c: c["layers"][1]["mixer"]["left"]["rot"].update(dims=7))
    broken(lambda c: c["layers"][1]["mixer"]["left"]["rot"].update(dims=64))
    broken(lambda c: c["layers"][1]["mixer"]["left"].pop("mask"))
    broken(lambda c: c["layers"][1]["mixer"]["right"].update(decay=[0.5]))
    base = cases.CONFIGS["mixed"]
    unscaled = copy.deepcopy(base)
    unscaled["layers"][0]["mixer"]["rot"]["scaling"] = None
    check(unscaled)
    no_rotation = copy.deepcopy(base)
    no_rotation["layers"][1]["mixer"]["rot"] = None
    check(no_rotation)
    broken(lambda c: c.pop("embedding"))
    broken(lambda c: c["embedding"]["bigram"].update(buckets=0))
    broken(lambda c: c["embedding"]["bigram"].update(mul_cur=1.5))
    broken(lambda c: c.pop("residual_mult"))
    broken(lambda c: c.pop("logit_scale"))
    broken(lambda c: c["layers"][0].update(type="parallel"))
    broken(lambda c: c["layers"][0]["mixer"].pop("scale"))
    broken(lambda c: c["layers"][0]["mixer"]["rot"].update(dims=6))
    broken(lambda c: c["layers"][0]["mixer"].update(rot_dim=7))
    broken(lambda c: c["layers"][0]["mixer"]["rot"].update(scaling={"factor": 2.0}))
    broken(lambda c: c["layers"][2]["mixer"].update(kv_from=1))       # not a latent layer
    broken(lambda c: c["layers"][2]["mixer"].update(kv_from=2))       # not an earlier one
    broken(lambda c: c["layers"][2]["mixer"].update(kv_rank=48))
    broken(lambda c: c["layers"][2]["mixer"]["rot"].update(base=3.0))
    broken(lambda c: c["layers"][1]["mixer"].update(decay=[0.5]))
    broken(lambda c: c["layers"][1]["mixer"]["rot"].update(dims=18))
    broken(lambda c: c["layers"][0]["mlp"]["router"].update(top=7))
    broken(lambda c: c["layers"][0]["mlp"].update(kind="other"))
    with pytest.raises(decoder.DecoderError):
        check("{")
    with pytest.raises(decoder.DecoderError):
        decoder.check_config(os.path.join(str(tmp_path), "missing.json"))


def test_operators_check_their_arguments(decoder):
    lib = decoder.lib()
    null = -1
    assert lib.qm_residual_norm_rows(None, 1, 0, None) == null
    p = C.create_string_buffer(64)
    at = C.addressof(p)
    op = decoder.ResidualNorm(x_in=at, norm_w=at, h=at, ld_h=64, width=64)
    assert lib.qm_residual_norm_rows(C.byref(op), 0, 0, None) == 0                 # nothing to do, nothing launched
    assert lib.qm_residual_norm_rows(C.byref(op), -1, 0, None) < 0
    op.width = 65
    assert lib.qm_residual_norm_rows(C.byref(op), 0, 0, None) < 0
    linear = decoder.DecoderLinear(x=at, w=at, out32=at, ldx=128, ldo=128, n=128, k=128)
    assert lib.qm_decoder_linear_rows(C.byref(linear), 1, 0, 0, None) == 0
    for field, bad in (("n", 100), ("k", 64), ("ldx", 127), ("ldo", 64), ("x", None), ("out32", None)):
        other = decoder.DecoderLinear(x=at, w=at, out32=at, ldx=128, ldo=128, n=128, k=128)
        setattr(other, field, bad)
        assert lib.qm_decoder_linear_rows(C.byref(other), 1, 0, 0, None) < 0, field
    assert lib.qm_decoder_linear_rows(C.byref(linear), 4, 0, 0, None) < 0
    attention = dict(proj=at, frequency=at, q_rot=at, k_cache=at, v_cache=at, out=at,
                     part=decoder.AttentionPartials(at, at, 4, 16, 1, 128), ld_proj=256, ld_out=128, position=0, rows=0, heads=4, kv_heads=2, dim=16,
                     vdim=16, k_stride=16, v_stride=16, ring=100, chunk=50, rot_dims=8)
    assert lib.qm_chunk_attention_rows(C.byref(decoder.ChunkAttention(**attention)), 0, None) == 0
    for change in (dict(kv_heads=3), dict(k_stride=20), dict(rot_dims=18), dict(rot_dims=7), dict(chunk=0), dict(dim=300), dict(ring=0), dict(ld_out=60),
                   dict(chunk=200), dict(position=-1), dict(proj=None), dict(frequency=None)):
        assert lib.qm_chunk_attention_rows(C.byref(decoder.ChunkAttention(**{**attention, **change})), 0, None) < 0, change
    decay = dict(proj=at, powers=at, state=at, out=at, ld_proj=100, rows=0, heads=2, dim=16, vdim=16)
    assert lib.qm_decay_attention_rows(C.byref(decoder.DecayAttention(**decay)), None) == 0
    for change in (dict(dim=257), dict(vdim=0), dict(heads=0), dict(rows=-1), dict(state=None)):
        assert lib.qm_decay_attention_rows(C.byref(decoder.DecayAttention(**{**decay, **change})), None) < 0, change
    delta = dict(proj=at, w2=at, w0=at, a_bias=at, state=at, out=at, ld_proj=100, rows=0, heads=2, dim=16, rank=4)
    assert lib.qm_general_delta_rows(C.byref(decoder.GeneralDelta(**delta)), None) == 0
    for change in (dict(dim=257), dict(rank=0), dict(heads=0), dict(rows=-1), dict(w2=None)):
        assert lib.qm_general_delta_rows(C.byref(decoder.GeneralDelta(**{**delta, **change})), None) < 0, change
    for change in (dict(rot_dims=18), dict(rot_dims=3, frequency=at), dict(rot_dims=8), dict(position=-1)):
        assert lib.qm_decay_attention_rows(C.byref(decoder.DecayAttention(**{**decay, "options": decoder.DECAY_ROTARY, **change})), None) < 0, change
    rows = dict(proj=at, q_norm=at, kv_norm=at, frequency=at, q_latent=at, latent_cache=at, key_cache=at, ld_proj=200, ld_q=128, ld_latent=128, rows=0,
                q_rank=40, kv_rank=72, rot_dim=16, key_stride=16)
    assert lib.qm_latent_rows_norm(C.byref(decoder.LatentRows(**rows)), 0, None) == 0
    for change in (dict(kv_rank=129), dict(kv_rank=0), dict(rot_dim=15), dict(key_stride=8), dict(ld_q=30), dict(position=-1), dict(key_cache=None)):
        assert lib.qm_latent_rows_norm(C.byref(decoder.LatentRows(**{**rows, **change})), 0, None) < 0, change
    latent = dict(q=at, frequency=at, up_k=at, up_v=at, latent_cache=at, key_cache=at, out=at, q_scratch=at, ml=at, acc=at, ld_query=200, ld_latent=128,
                  ld_out=128, rows=0, heads=3, dim=40, rot_dim=16, vdim=36, kv_rank=72, key_stride=16, splits=4)
    assert lib.qm_latent_attention_rows(C.byref(decoder.LatentAttention(**latent)), 0, None) == 0
    for change in (dict(heads=0), dict(kv_rank=2000), dict(ld_latent=60), dict(ld_query=100), dict(ld_out=100), dict(splits=65), dict(splits=0),
                   dict(key_stride=8), dict(rot_dim=3), dict(position=-1), dict(acc=None)):
        assert lib.qm_latent_attention_rows(C.byref(decoder.LatentAttention(**{**latent, **change})), 0, None) < 0, change
    experts = dict(x=at, logits=at, gate=at, up=at, down=at, out32=at, scratch=at, ld_logits=8, rows=0, experts=8, top=2, width_p=128, ff_p=128)
    assert lib.qm_expert_rows(C.byref(decoder.Experts(**experts)), 0, None) == 0
    for change in (dict(top=9), dict(top=0), dict(experts=2000, ld_logits=2000), dict(ld_logits=7), dict(width_p=100), dict(ff_p=64), dict(down=None),
                   dict(rows=4)):                                                  # (rows=4: no scratch)
        assert lib.qm_expert_rows(C.byref(decoder.Experts(**{**experts, **change})), 0, None) < 0, change
    handle = C.c_void_p()
    assert lib.qm_decoder_create(None, 0, 1, 1, 0, None, C.byref(handle)) == null
    assert lib.qm_decoder_step(None, 0, None, 0, None, 0, None, None) == null


def test_loading_fails_cleanly(decoder, tmp_path):
    """Without a device nothing past the configuration is reached; what is wrong with a directory is reported before."""
    with pytest.raises(decoder.DecoderError) as e:
        decoder.Decoder(str(tmp_path), 16)
    assert e.value.code == -7 and "config.json" in str(e.value)


def test_runner_reports_a_missing_model(tmp_path):
    p = subprocess.run([os.path.join(ROOT, "bin", "trace_run"), "--model", str(tmp_path), "--dtype", "float32", "--out", str(tmp_path),
                        "--max-tokens", "8"], input="", capture_output=True, text=True)
    assert p.returncode not in (0, 3) and "config.json" in p.stderr


# ---- the plain implementation ----------------------------------------------------------------------------------------

def test_rotation_turns_pairs_by_position_times_frequency():
    x = np.zeros((3, 1, 6))
    x[:, 0, 0], x[:, 0, 4] = 1.0, 7.0
    y = plain.rotate(x, 5, 4, 100.0)                            # pairs (0, 2) and (1, 3), channel 4 and 5 pass
    for t in range(3):
        assert np.allclose(y[t, 0], [np.cos(5 + t), 0, np.sin(5 + t), 0, 7, 0])
    x = np.zeros((1, 1, 6))
    x[0, 0, 3] = 1.0
    assert np.allclose(plain.rotate(x, 2, 4, 100.0)[0, 0], [0, -np.sin(2 * 100 ** -0.5), 0, np.cos(2 * 100 ** -0.5), 0, 0])


def test_chunks_count_from_the_sequences_start():
    v = plain.chunk_visible(7, 3)
    assert [list(np.nonzero(row)[0]) for row in v] == [[0], [0, 1], [0, 1, 2], [3], [3, 4], [3, 4, 5], [6]]


def test_decayed_attention_is_a_weighted_sum():
    rng = np.random.default_rng(0)
    q, k, v = rng.standard_normal((9, 2, 3)), rng.standard_normal((9, 2, 3)), rng.standard_normal((9, 2, 4))
    decay = [0.5, 1.0]
    o, state = plain.decayed_linear_attention(q, k, v, decay)
    for h in range(2):
        for t in range(9):
            want = sum(decay[h] ** (t - j) * (q[t, h] @ k[j, h]) * v[j, h] for j in range(t + 1))
            assert np.allclose(o[t, h], want)
        assert np.allclose(state[h], sum(decay[h] ** (8 - j) * np.outer(k[j, h], v[j, h]) for j in range(9)))


def test_delta_rule_writes_and_removes():
    """With no decay, full removal and orthonormal keys a key's value is replaced; with no removal values add up."""
    k = np.eye(3)[[0, 1, 0]][:, None, :]
    v = np.arange(9.0).reshape(3, 1, 3)
    ones = np.ones((3, 1, 3))
    o, state = plain.generalized_delta(k, ones, k, v, ones, unit_eps=0.0)
    assert np.allclose(o[:, 0], [v[0, 0], v[1, 0], v[2, 0]])
    assert np.allclose(state[0], [v[2, 0], v[1, 0], [0, 0, 0]])
    o, _ = plain.generalized_delta(k, ones, k, v, 0 * ones, unit_eps=0.0)
    assert np.allclose(o[2, 0], v[0, 0] + v[2, 0])
    o, _ = plain.generalized_delta(k, 0.5 * ones, k, v, 0 * ones, unit_eps=0.0)
    assert np.allclose(o[2, 0], 0.25 * v[0, 0] + v[2, 0])


def test_neighbours_turn_together():
    x = np.zeros((3, 1, 6))
    x[:, 0, 0], x[:, 0, 5] = 1.0, 7.0
    y = plain.rotate_neighbours(x, 5, [1.0, 0.1], 2.0)
    for t in range(3):
        assert np.allclose(y[t, 0], [2 * np.cos(5 + t), 2 * np.sin(5 + t), 0, 0, 0, 7])


def test_stretched_frequencies():
    f, magnitude = plain.yarn(16, 10000.0, dict(factor=6.0, original=300, fast=20.0, slow=1.0))
    unstretched, one = plain.yarn(16, 10000.0, None)
    assert one == 1 and np.isclose(magnitude, 0.1 * np.log(6) + 1)
    # pairs that turn often keep their frequency, those that turn less than once are stretched whole
    turns = 300 * unstretched / (2 * np.pi)
    assert np.allclose(f[turns > 20], unstretched[turns > 20]) and np.allclose(f[-1], unstretched[-1] / 6)
    assert np.all(f <= unstretched + 1e-15) and np.all(f >= unstretched / 6 - 1e-15)
    f, magnitude = plain.yarn(16, 10000.0, dict(factor=1.0, original=300, fast=20.0, slow=1.0))
    assert np.allclose(f, unstretched) and magnitude == 1


def test_retention_is_a_weighted_sum_of_turned_keys():
    rng = np.random.default_rng(0)
    q, k, v = rng.standard_normal((9, 2, 4)), rng.standard_normal((9, 2, 4)), rng.standard_normal((9, 2, 3))
    decay = [0.5, 1.0]
    o = plain.retention(q, k, v, decay, {"dims": 2, "base": 50.0})
    for h in range(2):
        for t in range(9):
            want = np.zeros(3)
            for j in range(t + 1):                              # one pair of frequency 1: only the distance counts
                c, s = np.cos(t - j), np.sin(t - j)
                turned = q[t, h, 0] * (c * k[j, h, 0] + s * k[j, h, 1]) + q[t, h, 1] * (c * k[j, h, 1] - s * k[j, h, 0])
                want += decay[h] ** (t - j) * 0.5 * (turned + q[t, h, 2:] @ k[j, h, 2:]) * v[j, h]
            assert np.allclose(o[t, h], want)


def test_latent_attention_in_the_latents_space():
    """Keys and values made from latents give what queries sent through up_k and results sent through up_v give."""
    spec = dict(heads=3, dim=5, rot_dim=4, vdim=6, kv_rank=7, scale=0.4, rot={"base": 30.0, "dims": 4})
    rng = np.random.default_rng(1)
    q, c, k = rng.standard_normal((8, 3, 9)), rng.standard_normal((8, 7)), rng.standard_normal((8, 4))
    up_k, up_v = rng.standard_normal((15, 7)), rng.standard_normal((18, 7))
    o = plain.latent_attention(q, c, k, up_k, up_v, spec)
    turned = plain.rotate_neighbours(q[..., 5:], 0, plain.yarn(4, 30.0, None)[0])
    for h in range(3):
        for t in range(8):
            score = (c[:t + 1] @ (up_k[5 * h:5 * h + 5].T @ q[t, h, :5]) + k[:t + 1] @ turned[t, h]) * 0.4
            p = np.exp(score - score.max())
            assert np.allclose(o[t, h], up_v[6 * h:6 * h + 6] @ ((p / p.sum()) @ c[:t + 1]))


def test_experts_of_the_highest_scores_are_weighted_with_them():
    h = np.array([[1.0, -2.0], [0.5, 3.0]])
    router = np.array([[1.0, 0.0], [0.0, 1.0], [-1.0, 0.0]])
    experts = [lambda x, e=e: np.full((1, 2), float(10 ** e)) for e in range(3)]
    s = plain.sigmoid(h @ router.T)
    out = plain.sigmoid_experts(h, router, experts, 2)
    assert np.allclose(out[0], s[0, 0] * 1 + s[0, 2] * 100) and np.allclose(out[1], s[1, 1] * 10 + s[1, 0] * 1)


def test_bigram_rows():
    assert list(plain.bigram_rows([4, 9, 2], dict(buckets=7, mul_prev=3, mul_cur=5))) == [7, (12 + 45) % 7, (27 + 10) % 7]


def test_layer_runs_of_a_loop():
    assert plain.layer_runs(cases.CONFIGS["looped"]) == [(0, None, False)] + [(1, 0, True), (2, 0, False), (1, 1, True), (2, 1, False),
                                                                               (1, 2, True), (2, 2, False)] + [(3, None, False)]
    assert [r[0] for r in plain.layer_runs(cases.CONFIGS["plain"])] == [0, 1, 2]


@pytest.mark.parametrize("name", cases.SANDWICH)
def test_plain_model_sees_a_planted_mistake_in_a_sandwich_layer(name):
    """Each mechanism of the tests' models moves the logits by far more than the product's tolerance when it is wrong."""
    cfg, w = cases.CONFIGS[name], cases.weights(cases.CONFIGS[name])
    tokens = cases.tokens_of(cfg, 90)
    want = plain.forward(cfg, w, tokens)

    def moved(change):
        c = copy.deepcopy(cfg)
        change(c)
        return cases.error(plain.forward(c, w, tokens), want)

    def every(kind, change):
        def apply(c):
            for layer in c["layers"]:
                if layer["type"] == kind:
                    change(layer["mixer"])
        return apply

    kinds = {layer["type"] for layer in cfg["layers"]}
    assert moved(lambda c: c.update(residual_mult=c["residual_mult"] * 1.2)) > 0.05
    assert moved(lambda c: c["embedding"]["bigram"].update(mul_cur=c["embedding"]["bigram"]["mul_cur"] + 1)) > 0.2
    if "retention" in kinds:
        assert moved(every("retention", lambda m: m.update(decay=[d * 0.97 for d in m["decay"]]))) > 0.004
        assert moved(every("retention", lambda m: m["rot"].update(base=m["rot"]["base"] * 2))) > 0.02
    if "latent_attention" in kinds:
        assert moved(every("latent_attention", lambda m: m.update(scale=m["scale"] * 1.1))) > 0.01
        assert moved(every("latent_attention", lambda m: m["rot"].update(base=m["rot"]["base"] * 2))) > 0.02
        if any("scaling" in layer["mixer"]["rot"] for layer in cfg["layers"]):
            assert moved(every("latent_attention", lambda m: m["rot"].pop("scaling", None))) > 0.05
    if any(layer["mlp"] and layer["mlp"]["kind"] == "moe" and layer["mlp"]["router"]["top"] > 1 for layer in cfg["layers"]):
        def fewer(c):
            for layer in c["layers"]:
                if layer["mlp"] and layer["mlp"]["kind"] == "moe":
                    layer["mlp"]["router"]["top"] -= 1
        assert moved(fewer) > 0.05


@pytest.mark.parametrize("name", cases.PARALLEL)
def test_plain_model_sees_a_planted_mistake(name):
    """The tests' weights make faults visible: a chunk that is one longer, a lost state, a missing loop vector, a key/value head
    taken for another all move some logits by far more than the product's tolerance."""
    cfg = cases.CONFIGS[name]
    w = cases.weights(cfg)
    tokens = cases.tokens_of(cfg, 90)
    want = plain.forward(cfg, w, tokens)

    def moved(change_cfg=None, change_weights=None):
        c, v = copy.deepcopy(cfg), dict(w)
        if change_cfg:
            change_cfg(c)
        if change_weights:
            change_weights(v)
        return cases.error(plain.forward(c, v, tokens), want)

    def longer(c):
        for layer in c["layers"]:
            if layer["type"] == "parallel":
                layer["mixer"]["left"]["mask"]["size"] += 1

    def forget(c):
        for layer in c["layers"]:
            if layer["type"] == "parallel":
                layer["mixer"]["right"]["decay"] = [d * 0.98 for d in layer["mixer"]["right"]["decay"]]

    if min(l["mixer"]["left"]["mask"]["size"] for l in cfg["layers"] if l["type"] == "parallel") < 90:
        assert moved(longer) > 0.1
    assert moved(forget) > 0.004
    if cfg.get("loop"):
        assert moved(None, lambda v: v.update({"loop.step": 0 * v["loop.step"]})) > 0.1
    for i, layer in enumerate(cfg["layers"]):
        if layer["type"] == "parallel" and layer["mixer"]["left"]["kv_heads"] > 1:
            key = f"l{i}.mix.left.k"
            assert moved(None, lambda v: v.update({key: np.roll(v[key], layer["mixer"]["left"]["dim"], axis=0)})) > 0.05
