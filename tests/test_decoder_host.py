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
                  "qm_chunk_attention": decoder.ChunkAttention, "qm_decay_attention": decoder.DecayAttention, "qm_general_delta": decoder.GeneralDelta}
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
    assert decoder.architectures() == ["Vabevik"]
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


def test_layer_runs_of_a_loop():
    assert plain.layer_runs(cases.CONFIGS["looped"]) == [(0, None, False)] + [(1, 0, True), (2, 0, False), (1, 1, True), (2, 1, False),
                                                                               (1, 2, True), (2, 2, False)] + [(3, None, False)]
    assert [r[0] for r in plain.layer_runs(cases.CONFIGS["plain"])] == [0, 1, 2]


@pytest.mark.parametrize("name", sorted(cases.CONFIGS))
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
