"""The decoder language models through the engine on the device: prompts, decoding, portions, sequences, generation and the
command line, against the plain implementation, on small models of several shapes."""
import importlib
import json
import os
import subprocess

import numpy as np
import pytest

import decoder_cases as cases
import decoder_oracle as plain

pytestmark = pytest.mark.gpu
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
LIMIT = {True: 3e-5, False: 6e-2}        # of the logits' spread; bf16: a planted mistake moves them by more


@pytest.fixture(scope="module")
def decoder():
    return importlib.import_module("qingming-qwen3-tts_amd.decoder")


class Model:
    def __init__(self, name, directory, count):
        self.cfg = cases.CONFIGS[name]
        self.weights = cases.weights(self.cfg)
        self.directory = str(directory)
        cases.write_model(self.directory, self.cfg, self.weights)
        self.tokens = cases.tokens_of(self.cfg, count)
        self.streams = []
        self.want = plain.forward(self.cfg, self.weights, self.tokens, self.streams)


@pytest.fixture(scope="module")
def models(tmp_path_factory):
    made = {}

    def make(name, count=170):
        if name not in made:
            made[name] = Model(name, tmp_path_factory.mktemp(name), count)
        return made[name]
    return make


def feed(engine, sequence, tokens, portions):
    """Logits of every position, the tokens fed in these portions."""
    got, at = [], 0
    for n in portions:
        got.append(engine.step(sequence, tokens[at:at + n], np.arange(n)))
        at += n
    assert at == len(tokens)
    return np.concatenate(got)


NAMES = sorted(cases.CONFIGS)


@pytest.mark.parametrize("f32", [True, False])
@pytest.mark.parametrize("name", NAMES)
def test_prompt_and_streams(decoder, models, name, f32):
    m = models(name)
    engine = decoder.Decoder(m.directory, len(m.tokens), float32=f32)
    s = engine.open()
    logits, streams = engine.step(s, m.tokens, np.arange(len(m.tokens)), streams=True)
    assert cases.error(logits, m.want) < LIMIT[f32]
    for i, want in enumerate(m.streams):
        assert cases.error(streams[i], want) < LIMIT[f32], i
    assert engine.runs == len(m.streams) == len(plain.layer_runs(m.cfg))


@pytest.mark.parametrize("f32", [True, False])
@pytest.mark.parametrize("name", NAMES)
def test_portions_decoding_and_reuse(decoder, models, name, f32):
    """One engine, its one sequence used again and again: every way of cutting gives the same logits."""
    m = models(name)
    n = len(m.tokens)
    engine = decoder.Decoder(m.directory, n, float32=f32)
    cuts = ([1] * n, [n - 40] + [1] * 40, [2] * (n // 2), [3, 1, 16, 15, 1, 1, 17, 33, 5, 64, n - 156], [n])
    for path in (0, 1, 2, 4):
        engine.set_path(path)
        for portions in cuts if path == 0 else cuts[1:4:2]:
            s = engine.open()
            got = feed(engine, s, m.tokens, portions)
            engine.close(s)
            assert cases.error(got, m.want) < LIMIT[f32], (path, portions)


@pytest.mark.parametrize("f32", [True, False])
@pytest.mark.parametrize("name", NAMES)
def test_sequences_side_by_side(decoder, models, name, f32):
    """Two sequences in turn, one of them closed and its memory used again by a third: none notices the others."""
    m = models(name)
    other = cases.tokens_of(m.cfg, len(m.tokens), seed=7)
    want_other = plain.forward(m.cfg, m.weights, other)
    engine = decoder.Decoder(m.directory, len(m.tokens), float32=f32, sequences=2)
    a, b = engine.open(), engine.open()
    with pytest.raises(decoder.DecoderError) as e:
        engine.open()
    assert e.value.code == -3
    got_a, got_b, at_a, at_b = [], [], 0, 0
    for n_a, n_b in ((40, 3), (1, 60), (1, 1), (1, 1), (1, 1), (17, 2), (1, 1)):
        got_a.append(engine.step(a, m.tokens[at_a:at_a + n_a], np.arange(n_a)))
        got_b.append(engine.step(b, other[at_b:at_b + n_b], np.arange(n_b)))
        at_a, at_b = at_a + n_a, at_b + n_b
    assert cases.error(np.concatenate(got_a), m.want[:at_a]) < LIMIT[f32]
    assert cases.error(np.concatenate(got_b), want_other[:at_b]) < LIMIT[f32]
    engine.close(b)
    c = engine.open()
    assert cases.error(feed(engine, c, m.tokens[:60], [20, 1, 1, 1, 37]), m.want[:60]) < LIMIT[f32]
    assert cases.error(engine.step(a, m.tokens[at_a:at_a + 1], [0]), m.want[at_a:at_a + 1]) < LIMIT[f32]


@pytest.mark.parametrize("f32", [True, False])
def test_passes_of_few_rows_and_small_rings(decoder, models, f32):
    """A prompt longer than a pass, in an engine whose rings are a few positions longer than the chunks."""
    for name, capacity in (("short_chunks", 100000), ("mixed", 300), ("retention", 100000)):
        m = models(name)
        for max_rows in (3, 20, 64):
            engine = decoder.Decoder(m.directory, capacity, float32=f32, max_rows=max_rows)
            assert engine.sequence_bytes < 2 ** 20
            s = engine.open()
            assert cases.error(feed(engine, s, m.tokens, [120] + [1] * 20 + [30]), m.want) < LIMIT[f32]


@pytest.mark.parametrize("name", ["short_chunks", "looped", "mixed", "latents"])
def test_long_decoding(decoder, models, name):
    m = models(name)
    tokens = cases.tokens_of(m.cfg, 420, seed=3)
    want = plain.forward(m.cfg, m.weights, tokens)
    for f32 in (True, False):
        engine = decoder.Decoder(m.directory, 420, float32=f32, max_rows=32)
        s = engine.open()
        assert cases.error(feed(engine, s, tokens, [20] + [1] * 400), want) < LIMIT[f32]


def test_wanted_places_in_any_order(decoder, models):
    m = models("plain")
    engine = decoder.Decoder(m.directory, len(m.tokens), float32=True, max_rows=50)
    want = [160, 3, 3, 99, 49, 50, 0]
    got = engine.step(engine.open(), m.tokens, want)
    assert cases.error(got, m.want[want]) < LIMIT[True]
    engine = decoder.Decoder(m.directory, len(m.tokens), float32=True)
    assert engine.step(engine.open(), m.tokens[:5]).shape == (0, m.cfg["vocab"])


def greedy(m, prompt, count):
    tokens = list(prompt)
    for _ in range(count):
        tokens.append(int(plain.forward(m.cfg, m.weights, tokens)[-1].argmax()))
    return tokens[len(prompt):]


@pytest.mark.parametrize("name", NAMES)
def test_greedy_generation(decoder, models, name):
    m = models(name)
    prompt = m.tokens[:23]
    want = greedy(m, prompt, 24)
    engine = decoder.Decoder(m.directory, 64, float32=True)
    for path in (0, 1, 2):
        engine.set_path(path)
        s = engine.open()
        assert list(engine.generate(s, prompt, 24)) == want
        engine.close(s)
    stop = want[9]
    s = engine.open()
    assert list(engine.generate(s, prompt, 24, stop_token=stop)) == want[:want.index(stop) + 1]
    engine.close(s)
    s = engine.open()                                            # a prompt of one token; a sequence that goes on
    first = engine.generate(s, prompt[:1], 3)
    assert list(first) == greedy(m, prompt[:1], 3)
    more = engine.generate(s, [first[-1]], 4)
    assert list(more) == greedy(m, list(prompt[:1]) + list(first), 4)


def test_sampled_generation_is_the_samplers(decoder, models):
    """top_k = 1 is the arg-max; a seed gives its own tokens again, all of them among the k most likely."""
    m = models("plain")
    engine = decoder.Decoder(m.directory, 80, float32=True)

    def run(**options):
        s = engine.open()
        out = list(engine.generate(s, m.tokens[:20], 30, **options))
        engine.close(s)
        return out

    assert run(top_k=1, temperature=0.7, seed=5) == run()
    a, b = run(top_k=8, temperature=1.0, seed=5), run(top_k=8, temperature=1.0, seed=6)
    assert a == run(top_k=8, temperature=1.0, seed=5) and a != b
    logits = plain.forward(m.cfg, m.weights, list(m.tokens[:20]) + a)
    for i, token in enumerate(a):
        assert token in np.argsort(-logits[19 + i])[:8]


def test_errors_leave_the_engine_usable(decoder, models):
    m = models("plain")
    engine = decoder.Decoder(m.directory, 40, float32=True)
    s = engine.open()
    for bad in (lambda: engine.step(s, []), lambda: engine.step(s, [m.cfg["vocab"]]), lambda: engine.step(s, [-1]), lambda: engine.step(s, m.tokens[:41]),
                lambda: engine.step(s, m.tokens[:4], [4]), lambda: engine.step(s + 1, m.tokens[:4]), lambda: engine.generate(s, m.tokens[:20], 22),
                lambda: engine.generate(s, m.tokens[:4], 4, top_k=300), lambda: engine.set_path(3)):
        with pytest.raises(decoder.DecoderError):
            bad()
    assert cases.error(feed(engine, s, m.tokens[:40], [39, 1]), m.want[:40]) < LIMIT[True]
    with pytest.raises(decoder.DecoderError):
        engine.step(s, [1])
    engine.close(s)
    with pytest.raises(decoder.DecoderError):
        engine.step(s, [1])


@pytest.mark.parametrize("model,name", [("plain", "l1.mix.w2"), ("mixed", "l2.mlp.e11.up"), ("mixed", "l0.mix.dkv"), ("retention", "bigram")])
@pytest.mark.parametrize("change,code", [("missing", -8), ("shape", -8), ("dtype", -8)])
def test_wrong_weights_are_refused(decoder, tmp_path, change, code, model, name):
    import torch
    from safetensors.torch import load_file, save_file
    cfg = cases.CONFIGS[model]
    cases.write_model(str(tmp_path), cfg, cases.weights(cfg))
    path = os.path.join(str(tmp_path), "model.safetensors")
    tensors = load_file(path)
    if change == "missing":
        del tensors[name]
    elif change == "shape":
        tensors[name] = tensors[name][:-1].contiguous()
    else:
        tensors[name] = tensors[name].to(torch.float32)
    save_file(tensors, path)
    with pytest.raises(decoder.DecoderError) as e:
        decoder.Decoder(str(tmp_path), 16)
    assert e.value.code == code and name in str(e.value)


def test_first_tokens_and_the_token_before(decoder, models):
    """A sequence's first token has none before it, also in memory that was used; the next step's first token has the last one's."""
    m = models("retention")
    engine = decoder.Decoder(m.directory, 64, float32=True)
    for portions in ([1, 1, 1, 1], [2, 2], [1, 3], [3, 1], [4]):
        s = engine.open()
        assert cases.error(feed(engine, s, m.tokens[:4], portions), m.want[:4]) < LIMIT[True]
        engine.generate(s, m.tokens[4:9], 3)
        engine.close(s)
    engine.set_path(2)
    s = engine.open()
    assert cases.error(feed(engine, s, m.tokens[:6], [1, 1, 3, 1]), m.want[:6]) < LIMIT[True]


@pytest.mark.parametrize("f32", [True, False])
def test_a_far_key_decides(decoder, tmp_path, f32):
    """Latent attention whose query looks for one token: its only occurrence is hundreds of positions back, at a pass's edge or in the
    middle, and the logits tell it from a sequence without it."""
    cfg = cases.sandwich(48, 96, [cases.latent(4, 24, 8, 32, 40, 64, cases.dense(64))], (13, 3, 1), residual_mult=2.0)
    w = cases.weights(cfg, seed=3)
    # token 7's latent stands out: a direction of its own through dkv and up_k, which every query carries through dq and up_q
    rng = np.random.default_rng(4)
    mark, mark_c, mark_q = (cases.bf16(v / np.linalg.norm(v)) for v in (rng.standard_normal(96), rng.standard_normal(64), rng.standard_normal(40)))
    w["embed"][7] = cases.bf16(60 * mark)
    w["l0.mix.dkv"][:64] = cases.bf16(0.3 * w["l0.mix.dkv"][:64] + 2.0 * np.outer(mark_c, mark))
    head = cases.bf16(np.ones(24) * 0.4)
    for h in range(4):
        w["l0.mix.uk"][24 * h:24 * h + 24] = cases.bf16(0.1 * w["l0.mix.uk"][24 * h:24 * h + 24] + 4.0 * np.outer(head, mark_c))
        w["l0.mix.uq"][32 * h:32 * h + 24] = cases.bf16(0.1 * w["l0.mix.uq"][32 * h:32 * h + 24] + 6.0 * np.outer(head, mark_q))
    cases.write_model(str(tmp_path), cfg, w)
    tokens = cases.tokens_of(cfg, 700, seed=2)
    tokens[tokens == 7] = 8
    for at in (0, 63, 64, 65, 127, 300, 511, 639):
        marked = tokens.copy()
        marked[at] = 7
        want = plain.forward(cfg, w, marked)
        if at == 0:
            # (half of the queries look for the mark, the others away from it)
            moved = np.abs(want - plain.forward(cfg, w, tokens)).max(axis=1)[650:] / np.abs(want).max()
            assert np.quantile(moved, 0.75) > 0.1
        engine = decoder.Decoder(str(tmp_path), 700, float32=f32)
        for portions in ([660] + [1] * 40, [at + 1, 699 - at], [64, 2, 62, 572]):
            s = engine.open()
            got = feed(engine, s, marked, portions)
            engine.close(s)
            assert cases.error(got[640:], want[640:]) < LIMIT[f32], (at, portions)


def test_trace_replay_program(models, tmp_path):
    m = models("looped")
    lines, at = [], {"a": 0, "b": 0}
    wanted = []
    for step, (name, n, want) in enumerate([("a", 60, [0, 59]), ("a", 1, [0]), ("a", 2, []), ("b", 30, [29]), ("b", 1, [0]), ("a", 25, [3, 24])]):
        tokens = m.tokens[at[name]:at[name] + n]
        end = ["a", "b"] if step == 5 else []
        lines.append(json.dumps({"step": step, "entries": [{"id": name, "tokens": [int(t) for t in tokens], "want": want}], "end": end}))
        wanted.append([at[name] + w for w in want])
        at[name] += n
    p = subprocess.run([os.path.join(ROOT, "bin", "trace_run"), "--model", m.directory, "--dtype", "float32", "--out", str(tmp_path), "--max-tokens", "200"],
                       input="\n".join(lines) + "\n", capture_output=True, text=True, timeout=100)
    assert p.returncode == 0, p.stderr
    assert [line for line in p.stdout.splitlines() if line.startswith("done")] == [f"done {i}" for i in range(6)]
    for step, places in enumerate(wanted):
        path = os.path.join(str(tmp_path), f"{step}.f32")
        assert os.path.exists(path) == bool(places)
        if places:
            got = np.fromfile(path, "<f4").reshape(len(places), -1)
            assert cases.error(got, m.want[places]) < LIMIT[True]


def test_generate_program(decoder, models):
    m = models("plain")
    prompts = [[int(t) for t in m.tokens[:9]], [int(t) for t in m.tokens[5:30]]]
    p = subprocess.run([os.path.join(ROOT, "bin", "generate"), "--model", m.directory, "--dtype", "float32", "--max-new", "6"],
                       input="\n".join(map(json.dumps, prompts)) + "\n", capture_output=True, text=True, timeout=100)
    assert p.returncode == 0, p.stderr
    assert [json.loads(line) for line in p.stdout.splitlines()] == [greedy(m, prompt, 6) for prompt in prompts]
