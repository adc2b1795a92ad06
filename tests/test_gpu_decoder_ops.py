"""The decoder language models' operators on the device, each mechanism alone, against the plain implementation."""
import ctypes as C
import importlib

import numpy as np
import pytest

import decoder_cases as cases
import decoder_oracle as plain

pytestmark = pytest.mark.gpu


@pytest.fixture(scope="module")
def decoder():
    return importlib.import_module("qingming-qwen3-tts_amd.decoder")


def put(a, dev, dtype=None):
    import torch
    return torch.from_numpy(np.ascontiguousarray(a)).to(dev) if dtype is None else torch.from_numpy(np.ascontiguousarray(a)).to(dtype).to(dev)


def get(t):
    import torch
    torch.cuda.synchronize()
    return t.float().cpu().numpy()


def activation(f32):
    import torch
    return torch.float32 if f32 else torch.bfloat16


def close(got, want, f32, tol32=2e-6, tol16=4e-3):
    scale = np.abs(want).max() + 1e-30
    worst = np.abs(got.astype(np.float64) - want).max() / scale
    assert worst <= (tol32 if f32 else tol16), worst


@pytest.mark.parametrize("f32", [True, False])
@pytest.mark.parametrize("width,ld,rows", [(96, 128, 3), (264, 384, 2), (1500, 1536, 2), (2048, 2048, 4), (4000, 4096, 2), (9000, 9088, 2)])
def test_residual_norm(decoder, dev, f32, width, ld, rows):
    import torch
    rng = np.random.default_rng(width)

    def padded(n):
        out = np.zeros((n, ld), np.float32)
        out[:, :width] = rng.standard_normal((n, width))
        return out

    x, y, step, norms = padded(7), [padded(7) for _ in range(3)], padded(1)[0], padded(3)
    embed = cases.bf16(padded(11))
    tokens = rng.integers(0, 11, 7).astype(np.int32)
    row_map = rng.permutation(7)[:rows].astype(np.int32)
    d = {n: put(v, dev) for n, v in (("x", x), ("y0", y[0]), ("y1", y[1]), ("y2", y[2]), ("step", step), ("norms", norms), ("tokens", tokens), ("map", row_map))}
    table = put(embed, dev, torch.bfloat16)
    eps, w = 0.01, slice(0, width)

    bigram = cases.bf16(padded(6))
    d["fed"], bigrams = put(np.concatenate([[-1], tokens]).astype(np.int32), dev), put(bigram, dev, torch.bfloat16)      # (no token before row 0's)

    def terms(src):
        return (0.5 * plain.rms_norm(y[0][src, w], norms[0, w], eps) - 0.25 * plain.rms_norm(y[1][src, w], norms[1, w], eps) + y[2][src, w])

    for mapped, embedded, count, stepped, pairs in ((False, False, 3, True, False), (True, False, 3, False, False), (True, True, 0, True, False),
                                                    (False, True, 2, False, False), (False, True, 0, False, True), (True, True, 2, False, True)):
        src = row_map if mapped else np.arange(rows)
        want = (embed[tokens[src]][:, w] if embedded else x[src, w]).astype(np.float64)
        if pairs:
            rows_of = [5 if i == 0 else (3 * int(tokens[i - 1]) + 4 * int(tokens[i])) % 5 for i in src]
            want = want + bigram[rows_of][:, w]
        if count == 3:
            want = want + terms(src)
        elif count == 2:
            want = want + 0.5 * plain.rms_norm(y[0][src, w], norms[0, w], eps) + y[2][src, w]
        if stepped:
            want = want + step[w]
        x_out = torch.full((rows, ld), 7.0, device=dev)
        h = torch.full((rows, ld), 7.0, device=dev, dtype=activation(f32))
        op = decoder.ResidualNorm(x_in=None if embedded else d["x"].data_ptr(), embed=table.data_ptr(), tokens=d["tokens"].data_ptr(),
                                  row_map=d["map"].data_ptr() if mapped else None, step_vec=d["step"].data_ptr() if stepped else None,
                                  norm_w=d["norms"].data_ptr() + 8 * ld, x_out=x_out.data_ptr(), h=h.data_ptr(), ld_h=ld, width=width, vocab=11,
                                  terms=count, eps=eps)
        if pairs:
            op.tokens, op.bigram = d["fed"].data_ptr() + 4, bigrams.data_ptr()
            op.buckets, op.mul_prev, op.mul_cur = 5, 3, 4
        chosen = [("y0", 0, 0.5), ("y1", 1, -0.25), ("y2", None, 1.0)] if count == 3 else [("y0", 0, 0.5), ("y2", None, 1.0)][:count]
        for i, (name, norm, scale) in enumerate(chosen):
            op.term[i] = decoder.ResidualTerm(d[name].data_ptr(), None if norm is None else d["norms"].data_ptr() + 4 * norm * ld, ld, scale, 0)
        assert decoder.lib().qm_residual_norm_rows(C.byref(op), rows, int(f32), torch.cuda.current_stream().cuda_stream) == 0
        got_x, got_h = get(x_out), get(h)
        close(got_x[:, w], want, True)
        close(got_h[:, w], plain.rms_norm(want, norms[2, w], eps), f32)
        assert np.all(got_x[:, width:] == 0) and np.all(got_h[:, width:] == 0)


@pytest.mark.parametrize("f32", [True, False])
@pytest.mark.parametrize("groups,size,ld", [(1, 96, 128), (1, 2048, 2048), (1, 5000, 5120), (1, 70, 128), (3, 20, 128), (16, 128, 2048), (2, 160, 384), (1, 1, 128)])
@pytest.mark.parametrize("silu", [0, 1])
def test_gated_norm(decoder, dev, f32, groups, size, ld, silu):
    import torch
    rng = np.random.default_rng(size)
    n, rows = groups * size, 3
    o, gate, weight = rng.standard_normal((rows, n)).astype(np.float32), rng.standard_normal((rows, n + 12)).astype(np.float32), rng.standard_normal(n).astype(np.float32)
    out = torch.full((rows, ld), 7.0, device=dev, dtype=activation(f32))
    d = [put(v, dev) for v in (o, weight, gate)]
    op = decoder.GatedNorm(o=d[0].data_ptr(), weight=None if silu else d[1].data_ptr(), silu=silu, gate=d[2].data_ptr(), out=out.data_ptr(), ld_o=n, ld_gate=n + 12, ld_out=ld,
                           groups=groups, size=size, eps=0.02)
    assert decoder.lib().qm_gated_norm_rows(C.byref(op), rows, int(f32), torch.cuda.current_stream().cuda_stream) == 0
    g = gate[:, :n].astype(np.float64)
    want = plain.rms_norm(o.astype(np.float64).reshape(rows, groups, size), 1.0, 0.02).reshape(rows, n) * (plain.silu(g) if silu else weight * plain.sigmoid(g))
    got = get(out)
    close(got[:, :n], want, f32)
    assert np.all(got[:, n:] == 0)


@pytest.mark.parametrize("f32", [True, False])
@pytest.mark.parametrize("n", [16, 48, 64, 80])
@pytest.mark.parametrize("rows,k,ldx,ldo", [(1, 128, 128, 128), (7, 256, 264, 132), (16, 128, 128, 128), (33, 384, 392, 140), (200, 2048, 2048, 128)])
def test_linear_of_few_columns(decoder, dev, f32, rows, k, ldx, ldo, n):
    import torch
    rng = np.random.default_rng(rows)
    x, w = cases.bf16(rng.standard_normal((rows, ldx))), cases.bf16(rng.standard_normal((n, k)) * k ** -0.5)
    xd, wd = put(x, dev, activation(f32)), put(w, dev, torch.bfloat16)
    out = torch.full((rows + 1, ldo), 7.0, device=dev)
    linear = decoder.DecoderLinear(x=xd.data_ptr(), w=wd.data_ptr(), out32=out.data_ptr(), ldx=ldx, ldo=ldo, n=n, k=k)
    assert decoder.lib().qm_decoder_linear_rows(C.byref(linear), 1, rows, int(f32), torch.cuda.current_stream().cuda_stream) == 0
    got = get(out)
    close(got[:rows, :n], x[:, :k].astype(np.float64) @ w.T, True, tol32=3e-6)
    assert np.all(got[rows:] == 7) and np.all(got[:, n:] == 7)


@pytest.mark.parametrize("f32", [True, False])
@pytest.mark.parametrize("rows", [1, 2, 3, 5, 9, 15, 16, 40, 130])
def test_linears(decoder, dev, f32, rows):
    """Three linears of their own inputs and reductions in one launch, the last a gate/up pair."""
    import torch
    rng = np.random.default_rng(rows)
    shapes = [(256, 128), (128, 896), (384, 640)]
    x = [cases.bf16(rng.standard_normal((rows, k))) for _, k in shapes]
    w = [cases.bf16(rng.standard_normal((n, k)) * k ** -0.5) for n, k in shapes]
    up = cases.bf16(rng.standard_normal(shapes[2]) * shapes[2][1] ** -0.5)
    xd = [put(v, dev, activation(f32)) for v in x]
    wd = [put(v, dev, torch.bfloat16) for v in w + [up]]
    outs = [torch.full((rows, shapes[i][0]), 7.0, device=dev, dtype=torch.float32 if i < 2 else activation(f32)) for i in range(3)]
    linears = (decoder.DecoderLinear * 3)()
    for i, (n, k) in enumerate(shapes):
        linears[i] = decoder.DecoderLinear(x=xd[i].data_ptr(), w=wd[i].data_ptr(), w_up=wd[3].data_ptr() if i == 2 else None,
                                           out32=outs[i].data_ptr() if i < 2 else None, out=outs[i].data_ptr() if i == 2 else None, ldx=k, ldo=n, n=n, k=k)
    assert decoder.lib().qm_decoder_linear_rows(linears, 3, rows, int(f32), torch.cuda.current_stream().cuda_stream) == 0
    for i in range(2):
        close(get(outs[i]), x[i].astype(np.float64) @ w[i].T, True, tol32=3e-6)
    gate = x[2].astype(np.float64) @ w[2].T
    close(get(outs[2]), plain.silu(gate) * (x[2].astype(np.float64) @ up.T), f32, tol32=3e-6, tol16=2e-2)


ATTENTION = [
    # heads, kv_heads, dim, vdim, chunk, rot_dims
    (4, 2, 16, 16, 50, 8), (3, 3, 24, 40, 37, 24), (5, 1, 36, 20, 64, 10), (6, 2, 64, 64, 200, 16), (2, 1, 136, 144, 300, 64), (8, 2, 128, 128, 256, 128),
    (4, 4, 8, 256, 33, 0), (16, 1, 32, 48, 70, 32), (7, 1, 20, 28, 5, 4),
]


class AttentionCase:
    """Projections of a sequence with a needle: at some positions one far key is made to stand out."""

    def __init__(self, shape, tokens, seed=0):
        self.heads, self.kv, self.dim, self.vdim, self.chunk, self.rot = shape
        rng = np.random.default_rng(seed)
        self.n, self.ld = tokens, self.heads * self.dim + self.kv * (self.dim + self.vdim) + 8
        self.k_at = self.heads * self.dim
        self.v_at = self.k_at + self.kv * self.dim
        self.proj = rng.standard_normal((tokens, self.ld)).astype(np.float32)
        # keys that many queries of their chunk point at: the first and the last of each chunk, one just outside for the next
        q = self.proj[:, :self.k_at].reshape(tokens, self.heads, self.dim)
        for p in range(0, tokens, self.chunk):
            for at in (p, min(p + self.chunk, tokens) - 1):
                self.proj[at, self.k_at:self.v_at] *= 6.0
        q *= 2.0
        self.base, self.scale = 500.0, self.dim ** -0.5

    def want(self, chunk=None):
        p = self.proj.astype(np.float64)
        heads = lambda a, count: a.reshape(self.n, count, -1)
        q = plain.rotate(heads(p[:, :self.k_at], self.heads), 0, self.rot, self.base)
        k = plain.rotate(heads(p[:, self.k_at:self.v_at], self.kv), 0, self.rot, self.base)
        v = heads(p[:, self.v_at:self.v_at + self.kv * self.vdim], self.kv)
        return plain.softmax_attention(q, k, v, self.scale, plain.chunk_visible(self.n, chunk or self.chunk)).reshape(self.n, -1)

    def run(self, decoder, dev, f32, portions, ring=None, rows_only=False, splits=4):
        import torch
        dtype = activation(f32)
        r8 = lambda n: (n + 7) // 8 * 8
        ks, vs, n_out = r8(self.dim), r8(self.vdim), self.heads * self.vdim
        ld_out = (n_out + 127) // 128 * 128
        ring = ring or self.n
        freq = put(self.base ** (-2.0 * np.arange(max(1, self.rot // 2)) / max(1, self.rot)), dev)
        kc = torch.full((self.kv, ring, ks), float("nan"), device=dev, dtype=dtype)
        vc = torch.full((self.kv, ring, vs), float("nan"), device=dev, dtype=dtype)
        proj = put(self.proj, dev)
        most = max(portions)
        per_split = -(-self.chunk // splits)
        ml = torch.zeros(most * self.heads * splits * 2, device=dev)
        acc = torch.zeros(most * self.heads * splits * self.vdim, device=dev)
        q_rot = torch.zeros(most * self.heads * ks, device=dev, dtype=dtype)
        got, at = [], 0
        for rows in portions:
            out = torch.full((rows, ld_out), 7.0, device=dev, dtype=dtype)
            op = decoder.ChunkAttention(proj=proj.data_ptr() + 4 * self.ld * at, frequency=freq.data_ptr(), q_rot=q_rot.data_ptr(), k_cache=kc.data_ptr(),
                                        v_cache=vc.data_ptr(), out=out.data_ptr(),
                                        part=decoder.AttentionPartials(ml.data_ptr(), acc.data_ptr(), self.heads, self.vdim, splits, per_split),
                                        ld_proj=self.ld, ld_out=ld_out, position=at, rows=rows, heads=self.heads, kv_heads=self.kv, dim=self.dim,
                                        vdim=self.vdim, k_stride=ks, v_stride=vs, ring=ring, chunk=self.chunk, rot_dims=self.rot, k_column=self.k_at,
                                        v_column=self.v_at, scale=self.scale, options=1 if rows_only else 0)
            assert decoder.lib().qm_chunk_attention_rows(C.byref(op), int(f32), torch.cuda.current_stream().cuda_stream) == 0
            out = get(out)
            assert np.all(out[:, n_out:] == 0)
            got.append(out[:, :n_out])
            at += rows
        return np.concatenate(got)


@pytest.mark.parametrize("shape", ATTENTION)
def test_chunk_attention(decoder, dev, shape):
    case = AttentionCase(shape, 230)
    want = case.want()
    if shape[4] < 230:       # the inputs tell a chunk from one that is a position longer or shorter
        scale = np.abs(want).max()
        assert min(np.abs(case.want(shape[4] + d) - want).max() for d in (1, -1)) > 0.1 * scale
    cuts = [230], [100, 2, 28, 1, 1, 17, 3, 16, 62], [1] * 8 + [222], [60, 15, 2, 2, 2, 2] + [1] * 60 + [87]
    for portions in cuts:
        close(case.run(decoder, dev, True, portions), want, True, tol32=2e-5)
        for rows_only in (False, True):
            close(case.run(decoder, dev, False, portions, rows_only=rows_only), want, False, tol16=3e-2)


@pytest.mark.parametrize("shape", [ATTENTION[0], ATTENTION[2], ATTENTION[8]])
def test_chunk_attention_over_a_ring(decoder, dev, shape):
    """A ring of chunk + portion - 1 positions: slots are used again while their old keys have just left the chunk."""
    case = AttentionCase(shape, 410, seed=5)
    want = case.want()
    for most in (1, 2, 20, 33):
        portions = [most] * (410 // most) + ([410 % most] if 410 % most else [])
        ring = case.chunk + most - 1
        close(case.run(decoder, dev, True, portions, ring=ring), want, True, tol32=2e-5)
        close(case.run(decoder, dev, False, portions, ring=ring), want, False, tol16=3e-2)


def test_two_attention_kernels_agree(decoder, dev):
    case = AttentionCase((8, 4, 64, 64, 512, 32), 700, seed=9)
    a, b = case.run(decoder, dev, False, [700]), case.run(decoder, dev, False, [700], rows_only=True)
    assert np.abs(a - b).max() <= 2e-2 * np.abs(b).max()


@pytest.mark.parametrize("chunked", [False, True])
@pytest.mark.parametrize("heads,dim,vdim", [(3, 16, 24), (2, 20, 36), (1, 48, 16), (4, 64, 128), (2, 132, 200), (1, 256, 256), (2, 7, 9)])
def test_decay_attention(decoder, dev, chunked, heads, dim, vdim):
    import torch
    rng = np.random.default_rng(dim)
    n = 230
    decay = np.array([0.999, 1.0, 0.3, 0.0][:heads])
    ld = heads * (2 * dim + vdim) + 12
    proj = rng.standard_normal((n, ld)).astype(np.float32)
    k_at, v_at = heads * dim + 4, 2 * heads * dim + 8
    part = lambda at, count, size: plain.silu(proj[:, at:at + count * size].astype(np.float64)).reshape(n, count, size)
    want, state = plain.decayed_linear_attention(part(0, heads, dim), part(k_at, heads, dim), part(v_at, heads, vdim), decay)
    powers = put(np.power(decay[:, None], np.arange(decoder.DECAY_POWERS)[None]).astype(np.float32), dev)
    pd = put(proj, dev)
    for portions in ([n], [100, 2, 28, 1, 17, 64, 16, 2], [1] * 20 + [65, 145]):
        s = torch.zeros((heads, dim, vdim), device=dev)
        got, at = [], 0
        for rows in portions:
            out = torch.full((rows, heads * vdim), 7.0, device=dev)
            floats = decoder.lib().qm_decay_attention_scratch_floats(rows, heads, dim, vdim)
            assert (floats > 0) == (rows >= 16)
            scratch = torch.full((max(1, floats),), float("nan"), device=dev)
            op = decoder.DecayAttention(proj=pd.data_ptr() + 4 * ld * at, powers=powers.data_ptr(), state=s.data_ptr(), out=out.data_ptr(),
                                        scratch=scratch.data_ptr() if chunked else None, ld_proj=ld, scratch_floats=floats, rows=rows, heads=heads, dim=dim,
                                        vdim=vdim, q_column=0, k_column=k_at, v_column=v_at)
            assert decoder.lib().qm_decay_attention_rows(C.byref(op), torch.cuda.current_stream().cuda_stream) == 0
            got.append(get(out))
            at += rows
        close(np.concatenate(got), want.reshape(n, -1), True, tol32=5e-6)
        close(get(s), state, True, tol32=5e-6)


@pytest.mark.parametrize("chunked", [False, True])
@pytest.mark.parametrize("heads,dim,rank", [(3, 16, 5), (2, 20, 16), (1, 48, 64), (4, 64, 8), (2, 100, 33), (2, 128, 64), (1, 160, 300), (1, 256, 24)])
def test_general_delta(decoder, dev, chunked, heads, dim, rank):
    import torch
    rng = np.random.default_rng(dim + rank)
    n, every = 170, heads * dim
    ld = 4 * every + rank + 8
    proj = rng.standard_normal((n, ld)).astype(np.float32)
    proj[50:60, every:2 * every] = proj[40:50, every:2 * every]          # keys that come back
    columns = dict(r_column=0, k_column=every, v_column=2 * every, a_column=3 * every, z_column=4 * every)
    w2 = (rng.standard_normal((rank, every)) * 2 * rank ** -0.5).astype(np.float32)
    w0, bias = (rng.standard_normal(every) * 3 - 2).astype(np.float32), rng.standard_normal(every).astype(np.float32)
    p = proj.astype(np.float64)
    part = lambda name: p[:, columns[name]:columns[name] + every].reshape(n, heads, dim)
    w = np.exp(-np.exp(-0.5) * plain.sigmoid(np.tanh(p[:, 4 * every:4 * every + rank]) @ w2 + w0)).reshape(n, heads, dim)
    a = plain.sigmoid(part("a_column") + bias.reshape(heads, dim))
    want, state = plain.generalized_delta(part("r_column"), w, part("k_column"), part("v_column"), a)
    d = [put(v, dev) for v in (proj, w2, w0, bias)]
    for portions in ([n], [70, 2, 28, 1, 16, 32, 21], [1] * 12 + [33, 125]):
        s = torch.zeros((heads, dim, dim), device=dev)
        got, at = [], 0
        for rows in portions:
            out = torch.full((rows, every), 7.0, device=dev)
            floats = decoder.lib().qm_general_delta_scratch_floats(rows, heads, dim)
            scratch = torch.full((max(1, floats),), float("nan"), device=dev)
            op = decoder.GeneralDelta(proj=d[0].data_ptr() + 4 * ld * at, w2=d[1].data_ptr(), w0=d[2].data_ptr(), a_bias=d[3].data_ptr(), state=s.data_ptr(),
                                      out=out.data_ptr(), scratch=scratch.data_ptr() if chunked else None, ld_proj=ld, scratch_floats=floats, rows=rows,
                                      heads=heads, dim=dim, rank=rank, unit_eps=1e-6, **columns)
            assert decoder.lib().qm_general_delta_rows(C.byref(op), torch.cuda.current_stream().cuda_stream) == 0
            got.append(get(out))
            at += rows
        close(np.concatenate(got), want.reshape(n, -1), True, tol32=2e-5)
        close(get(s), state, True, tol32=2e-5)


@pytest.mark.parametrize("chunked", [False, True])
@pytest.mark.parametrize("heads,dim,vdim,rot_dims", [(3, 16, 24, 16), (2, 20, 36, 6), (1, 48, 16, 0), (4, 64, 128, 64), (2, 132, 200, 130), (2, 256, 64, 256)])
def test_retention(decoder, dev, chunked, heads, dim, vdim, rot_dims):
    """The decayed attention with rotated queries and keys, scaled keys and plain values."""
    import torch
    rng = np.random.default_rng(dim)
    n, base = 230, 700.0
    decay = np.array([0.999, 1.0, 0.3, 0.0][:heads])
    ld = heads * (2 * dim + vdim) + 12
    proj = rng.standard_normal((n, ld)).astype(np.float32)
    k_at, v_at = heads * dim + 4, 2 * heads * dim + 8
    proj[3, k_at:k_at + heads * dim] *= 30.0                          # an early key that later queries see through the decay
    part = lambda at, count, size: proj[:, at:at + count * size].astype(np.float64).reshape(n, count, size)
    q, k, v = part(0, heads, dim), part(k_at, heads, dim), part(v_at, heads, vdim)
    want = plain.retention(q, k, v, decay, {"dims": rot_dims, "base": base}).reshape(n, -1)
    powers = put(np.power(decay[:, None], np.arange(decoder.DECAY_POWERS)[None]).astype(np.float32), dev)
    frequency = put(base ** (-2.0 * np.arange(max(1, rot_dims // 2)) / max(1, rot_dims)), dev)
    for portions in ([n], [100, 2, 28, 1, 17, 64, 16, 2], [1] * 20 + [65, 145]):
        pd = put(proj, dev)                                           # (rotated in place)
        s = torch.zeros((heads, dim, vdim), device=dev)
        got, at = [], 0
        for rows in portions:
            out = torch.full((rows, heads * vdim), 7.0, device=dev)
            floats = decoder.lib().qm_decay_attention_scratch_floats(rows, heads, dim, vdim)
            scratch = torch.full((max(1, floats),), float("nan"), device=dev)
            where = torch.tensor([at], dtype=torch.int32, device=dev)
            op = decoder.DecayAttention(proj=pd.data_ptr() + 4 * ld * at, powers=powers.data_ptr(), state=s.data_ptr(), out=out.data_ptr(),
                                        scratch=scratch.data_ptr() if chunked else None, frequency=frequency.data_ptr(), ld_proj=ld, scratch_floats=floats,
                                        rows=rows, heads=heads, dim=dim, vdim=vdim, q_column=0, k_column=k_at, v_column=v_at, options=decoder.DECAY_ROTARY,
                                        rot_dims=rot_dims, position=at, k_scale=dim ** -0.5)
            if rows == 1:
                op.position, op.position_dev = 0, where.data_ptr()
            assert decoder.lib().qm_decay_attention_rows(C.byref(op), torch.cuda.current_stream().cuda_stream) == 0
            got.append(get(out))
            at += rows
        close(np.concatenate(got), want, True, tol32=5e-6)


LATENT = [
    # heads, dim, rot_dim, vdim, kv_rank, scaling
    (3, 16, 8, 24, 40, None), (7, 48, 12, 40, 64, (3.0, 100, 20.0, 1.5)), (5, 20, 6, 28, 100, None), (16, 64, 32, 64, 256, None), (17, 128, 64, 128, 512, None),
    (1, 33, 10, 17, 300, (4.0, 50, 8.0, 0.5)), (2, 40, 64, 72, 128, None), (2, 200, 80, 24, 560, None), (2, 16, 70, 300, 96, None), (40, 8, 2, 8, 24, None),
]


class LatentCase:
    """Projections of a sequence; some latents stand out so that single keys far away, at the edges of passes and tiles, decide."""

    def __init__(self, shape, tokens, seed=0):
        self.heads, self.dim, self.rot, self.vdim, self.rank, scaling = shape
        rng = np.random.default_rng(seed)
        self.n, self.base = tokens, 900.0
        self.scaling = dict(zip(("factor", "original", "fast", "slow"), scaling)) if scaling else None
        self.per_head = self.dim + self.rot
        self.proj = rng.standard_normal((tokens, 20 + self.rank + self.rot + 8)).astype(np.float32)          # 20 columns of a query latent
        self.kv_at = 20 + 4
        self.q = (2.0 * rng.standard_normal((tokens, self.heads * self.per_head + 4))).astype(np.float32)
        self.kv_norm = (1 + 0.2 * rng.standard_normal(self.rank)).astype(np.float32)
        self.q_norm = (1 + 0.2 * rng.standard_normal(20)).astype(np.float32)
        for at in (0, 1, 63, 64, 127, 128, tokens - 40):
            self.proj[at, self.kv_at + self.rank:self.kv_at + self.rank + self.rot] *= 4.0                   # (the latent itself is normed)
        self.up_k = cases.bf16(rng.standard_normal((self.heads * self.dim, self.rank)) * self.rank ** -0.5)
        self.up_v = cases.bf16(rng.standard_normal((self.heads * self.vdim, self.rank)) * self.rank ** -0.5)
        self.scale, self.eps = self.per_head ** -0.5, 0.01
        self.spec = {"heads": self.heads, "dim": self.dim, "rot_dim": self.rot, "vdim": self.vdim, "kv_rank": self.rank, "scale": self.scale,
                     "rot": {"base": self.base, "dims": self.rot, "scaling": self.scaling}}

    def kept(self):
        p = self.proj[:, self.kv_at:self.kv_at + self.rank + self.rot].astype(np.float64)
        return plain.latent_of(p, self.spec, np.eye(self.rank + self.rot), self.kv_norm.astype(np.float64), self.eps)

    def want(self):
        q = self.q[:, :self.heads * self.per_head].astype(np.float64).reshape(self.n, self.heads, self.per_head)
        return plain.latent_attention(q, *self.kept(), self.up_k.astype(np.float64), self.up_v.astype(np.float64), self.spec).reshape(self.n, -1)

    def run(self, decoder, dev, f32, portions, rows_only=False, splits=5):
        import torch
        lib, dtype = decoder.lib(), activation(f32)
        stream = torch.cuda.current_stream().cuda_stream
        up128 = lambda n: (n + 127) // 128 * 128
        ld, key_stride, n_out = up128(self.rank), (self.rot + 7) // 8 * 8, self.heads * self.vdim
        ld_out = up128(n_out)
        v_row = (self.heads * self.dim + 7) // 8 * 8
        up_rows = up128(v_row + n_out)
        up = np.zeros((up_rows, ld), np.float32)
        up[:self.heads * self.dim, :self.rank] = self.up_k
        up[v_row:v_row + n_out, :self.rank] = self.up_v
        up = put(up, dev, torch.bfloat16)
        frequencies, magnitude = plain.yarn(self.rot, self.base, self.scaling)
        freq, proj, q = put(frequencies, dev), put(self.proj, dev), put(self.q, dev)
        kv_norm, q_norm = put(self.kv_norm, dev), put(self.q_norm, dev)
        latent = torch.full((self.n, ld), float("nan"), device=dev, dtype=dtype)
        keys = torch.full((self.n, key_stride), float("nan"), device=dev, dtype=dtype)
        most, stride = max(portions), lib.qm_latent_query_stride(self.rank, self.rot)
        q_scratch = torch.full((most * self.heads * stride,), float("nan"), device=dev, dtype=dtype)
        ml = torch.full((most * self.heads * splits * 2,), float("nan"), device=dev)
        acc = torch.full((most * self.heads * splits * self.rank,), float("nan"), device=dev)
        nbytes = lib.qm_latent_expanded_bytes(self.n, self.heads, self.dim, self.rot, self.vdim, up_rows)
        expanded = torch.full((nbytes // 2,), float("nan"), device=dev, dtype=torch.bfloat16)
        got, norms, at = [], [], 0
        for rows in portions:
            where = torch.tensor([at], dtype=torch.int32, device=dev)
            latent_q = torch.full((rows, 128), 7.0, device=dev, dtype=dtype)
            keep = decoder.LatentRows(proj=proj.data_ptr() + 4 * self.proj.shape[1] * at, q_norm=q_norm.data_ptr(), kv_norm=kv_norm.data_ptr(),
                                      frequency=freq.data_ptr(), q_latent=latent_q.data_ptr(), latent_cache=latent.data_ptr(), key_cache=keys.data_ptr(),
                                      ld_proj=self.proj.shape[1], ld_q=128, ld_latent=ld, position=at, rows=rows, q_rank=20, kv_rank=self.rank,
                                      rot_dim=self.rot, key_stride=key_stride, q_column=0, kv_column=self.kv_at, eps=self.eps, magnitude=magnitude)
            assert lib.qm_latent_rows_norm(C.byref(keep), int(f32), stream) == 0
            norms.append(get(latent_q))
            out = torch.full((rows, ld_out), 7.0, device=dev, dtype=dtype)
            op = decoder.LatentAttention(q=q.data_ptr() + 4 * self.q.shape[1] * at, frequency=freq.data_ptr(), up_k=up.data_ptr(),
                                         up_v=up.data_ptr() + 2 * v_row * ld, latent_cache=latent.data_ptr(), key_cache=keys.data_ptr(), out=out.data_ptr(),
                                         q_scratch=q_scratch.data_ptr(), ml=ml.data_ptr(), acc=acc.data_ptr(), expanded=expanded.data_ptr(),
                                         ld_query=self.q.shape[1], ld_latent=ld, ld_out=ld_out, expanded_bytes=nbytes, position=at, rows=rows,
                                         heads=self.heads, dim=self.dim, rot_dim=self.rot, vdim=self.vdim, kv_rank=self.rank, key_stride=key_stride,
                                         splits=splits, up_rows=up_rows, up_v_row=v_row, options=decoder.ATTENTION_ROWS if rows_only else 0,
                                         scale=self.scale, magnitude=magnitude)
            if rows == 1:
                op.position, op.position_dev = 0, where.data_ptr()
            assert lib.qm_latent_attention_rows(C.byref(op), int(f32), stream) == 0
            out = get(out)
            assert np.all(out[:, n_out:] == 0)
            got.append(out[:, :n_out])
            at += rows
        return np.concatenate(got), np.concatenate(norms), get(latent), get(keys)


@pytest.mark.parametrize("shape", LATENT)
def test_latent_attention(decoder, dev, shape):
    case = LatentCase(shape, 230)
    want, (latent, key_part) = case.want(), case.kept()
    q_latent = plain.rms_norm(case.proj[:, :20].astype(np.float64), case.q_norm, case.eps)
    for portions in ([230], [100, 2, 28, 1, 1, 17, 3, 16, 62], [1] * 8 + [222], [60, 15, 2, 2, 2, 2] + [1] * 60 + [87]):
        got, norms, c, k = case.run(decoder, dev, True, portions)
        close(got, want, True, tol32=2e-5)
        close(norms[:, :20], q_latent, True, tol32=3e-6)
        close(c[:, :case.rank], latent, True, tol32=3e-6)
        close(k[:, :case.rot], key_part, True, tol32=3e-6)
        assert np.all(norms[:, 20:] == 0) and np.all(c[:, case.rank:] == 0) and np.all(k[:, case.rot:] == 0)
        for rows_only in (False, True):
            got, norms, c, k = case.run(decoder, dev, False, portions, rows_only=rows_only)
            close(got, want, False, tol16=3e-2)
            close(c[:, :case.rank], latent, False)


@pytest.mark.parametrize("splits", [1, 2, 32, 64])
def test_latent_attention_splits(decoder, dev, splits):
    case = LatentCase((6, 24, 8, 16, 72, None), 700, seed=2)
    want = case.want()
    portions = [570, 1, 1, 5] + [1] * 70 + [15, 38]
    close(case.run(decoder, dev, True, portions, splits=splits)[0], want, True, tol32=2e-5)
    for rows_only in (False, True):
        close(case.run(decoder, dev, False, portions, splits=splits, rows_only=rows_only)[0], want, False, tol16=3e-2)


def test_many_positions_are_expanded_in_several_linears(decoder, dev):
    case = LatentCase((2, 16, 8, 16, 32, None), 4400, seed=3)
    close(case.run(decoder, dev, False, [2100, 2300])[0], case.want(), False, tol16=3e-2)


@pytest.mark.parametrize("f32", [True, False])
@pytest.mark.parametrize("rows", [1, 2, 5, 16, 40, 300])
@pytest.mark.parametrize("experts,top,width,ff", [(9, 3, 200, 72), (1, 1, 128, 128), (5, 5, 100, 200), (70, 6, 130, 40), (300, 3, 128, 96), (3, 1, 256, 384)])
def test_experts(decoder, dev, f32, rows, experts, top, width, ff):
    import torch
    rng = np.random.default_rng(experts + rows)
    up128 = lambda n: (n + 127) // 128 * 128
    wp, fp = up128(width), up128(ff)
    x = cases.bf16(rng.standard_normal((rows, width)))
    router = rng.standard_normal((experts, width)) * width ** -0.5
    logits = (x @ router.T).astype(np.float32)
    if experts > 1:
        logits[0, 1] = logits[0, 0]                                   # equals: the lower number first
    if rows > 30:
        logits[:, -1] += 4.0                                          # an expert that nearly every row takes
    gate, up, down = (cases.bf16(rng.standard_normal(s) * s[2] ** -0.5) for s in ((experts, ff, width), (experts, ff, width), (experts, width, ff)))

    def padded(a, *shape):
        out = np.zeros(shape, np.float32)
        out[tuple(slice(0, n) for n in a.shape)] = a
        return out

    xd = put(padded(x, rows, wp), dev, activation(f32))
    ld = experts + 5
    ld_logits = put(padded(logits, rows, ld), dev)
    wd = [put(padded(a, experts, *s), dev, torch.bfloat16) for a, s in ((gate, (fp, wp)), (up, (fp, wp)), (down, (wp, fp)))]
    want = np.zeros((rows, width))
    score = plain.sigmoid(logits.astype(np.float64))
    for t in range(rows):
        for e in np.argsort(-logits[t], kind="stable")[:top]:
            want[t] += score[t, e] * plain.gated_mlp(x[t:t + 1].astype(np.float64), *(w[e].astype(np.float64) for w in (gate, up, down)))[0]
    for options in (0, decoder.EXPERTS_ROWS):
        nbytes = decoder.lib().qm_expert_scratch_bytes(rows, experts, top, wp, fp, int(f32))
        scratch = torch.full((nbytes // 4,), float("nan"), device=dev)
        out = torch.full((rows, wp), 7.0, device=dev)
        op = decoder.Experts(x=xd.data_ptr(), logits=ld_logits.data_ptr(), gate=wd[0].data_ptr(), up=wd[1].data_ptr(), down=wd[2].data_ptr(),
                             out32=out.data_ptr(), scratch=scratch.data_ptr(), ld_logits=ld, scratch_bytes=nbytes, rows=rows, experts=experts, top=top,
                             width_p=wp, ff_p=fp, options=options)
        assert decoder.lib().qm_expert_rows(C.byref(op), int(f32), torch.cuda.current_stream().cuda_stream) == 0
        got = get(out)
        close(got[:, :width], want, f32, tol32=5e-6, tol16=2e-2)
        assert np.all(got[:, width:] == 0)
