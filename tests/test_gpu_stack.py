"""GPU: the configured layer stacks (Tupitar, Mafurax) against oracle/stack_oracle.py — every mechanism alone, whole models in both compute types, and what must not matter:
portions, batches, pages and sequences."""
import ctypes as C
import json
import os
import subprocess
import sys

import numpy as np
import pytest

from conftest import ROOT
from oracle import stack_oracle as so
from stack_cases import CONFIGS, ROWS, SEEDS, attend, config, latent, mafurax, mamba, parallel, tokens

pytestmark = pytest.mark.gpu
TOL = {"float32": 3e-5, "bfloat16": 0.03}                 # of the reference's root mean square
DTYPES = ["float32", "bfloat16"]


def rel(a, b):
    a, b = np.asarray(a, np.float64), np.asarray(b, np.float64)
    return float(np.sqrt(np.mean((a - b) ** 2) / np.mean(b ** 2)))


def near(a, b, dtype, f=1.0):
    """every row (last axis) within the tolerance of the compute type"""
    a, b = np.asarray(a, np.float64), np.asarray(b, np.float64)
    assert a.shape == b.shape
    e = np.sqrt(((a - b) ** 2).mean(-1) / (b ** 2).mean(-1))
    assert np.isfinite(a).all() and e.max() < f * TOL[dtype], "worst row %s: %.3g" % (np.unravel_index(e.argmax(), e.shape), e.max())


# ---- mechanisms alone --------------------------------------------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("n,k,rows", [(1, 1, 1), (17, 31, 3), (130, 33, 64), (300, 75, 16), (48, 600, 17), (513, 96, 33), (260, 288, 65), (1100, 320, 500), (2050, 160, 1500)])
def test_dense(bamd, dtype, n, k, rows):
    r = np.random.default_rng(n + k)
    w = so.f32_to_bf16(r.standard_normal((n, k)))
    x = so.round_bf16(r.standard_normal((rows, k)))
    want = x.astype(np.float64) @ so.bf16_to_f32(w).T.astype(np.float64)
    scale = np.sqrt(k)
    for impl in (0, 1, 2, 3):
        if impl == 1 and rows > 64:
            continue
        tol = 2e-6 if impl < 2 or dtype == "float32" else 0.02
        assert np.abs(bamd.op_dense(w, x, dtype, impl) - want).max() < tol * scale * 4, impl
    if dtype == "float32":                               # operands keep their 32 bits
        x = r.standard_normal((rows, k)).astype(np.float32)
        want = x.astype(np.float64) @ so.bf16_to_f32(w).T.astype(np.float64)
        for impl in (0, 1):
            if impl == 0 or rows <= 64:
                assert np.abs(bamd.op_dense(w, x, dtype, impl) - want).max() < 8e-6 * scale


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("E,rows,pos0,with_y,with_mu", [(75, 5, 0, True, True), (75, 5, 9, True, True), (33, 1, 4, True, True), (1, 3, 0, True, True), (300, 4, 0, False, True), (96, 3, 2, True, False), (2000, 2, 7, True, True)])
def test_residual_norm_and_token_shift(bamd, dtype, E, rows, pos0, with_y, with_mu):
    r = np.random.default_rng(E + rows)
    x, y, prev = r.standard_normal((rows, E)), r.standard_normal((rows, E)) * 3, r.standard_normal(E)
    mu = r.uniform(0, 1, E) if with_mu else None
    xo, h, last = bamd.op_residual_rows(x, y if with_y else None, 0.7, 1e-3, mu, prev, pos0, dtype)
    ref = np.stack([xi + so.scalar_norm(yi, 0.7, 1e-3) if with_y else xi for xi, yi in zip(x, y)])
    near(xo, ref, "float32")
    if with_mu:
        front = np.concatenate([(prev if pos0 else np.zeros(E))[None], ref[:-1]])
        near(h, np.stack([so.token_shift(a, b, mu) for a, b in zip(ref, front)]), dtype)
        near(last, ref[-1], "float32")
    else:
        near(h, ref, dtype)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("F", [1, 40, 333, 3000])
def test_poly_norm(bamd, dtype, F):
    r = np.random.default_rng(F)
    z, coef = r.standard_normal((6, F)) * np.array([1e-3, 0.1, 1, 3, 10, 50])[:, None], [0.8, -0.5, 0.6, 0.25]
    near(bamd.op_poly_norm(z, coef, 1e-4, dtype), np.stack([so.poly_norm(v, *coef, 1e-4) for v in z]), dtype)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("n,groups", [(60, 1), (60, 5), (120, 3), (256, 64), (20, 20), (4096, 8)])
def test_group_norm(bamd, dtype, n, groups):
    r = np.random.default_rng(n + groups)
    y, w = r.standard_normal((3, n)) * np.repeat(r.uniform(0.1, 10, groups), n // groups), 1 + r.standard_normal(n)
    near(bamd.op_group_norm(y, w, groups, 1e-5, dtype), np.stack([so.grouped_norm(v, groups, w, 1e-5) for v in y]), dtype)


def plain_ssm(rows, H, P, N, G, conv, cb, dtb, A, D, hist, S):
    inner, out = H * P, []
    for row in rows:
        z, xbc, dt = np.split(row, [inner, 2 * inner + 2 * G * N])
        xbc, hist = so.causal_conv(conv, cb, hist, xbc)
        x, B, C_ = np.split(so.silu(xbc), [inner, inner + G * N])
        dt = so.softplus(dt + dtb)
        y = np.zeros(inner)
        for i in range(H):
            g = i // (H // G)
            S[i], y[i * P:(i + 1) * P] = so.ssd_step(S[i], dt[i], A[i], D[i], B[g * N:(g + 1) * N], C_[g * N:(g + 1) * N], x[i * P:(i + 1) * P])
        out.append(y * so.silu(z))
    return np.array(out), hist, S


@pytest.mark.parametrize("H,P,N,G,taps", [(1, 1, 1, 1, 1), (3, 20, 24, 1, 4), (4, 10, 12, 4, 2), (4, 16, 40, 2, 3), (2, 130, 33, 1, 7), (1, 64, 256, 1, 4), (2, 24, 128, 2, 5)])
def test_ssm(bamd, H, P, N, G, taps):
    """portions from one token up, first tokens (taps reach before the start), state and convolution inputs handed from portion to portion, fast and slow decays"""
    r = np.random.default_rng(H * P + N)
    inner, ch = H * P, H * P + 2 * G * N
    conv, cb, dtb, A, D = r.standard_normal((ch, taps)), r.standard_normal(ch) * 0.3, r.uniform(-6, 1, H), r.uniform(-4, 2, H), r.standard_normal(H)
    f = lambda a: np.asarray(a, np.float32)
    rows = f(r.standard_normal((70, inner + ch + H)))
    rows[::9, -H:] -= 30                                  # a step size of almost zero: the state stays as it is
    rows[5::11, -H:] += 25                                # and a large one: it is forgotten
    conv, cb, dtb, A, D = map(f, (conv, cb, dtb, A, D))
    hist, S = np.zeros((taps - 1, ch)), np.zeros((H, N, P))
    gh, gs, pos = f(hist), f(S) + 7, 0                    # what a fresh sequence finds in its place must not matter
    gh = gh + 7
    for n in (1, 1, 2, 15, 16, 17, 18):
        part = rows[pos:pos + n]
        want, hist, S = plain_ssm(part.astype(np.float64), H, P, N, G, conv, cb, dtb, A, D, hist, S)
        got, gh, gs = bamd.op_ssm(part, pos, H, P, N, G, conv, cb, dtb, A, D, gh, gs)
        assert rel(got, want) < 2e-5, pos
        assert rel(gs, S) < 2e-5 and (taps == 1 or rel(gh, hist) < 1e-6)
        pos += n


def plain_attention(q, c, gate, past, uk, uv, c_norm, sink, scale, eps, H):
    T, _, d = q.shape
    lat = np.stack([so.rms(v, eps) * c_norm for v in c])
    every = lat if past is None else np.concatenate([past, lat])
    uk, uv = so.bf16_to_f32(uk).astype(np.float64), so.bf16_to_f32(uv).astype(np.float64)
    k, v = (every @ uk.T).reshape(len(every), H, d), (every @ uv.T).reshape(len(every), H, -1)
    out = np.zeros((T, H, v.shape[2]))
    for t in range(T):
        n = len(every) - T + t + 1
        for h in range(H):
            s = k[:n, h] @ q[t, h] * scale
            p = so.sink_softmax(s, sink[h]) if sink is not None else np.exp(s - s.max()) / np.exp(s - s.max()).sum()
            out[t, h] = p @ v[:n, h] * (so.sigmoid(gate[t, h]) if gate is not None else 1)
    return out


def attention_case(H, d, dv, R, T, pos0, seed, dtype):
    r = np.random.default_rng(seed)
    rd = so.round_bf16 if dtype == "bfloat16" else (lambda a: np.asarray(a, np.float32))
    return dict(q=rd(r.standard_normal((T, H, d))), c=rd(r.standard_normal((T, R))), gate=r.standard_normal((T, H)).astype(np.float32), past=rd(r.standard_normal((pos0, R))) if pos0 else None,
                uk=so.f32_to_bf16(r.standard_normal((H * d, R)) / np.sqrt(R)), uv=so.f32_to_bf16(r.standard_normal((H * dv, R)) / np.sqrt(R)), c_norm=rd(1 + 0.2 * r.standard_normal(R)),
                sink=r.standard_normal(H).astype(np.float32), scale=1.5 / np.sqrt(d), eps=1e-5)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,d,dv,R", [(1, 8, 8, 8), (3, 24, 40, 36), (5, 33, 12, 20), (17, 16, 32, 64), (2, 72, 130, 100), (2, 128, 64, 200), (1, 200, 16, 300), (2, 64, 128, 700)])
@pytest.mark.parametrize("T,pos0", [(1, 0), (3, 0), (63, 0), (130, 0), (2, 63), (2, 64), (66, 130), (1, 63), (1, 64), (1, 200), (1, 500)])
def test_latent_attention(bamd, dtype, H, d, dv, R, T, pos0):
    a = attention_case(H, d, dv, R, T, pos0, H * d + T + pos0, dtype)
    want = plain_attention(H=H, **a)
    for decode in ((False, True) if T == 1 else (False,)):
        got = bamd.op_latent_attention(dtype=dtype, decode=decode, **a)
        near(got.reshape(T, -1), want.reshape(T, -1), dtype)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("pos0", [0, 127, 250])
def test_one_key_stands_out(bamd, dtype, pos0):
    """one score far above hundreds of others, at the first positions, on both sides of every page border, at the query itself, and just behind it (never seen)"""
    H, d, dv, R, n = 2, 24, 40, 36, 300
    T = n - pos0
    a = attention_case(H, d, dv, R, n, 0, 77, dtype)
    lat = np.stack([so.rms(v, a["eps"]) * a["c_norm"] for v in a["c"]])
    k = (lat @ so.bf16_to_f32(a["uk"]).T.astype(np.float64)).reshape(n, H, d)
    for key in (0, 1, 2, 62, 63, 64, 65, 127, 128, 191, 192, 250, 255, 256, 298, 299):
        q = np.zeros((n, H, d))
        q[:] = k[key] / (k[key] ** 2).sum(-1, keepdims=True)
        rd = so.round_bf16 if dtype == "bfloat16" else (lambda v: np.asarray(v, np.float32))
        case = dict(a, q=rd(q[pos0:]), c=a["c"][pos0:], gate=a["gate"][pos0:], past=rd(lat[:pos0]) if pos0 else None, scale=24.0)
        want = plain_attention(H=H, **case)
        near(bamd.op_latent_attention(dtype=dtype, **case).reshape(T, -1), want.reshape(T, -1), dtype, 3)
    # the same, decoded: the query is the last position
    for key in (0, 63, 64, 191, 298, 299):
        case = dict(a, q=rd(k[key][None] / (k[key] ** 2).sum(-1)[None, :, None]), c=a["c"][-1:], gate=a["gate"][-1:], past=rd(lat[:-1]), scale=24.0)
        want = plain_attention(H=H, **case)
        near(bamd.op_latent_attention(dtype=dtype, decode=True, **case).reshape(1, -1), want.reshape(1, -1), dtype, 3)


@pytest.mark.parametrize("decode", [False, True])
@pytest.mark.parametrize("dtype", DTYPES)
def test_sinks_and_gates(bamd, dtype, decode):
    """sinks from nothing to almost everything, none at all, gates open, shut and absent"""
    H, d, dv, R = 4, 16, 16, 24
    a = attention_case(H, d, dv, R, 1, 150, 5, dtype)
    for sink in ([-60, -2, 4, 9], [80, 0, 30, -80], None):
        for gate in (np.array([[-30, -1, 2, 30.]], np.float32), None):
            case = dict(a, sink=None if sink is None else np.array(sink, np.float32), gate=gate)
            want, got = plain_attention(H=H, **case), bamd.op_latent_attention(dtype=dtype, decode=decode, **case)
            live = np.abs(want).max(-1) > 1e-6
            near(got[live], want[live], dtype)
            assert np.abs(got[~live]).max(initial=0) < 1e-6


# ---- whole models ------------------------------------------------------------------------------------------------------------------------------------------
class Case:
    def __init__(self, folder, cfg, seed, rows=None):
        self.folder, self.cfg = folder, cfg
        w = so.random_model(cfg, seed, rows)
        so.write_model(folder, cfg, w)
        self.oracle = so.StackModel(cfg, w)
        self.known = {}

    def logits(self, toks):
        key = tuple(toks)
        if key not in self.known:
            self.known[key] = self.oracle.forward(toks)
        return self.known[key]


@pytest.fixture(scope="module")
def cases(tmp_path_factory):
    d = tmp_path_factory.mktemp("stack")
    return {n: Case(str(d / n), c, SEEDS[n], ROWS.get(n)) for n, c in sorted(CONFIGS.items())}


@pytest.fixture(params=[(n, t) for n in sorted(CONFIGS) for t in DTYPES], ids=lambda p: "-".join(p))
def run(request, bamd, cases):
    name, dtype = request.param
    m = bamd.Model(cases[name].folder, dtype=dtype)
    c = bamd.Context(m, 512, 4)
    yield cases[name], c, dtype
    c.close(); m.close()


def everywhere(toks):
    return list(range(len(toks)))


@pytest.mark.parametrize("n", [1, 2, 3, 5, 64, 65, 150])
def test_prompt(run, n):
    case, c, dtype = run
    t = tokens(case.cfg, 150, 1)[:n]
    near(c.decode_batch([(0, t, everywhere(t))]), case.logits(tokens(case.cfg, 150, 1))[:n], dtype)


def test_prompt_against_decoding(run):
    """token by token from the first one, over two page borders"""
    case, c, dtype = run
    t = tokens(case.cfg, 150, 1)
    got = np.concatenate([c.decode_batch([(2, [x], [0])]) for x in t])
    near(got, case.logits(t), dtype)


@pytest.mark.parametrize("size", [2, 3, 7, 33, 64, 65, 100])
def test_portions(run, size):
    case, c, dtype = run
    t = tokens(case.cfg, 150, 1)
    got = np.concatenate([c.decode_batch([(1, t[i:i + size], everywhere(t[i:i + size]))]) for i in range(0, len(t), size)])
    near(got, case.logits(t), dtype)
    assert c.seq_len(1) == 150


def test_unequal_batch_against_each_alone(run):
    case, c, dtype = run
    lens = [1, 70, 23, 129]
    t = [tokens(case.cfg, n + 10, 20 + n) for n in lens]
    got = c.decode_batch([(s, t[s][:n], everywhere(t[s][:n])) for s, n in enumerate(lens)])
    at = 0
    for s, n in enumerate(lens):
        near(got[at:at + n], case.logits(t[s])[:n], dtype)
        at += n
    for k in range(10):                                   # decoded together; the shorter ones stop earlier
        live = [s for s in range(4) if k < 4 + 2 * s]
        got = c.decode_batch([(s, [t[s][lens[s] + k]], [0]) for s in live])
        for g, s in zip(got, live):
            near(g, case.logits(t[s])[lens[s] + k], dtype)
        for s in range(4):
            if k == 3 + 2 * s:
                c.seq_free(s)


def test_mixed_batch(run):
    """a decoding sequence, a continued prompt and a fresh one in the same batch; places wanted in one of them only"""
    case, c, dtype = run
    t = tokens(case.cfg, 150, 1)
    c.decode_batch([(0, t[:80], []), (1, t[:5], [])])
    got = c.decode_batch([(1, t[5:71], [0, 65]), (0, t[80:81], [0]), (3, t[:9], [])])
    near(got, case.logits(t)[[5, 70, 80]], dtype)
    got = c.decode_batch([(0, t[81:82], [0]), (1, t[71:72], []), (3, t[9:10], [0])])
    near(got, case.logits(t)[[81, 9]], dtype)


def test_pages_and_sequences_used_again(run):
    case, c, dtype = run
    t, u = tokens(case.cfg, 150, 1), tokens(case.cfg, 140, 9)
    for s in range(4):
        c.decode_batch([(s, u[:100 + s], [])])
    for s in (2, 0):
        c.seq_free(s)
    near(c.decode_batch([(2, t[:70], everywhere(t[:70]))]), case.logits(t)[:70], dtype)
    near(c.decode_batch([(0, t[:3], [0, 1, 2])]), case.logits(t)[:3], dtype)
    got = c.decode_batch([(1, u[101:102], [0]), (3, u[103:104], [0]), (2, t[70:71], [0]), (0, t[3:4], [0])])
    near(got[2:], case.logits(t)[[70, 3]], dtype)
    near(got[:2], case.logits(u)[[101, 103]], dtype)
    for s in range(4):
        c.seq_free(s)
    near(c.decode_batch([(3, t, everywhere(t))]), case.logits(t), dtype)


def test_decode_interface(run):
    """bamd_decode on sequence 0: a new prompt at position 0 replaces it, positions cannot be taken back"""
    import booster_amd
    case, c, dtype = run
    t = tokens(case.cfg, 150, 1)
    c.decode(t[:30], 0)
    near(c.decode(t[:40], 0), case.logits(t)[39], dtype)
    near(c.decode(t[40:41], 40), case.logits(t)[40], dtype)
    near(c.last_logits(), case.logits(t)[40], dtype)
    with pytest.raises(booster_amd.BamdError, match="41 tokens"):
        c.decode(t[:5], 30)
    with pytest.raises(booster_amd.BamdError):
        c.kv_seq_add(0, 10, 1)
    with pytest.raises(booster_amd.BamdError):
        c.kv_seq_rm(10, -1)
    c.kv_seq_rm(0, -1)
    assert c.seq_len(0) == 0


def test_greedy_generation(run):
    """the device loop, the same in a batch of unequal sequences, and the scheduler over more requests than sequences: the same tokens; in 32-bit the plain statement's"""
    from booster_amd.scheduler import Scheduler
    case, c, dtype = run
    prompts = [tokens(case.cfg, n, 40 + n) for n in (1, 63, 20, 40, 7, 64)]
    n_new = 12
    alone, first = [], []
    for p in prompts:
        first.append(int(np.argmax(c.decode(p, 0))))
        out, _ = c.generate_greedy(len(p), n_new - 1)
        assert out[0] == first[-1]
        last = c.last_logits()
        alone.append([int(x) for x in out])
        assert int(np.argmax(last)) == alone[-1][-1]
        c.seq_free(0)
    if dtype == "float32":
        for p, a in zip(prompts[:4], alone):
            st = case.oracle.new_state()
            l = case.oracle.forward(p, st)[-1]
            for tok in a:
                top = np.sort(l)[-2:]
                assert int(np.argmax(l)) == tok or top[1] - top[0] < 1e-4 * np.abs(l).max()
                l = case.oracle.forward([tok], st)[-1]
    for s in range(4):
        c.decode_batch([(s, prompts[s], [])])
    out, _ = c.generate_greedy_seqs([0, 1, 2, 3], first[:4], n_new - 1)
    for s in range(4):
        c.seq_free(s)
    sched = Scheduler(c).generate(prompts, n_new)
    if dtype == "float32":
        assert [[int(x) for x in o] for o in out] == alone[:4] and sched == alone
    else:                                                 # rounding may pick another of two near equals: the first tokens agree
        assert [int(o[0]) for o in out] == first[:4] and [o[0] for o in sched] == first


@pytest.mark.parametrize("name", ["odd", "side", "side_long"])
def test_long_decoding(bamd, cases, name):
    """hundreds of decoded tokens behind a short prompt: in one device loop, then token by token, over page borders; the state of a sequence beside it stays"""
    case = cases[name]
    m = bamd.Model(case.folder, dtype="float32"); c = bamd.Context(m, 704, 2)
    p = tokens(case.cfg, 6, 3)
    c.decode_batch([(1, tokens(case.cfg, 9, 4), [])])
    c.decode(p, 0)
    out, _ = c.generate_greedy(len(p), 301)
    seq = p + [int(x) for x in out[:-1]]
    want = case.logits(seq)
    near(c.last_logits(), want[-1], "float32")
    assert all(int(np.argmax(l)) == int(t) for l, t in zip(want[len(p) - 1:], out))
    more = tokens(case.cfg, 30, 5)
    st = case.oracle.new_state(); case.oracle.forward(seq, st)
    ref = case.oracle.forward(more, st)
    near(np.stack([c.decode([t], len(seq) + i) for i, t in enumerate(more)]), ref, "float32")
    near(c.decode_batch([(1, [1], [0])])[0], case.logits(tokens(case.cfg, 9, 4) + [1])[-1], "float32")
    c.close(); m.close()


@pytest.mark.parametrize("design", ["Tupitar", "Mafurax"])
@pytest.mark.parametrize("dtype", DTYPES)
def test_many_wanted_places_and_passes(bamd, dtype, design, tmp_path):
    """more rows than one pass holds (2048), more wanted places than the logits buffer, a prompt cut between passes, a wide latent and larger matrices; scans in segments, a window and kept
    tokens far behind the queries"""
    cfg = config(128, 97, [latent(2, 16, 24, 40, 0.3, ff=64), mamba(2, 12, 10, 1, 1, 4, ff=48)], max_positions=1600)
    if design == "Mafurax":
        cfg = mafurax(128, 97, [parallel(attend(4, 2, 16, 24, 0.5, 10.0, 120, 200, 9), 0.8, (2, 20, 24, 16.0), 1.0, ff=64, limit=1.0),
                                parallel(attend(2, 1, 24, 16, 0.4, 12.0, 800, 900, 0), 0.8, (3, 12, 16, 16.0), 1.0, ff=48, limit=1.0)])
    case = Case(str(tmp_path / "m"), cfg, 3)
    m = bamd.Model(case.folder, dtype=dtype); c = bamd.Context(m, 3200, 3)
    t = [tokens(cfg, n, n) for n in (900, 1500, 40)]
    want = [[0, 899], list(range(1200, 1400)) + [1499], everywhere(t[2])]
    got = c.decode_batch([(s, t[s], want[s]) for s in range(3)])
    at = 0
    for s in range(3):
        near(got[at:at + len(want[s])], case.logits(t[s])[want[s]], dtype, 2)      # the worst of some 240 rows
        at += len(want[s])
    c.close(); m.close()


def test_limits(bamd, cases):
    import booster_amd
    case = cases["odd"]
    m = bamd.Model(case.folder, dtype="bfloat16"); c = bamd.Context(m, 1024, 2)
    t = tokens(case.cfg, 700, 1)
    c.decode_batch([(0, t, [])])
    for bad in ([(0, [1], [0])],                          # behind the last learned position
                [(2, [1], [0])], [(1, [], [])], [(1, [case.cfg["vocab"]], [0])], [(1, [-1], [0])], [(1, [1, 2], [2])], [(1, [1, 2], [1, 0])], [(1, [1], []), (1, [2], [])],
                [(1, t[:480], [])]):                      # 700 + 480 positions do not fit
        with pytest.raises(booster_amd.BamdError):
            c.decode_batch(bad)
    assert c.seq_len(0) == 700 and c.seq_len(1) == 0      # refused batches leave the sequences alone
    with pytest.raises(booster_amd.BamdError):
        c.generate_greedy(700, 1)
    near(c.decode_batch([(1, t[:50], [49])]), case.logits(t[:50])[-1:], "bfloat16")
    c.close(); m.close()
    broken = dict(case.cfg, layers=[dict(case.cfg["layers"][0], type="nope")])
    os.makedirs(case.folder + "_b", exist_ok=True)
    json.dump(broken, open(case.folder + "_b/config.json", "w"))
    if not os.path.exists(case.folder + "_b/model.safetensors"):
        os.symlink(case.folder + "/model.safetensors", case.folder + "_b/model.safetensors")
    with pytest.raises(booster_amd.BamdError, match="nope"):
        bamd.Model(case.folder + "_b")
    json.dump(dict(case.cfg, width=76), open(case.folder + "_b/config.json", "w"))
    with pytest.raises(booster_amd.BamdError, match="expected shape"):
        bamd.Model(case.folder + "_b")


@pytest.mark.parametrize("name", ["odd", "side"])
@pytest.mark.parametrize("dtype", DTYPES)
def test_layer_split_stages(bamd, cases, dtype, name):
    """the layers over two stages with the hidden state handed over: prompt, portions and single tokens"""
    import torch
    case = cases[name]
    t = tokens(case.cfg, 150, 1)
    E = case.cfg["width"]
    a = bamd.Model(case.folder, layer_first=0, layer_last=1, with_output=False, dtype=dtype)
    b = bamd.Model(case.folder, layer_first=1, layer_last=-1, with_embd=False, dtype=dtype)
    ca, cb = bamd.Context(a, 256), bamd.Context(b, 256)
    hid = torch.zeros((128, E), device="cuda", dtype=torch.float32)
    tok = torch.zeros(1, device="cuda", dtype=torch.int32)
    s = torch.cuda.current_stream().cuda_stream
    pos = 0
    for n in (70, 2, 33):
        assert ca.stage_prefill(t[pos:pos + n], n, pos, None, hid.data_ptr(), False, s)
        assert cb.stage_prefill(None, n, pos, hid.data_ptr(), None, True, s)
        pos += n
        near(cb.stage_logits(s), case.logits(t)[pos - 1], dtype)
    for _ in range(6):
        tok.fill_(t[pos])
        ca.stage_step(0, pos, None, hid.data_ptr(), 0, 0, s, token_dev_ptr=tok.data_ptr())
        cb.stage_step(0, pos, hid.data_ptr(), None, 1, 0, s)
        pos += 1
        near(cb.stage_logits(s), case.logits(t)[pos - 1], dtype)
        assert cb.stage_argmax(s) == int(np.argmax(cb.stage_logits(s)))
        cb.stage_token_to(tok.data_ptr(), s); torch.cuda.synchronize()
        assert int(tok[0]) == int(np.argmax(cb.stage_logits(s)))
    for x in (ca, cb, a, b):
        x.close()


@pytest.mark.parametrize("name", ["wide", "side_wide"])
def test_replays_with_other_work_between(bamd, cases, name):
    """the decoding graph, replayed with prompts, other sequences and eager work between its replays, gives what a fresh context gives"""
    case = cases[name]
    t = tokens(case.cfg, 80, 6)
    m = bamd.Model(case.folder, dtype="float32"); c = bamd.Context(m, 512, 3)
    c.decode_batch([(0, t[:40], [])])
    for k in range(40, 60):
        got = c.decode_batch([(0, [t[k]], [0])])
        near(got, case.logits(t)[k:k + 1], "float32")
        if k % 3 == 0:
            c.decode_batch([(1, t[:k], [k - 1])]); c.decode_batch([(1, [t[k]], [])]); c.seq_free(1)
        if k % 4 == 0:
            near(bamd.op_poly_norm(np.ones((2, 40)), [1, 1, 1, 1], 0.0, "float32"), np.full((2, 40), 4.0), "float32")
        if k % 5 == 0:
            c.decode_batch([(2, [t[0]], [0])]); c.seq_free(2)
    c.close(); m.close()


@pytest.mark.parametrize("design", ["Tupitar", "Mafurax"])
def test_bridge_serves_a_model_folder(bamd, design, tmp_path):
    """initContext / doInference on a folder with tokenizer.gguf: prompt, Janus sampling on the device's logits, text out; without a tokenizer the request is refused"""
    from booster_amd import gguf
    from test_gpu_bridge import bind, ctx_args
    L = bind(bamd)
    vocab = gguf.synthetic_spm_vocab()
    cfg = config(60, len(vocab["tokens"]), [mamba(2, 12, 16, 1, 2, 4, ff=50), latent(3, 16, 20, 24, 0.3, ff=64)], max_positions=192)
    if design == "Mafurax":
        cfg = mafurax(60, len(vocab["tokens"]), [parallel(attend(4, 2, 16, 20, 0.4, 7.0, 30, 9, 2), 0.9, (2, 12, 16, 4.0), 0.8, ff=50, limit=0.9)])
    jobs = [(design + n).encode() for n in ("-none", "-a", "-b")]
    d = str(tmp_path / "m")
    so.write_model(d, cfg, so.random_model(cfg, 8))
    ctx = L.initContext(*ctx_args(6, d, (100, 0, 0, 0), 128, 24))
    assert ctx and L.doInference(6, ctx, jobs[0], b"s", b"the cat sat") == 1
    gguf.write_synthetic_llama(d + "/tokenizer.gguf", E=256, H=2, Hkv=1, L=1, F=256, V=len(vocab["tokens"]), seed=2, vocab=vocab)
    ctx = L.initContext(*ctx_args(6, d, (100, 0, 0, 0), 128, 24))
    assert ctx
    for job in jobs[1:]:                  # the second request starts over in the same context
        n = L.doInference(6, ctx, job, b"s", b"the cat sat on the hat")
        prompt = L.getPromptTokenCount(job)
        assert prompt > 4 and prompt <= n <= prompt + 23
        text = L.status(job)
        assert b"the cat sat on the hat" in text
    # hi = lo = 1: only the top candidate survives, the draw is the arg-max of the penalised logits and both requests agree
    assert L.status(jobs[1]) == L.status(jobs[2])


@pytest.mark.parametrize("name", ["odd", "side"])
def test_trace_run(bamd, cases, name, tmp_path):
    """bin/trace_run replays requests step by step and writes the wanted logits"""
    case = cases[name]
    t = tokens(case.cfg, 150, 1)
    steps = [{"step": 0, "entries": [{"id": "x", "tokens": t[:70], "want": [69, 3]}, {"id": "y", "tokens": t[:5], "want": []}], "end": []},
             {"step": 1, "entries": [{"id": "y", "tokens": [t[5]], "want": [0]}, {"id": "x", "tokens": [t[70]], "want": [0]}], "end": ["y"]},
             {"step": 2, "entries": [{"id": "x", "tokens": [t[71]], "want": []}], "end": ["x"]},
             {"step": 3, "entries": [{"id": "y", "tokens": t[:9], "want": [8]}], "end": ["y"]}]
    for dtype in DTYPES:
        out = tmp_path / dtype
        out.mkdir()
        p = subprocess.run([sys.executable, os.path.join(ROOT, "bin", "trace_run"), "--model", case.folder, "--dtype", dtype, "--out", str(out), "--max-tokens", "256"],
                           input="".join(json.dumps(s) + "\n" for s in steps), capture_output=True, text=True, timeout=100)
        assert p.returncode == 0, p.stderr[-2000:]
        assert [l for l in p.stdout.splitlines() if l.startswith("done")] == ["done %d" % i for i in range(4)]
        want = case.logits(t)
        for step, rows in ((0, [69, 3]), (1, [5, 70]), (3, [8])):
            got = np.fromfile(str(out / ("%d.f32" % step)), "<f4").reshape(len(rows), -1)
            near(got, want[rows], dtype)
        assert not (out / "2.f32").exists()


@pytest.mark.parametrize("name", ["odd", "side"])
def test_command_line(bamd, cases, name, capsys):
    """python -m booster_amd: several requests of a folder together; a GGUF model through the same scheduler, one request after the other"""
    from booster_amd.__main__ import main
    from conftest import GOLDEN
    case = cases[name]
    prompts = [tokens(case.cfg, n, n) for n in (5, 70, 33)]
    assert main(["--model", case.folder, "--dtype", "float32", "-n", "6"] + [x for p in prompts for x in ("--tokens", ",".join(map(str, p)))]) == 0
    got = [[int(t) for t in l.split(",")] for l in capsys.readouterr().out.split()]
    m = bamd.Model(case.folder, dtype="float32"); c = bamd.Context(m, 128)
    for p, g in zip(prompts, got):
        first = int(np.argmax(c.decode(p, 0)))
        assert g == [int(x) for x in c.generate_greedy(len(p), 5)[0]] and g[0] == first
    c.close(); m.close()
    path = os.path.join(GOLDEN, "tiny_a.gguf")
    assert main(["--model", path, "-n", "6", "--tokens", "1,5,9,2", "--tokens", "3,4"]) == 0
    got = [[int(t) for t in l.split(",")] for l in capsys.readouterr().out.split()]
    m = bamd.Model(path); c = bamd.Context(m, 128)
    for p, g in zip(([1, 5, 9, 2], [3, 4]), got):
        c.decode(p, 0)
        assert g == [int(x) for x in c.generate_greedy(len(p), 5)[0]]
    c.close(); m.close()
