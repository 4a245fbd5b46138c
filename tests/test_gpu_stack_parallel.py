"""GPU: the mechanisms of the Mafurax design alone, against oracle/stack_oracle.py — attention over cached keys and values, gated linear attention, layer norms around a
sublayer, the clamped gated unit.  Whole models: test_gpu_stack.py."""
import functools

import numpy as np
import pytest

from oracle import stack_oracle as so
from test_gpu_stack import DTYPES, near, rel

pytestmark = pytest.mark.gpu


def rounder(dtype):
    return so.round_bf16 if dtype == "bfloat16" else (lambda a: np.asarray(a, np.float32))


# ---- rows --------------------------------------------------------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("E,rows,with_y,with_pre", [(75, 5, True, True), (2, 3, True, True), (96, 4, False, True), (96, 4, True, False), (300, 70, True, True), (1028, 2, True, True), (3000, 3, True, True), (9001, 2, True, True)])
def test_layer_norms_around_a_sublayer(bamd, dtype, E, rows, with_y, with_pre):
    """rows with means far from zero, and small and large spreads"""
    r = np.random.default_rng(E + rows)
    spread = 10.0 ** r.uniform(-1, 1, (rows, 1))
    x, y = r.standard_normal((rows, E)) * spread + 3, r.standard_normal((rows, E)) * spread[::-1] - 20 * spread[::-1]
    g, gi = r.standard_normal(E), 1 + 0.3 * r.standard_normal(E)
    xo, h = bamd.op_layer_rows(x, y if with_y else None, g, gi if with_pre else None, 1e-4, dtype)
    f = lambda a: np.asarray(a, np.float32).astype(np.float64)
    x, y = f(x), f(y)
    ref = np.stack([a + so.layer_norm(b, g, 1e-4) if with_y else a for a, b in zip(x, y)])
    near(xo, ref, "float32")
    near(h, np.stack([so.layer_norm(a, gi, 1e-4) for a in ref]) if with_pre else ref, dtype)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("F,rows,limit", [(1, 1, 1.0), (40, 3, 0.5), (333, 2, 2.0), (3000, 2, 7.0)])
def test_clamped_glu(bamd, dtype, F, rows, limit):
    """values inside, at and far beyond the limits, on both sides"""
    r = np.random.default_rng(F)
    g, u = r.standard_normal((rows, F)) * 3, r.standard_normal((rows, F)) * 3
    g.flat[:5], u.flat[:5] = [limit, 100, -100, -limit, 0][:g.size], [100, -100, limit, -1, -limit][:u.size]
    got, want = bamd.op_clamped_glu(g, u, limit, dtype), so.clamped_glu(g, u, limit)
    assert np.abs(got - want).max() < (1e-5 if dtype == "float32" else 0.005) * (1 + np.abs(want).max())


# ---- attention ---------------------------------------------------------------------------------------------------------------------------------------------
@functools.lru_cache(None)
def seen_keys(n, size, keep_first):
    return [[j for j in range(i + 1) if so.visible(i, j, {"size": size, "keep_first": keep_first})] for i in range(n)]


def plain(a, T):
    """queries at the last T positions of the keys and values"""
    q, k, v = (np.asarray(a[x], np.float64) for x in "qkv")
    H, G = q.shape[1], k.shape[1]
    if a["past_k"] is not None:
        k, v = np.concatenate([a["past_k"], np.stack([[so.rms(x, a["eps"]) for x in row] for row in k]) if a["unit"] else k]), np.concatenate([a["past_v"], v])
    elif a["unit"]:
        k = np.stack([[so.rms(x, a["eps"]) for x in row] for row in k])
    n = len(k)
    out = np.zeros((T, H, v.shape[2]))
    bucket = None if a["rel"] is None else np.array([so.distance_bucket(x, len(a["rel"]), a["bias_max"]) for x in range(n)])
    for t in range(T):
        i = n - T + t
        seen = np.array(seen_keys(n, a["window"], a["keep"])[i])
        for h in range(H):
            qh = so.rms(q[t, h], a["eps"]) if a["unit"] else q[t, h]
            s = k[seen, h // (H // G)] @ qh * a["scale"]
            if a["cap"]:
                s = so.softcap(s, a["cap"])
            bias = 0 * s if a["rel"] is None else a["rel"][bucket[i - seen], h]
            out[t, h] = so.biased_softmax(s, bias) @ v[seen, h // (H // G)] * (so.sigmoid(a["gate"][t, h]) if a["gate"] is not None else 1) * a.get("out_scale", 1.0)
    return out


def case(dtype, H, G, d, dv, T, pos0, window, keep, rows=8, top=60, cap=8.0, unit=True, seed=0):
    """the keys in front as a cache of that type holds them"""
    r, rd = np.random.default_rng(seed + H * d + T + pos0 + window), rounder(dtype)
    k, v = r.standard_normal((pos0 + T, G, d)), rd(r.standard_normal((pos0 + T, G, dv)))
    past = rd(np.stack([[so.rms(x, 1e-5) for x in row] for row in k[:pos0]])) if pos0 else None
    return dict(q=rd(r.standard_normal((T, H, d))), k=rd(k[pos0:]), v=v[pos0:], gate=r.standard_normal((T, H)).astype(np.float32), past_k=past, past_v=v[:pos0] if pos0 else None, scale=2.0 / np.sqrt(d), cap=cap, eps=1e-5,
                unit=unit, rel=r.standard_normal((rows, H)).astype(np.float32) if rows else None, bias_max=top, window=window, keep=keep)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,G,d,dv", [(1, 1, 8, 8), (6, 2, 24, 40), (3, 3, 33, 12), (34, 2, 16, 32), (4, 1, 72, 130), (2, 2, 128, 64), (2, 1, 200, 16), (8, 4, 1, 3)])
@pytest.mark.parametrize("T,pos0,window,keep", [(1, 0, 5, 2), (3, 0, 1, 0), (130, 0, 20, 3), (200, 0, 64, 65), (2, 63, 30, 1), (2, 64, 1000, 0), (70, 130, 65, 5), (1, 63, 10, 3), (1, 64, 64, 64), (1, 300, 63, 70), (1, 500, 1 << 20, 0)])
def test_window_attention(bamd, dtype, H, G, d, dv, T, pos0, window, keep):
    a = case(dtype, H, G, d, dv, T, pos0, window, keep)
    want = plain(a, T).reshape(T, -1)
    for splits in (0, 1, 2, 7) if T == 1 else (0,):
        near(bamd.op_kv_attention(dtype=dtype, splits=splits, **a).reshape(T, -1), want, dtype)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("splits", [0, 3])
def test_every_part_may_be_absent(bamd, dtype, splits):
    """no unit norm, no cap, no bias, no gate; an output scale"""
    base = case(dtype, 4, 2, 24, 24, 1, 150, 40, 3)
    for change in (dict(unit=False), dict(cap=0.0), dict(rel=None), dict(gate=None), dict(unit=False, cap=0.0, rel=None, gate=None), dict(out_scale=-1.7), dict(gate=np.array([[-30, 0, 2, 30.]], np.float32))):
        a = dict(base, **change)
        want, got = plain(a, 1), bamd.op_kv_attention(dtype=dtype, splits=splits, **a)
        live = np.abs(want).max(-1) > 1e-6
        near(got[live], want[live], dtype)
        assert np.abs(got[~live]).max(initial=0) < 1e-6


def pointed(dtype, n, pos0, window, keep, key, cap=40.0, d=24):
    """every query asks for one key: its score is far above the others' """
    a = case(dtype, 2, 1, d, 40, n, 0, window, keep, rows=6, top=90, cap=cap, seed=3)
    k = np.stack([so.rms(x[0], 1e-5) for x in a["k"]])
    rd = rounder(dtype)
    a["q"] = rd(np.repeat(np.repeat(k[key][None, None], n, 0), 2, 1))[pos0:]
    a["past_k"], a["past_v"] = (rd(k[:pos0])[:, None], a["v"][:pos0]) if pos0 else (None, None)
    a.update(k=a["k"][pos0:], v=a["v"][pos0:], gate=a["gate"][pos0:], scale=22.0 / d)
    return a


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("window,keep", [(1, 1), (64, 0), (65, 5), (63, 64), (100, 65), (128, 66), (31, 0)])
def test_one_key_stands_out_in_prompts(bamd, dtype, window, keep):
    """first tokens, page borders, far away: just inside and just outside the window and the kept tokens for the queries behind it"""
    n = 300
    for pos0 in (0, 129, 250):
        for key in sorted({0, keep - 1, keep, 62, 63, 64, 65, 127, 128, 191, 192, 250, 256, 298} - {-1}):
            a = pointed(dtype, n, pos0, window, keep, key)
            near(bamd.op_kv_attention(dtype=dtype, **a).reshape(n - pos0, -1), plain(a, n - pos0).reshape(n - pos0, -1), dtype, 3)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("window,keep", [(1, 0), (1, 1), (64, 0), (65, 5), (63, 64), (100, 65), (300, 3)])
def test_one_key_stands_out_in_decoding(bamd, dtype, window, keep):
    for last in (64, 65, 127, 128, 200, 255, 256):
        keys = {0, keep - 1, keep, last, last - 1, last - window + 1, last - window, 63, 64}
        for key in sorted(k for k in keys if 0 <= k <= last):
            a = pointed(dtype, last + 1, last, window, keep, key)
            want = plain(a, 1).reshape(1, -1)
            for splits in (1, 4):
                near(bamd.op_kv_attention(dtype=dtype, splits=splits, **a).reshape(1, -1), want, dtype, 3)


@pytest.mark.parametrize("rows,top", [(2, 2), (2, 9), (6, 90), (8, 5), (32, 200), (5, 40)])
def test_bias_of_every_distance(bamd, rows, top):
    """equal scores: the weights are the biases alone; rows far apart, so that a neighbouring row would show"""
    n, H = 260, 3
    a = case("float32", H, 1, 8, 250, n, 0, 1 << 20, 0, rows=rows, top=top)
    a.update(q=np.zeros((n, H, 8), np.float32), gate=None, v=np.concatenate([np.eye(250), np.zeros((10, 250))])[:, None].astype(np.float32), rel=(a["rel"] * 2).astype(np.float32))
    got = bamd.op_kv_attention(dtype="float32", **a)
    want = plain(a, n)
    assert np.abs(got - want).max() < 2e-5
    last = dict(a, q=a["q"][-1:], k=a["k"][-1:], v=a["v"][-1:], past_k=np.stack([[so.rms(x, 1e-5) for x in row] for row in a["k"][:-1]]), past_v=a["v"][:-1])
    assert np.abs(bamd.op_kv_attention(dtype="float32", splits=2, **last) - want[-1:]).max() < 2e-5


@pytest.mark.parametrize("dtype", DTYPES)
def test_scores_at_the_cap(bamd, dtype):
    """raw scores from nothing to a hundred times the cap"""
    for cap in (0.5, 5.0, 50.0):
        a = case(dtype, 3, 1, 16, 24, 80, 0, 1 << 20, 0, cap=cap)
        for scale in (1e-4, 0.1, 2.0, 40.0):
            a["scale"] = scale
            if dtype == "bfloat16" and scale > 1 and cap > 5:
                continue                                 # rounded operands decide which key wins
            near(bamd.op_kv_attention(dtype=dtype, **a).reshape(80, -1), plain(a, 80).reshape(80, -1), dtype, 2)


# ---- gated linear attention --------------------------------------------------------------------------------------------------------------------------------
def gla_case(H, d, dv, R, T, seed):
    r, f = np.random.default_rng(seed), lambda a: np.asarray(a, np.float32)
    return dict(q=f(r.standard_normal((T, H, d))), k=f(r.standard_normal((T, H, d))), v=f(r.standard_normal((T, H, dv))), gate=f(r.standard_normal((T, H, dv))), low=f(r.standard_normal((T, R))),
                a2=so.f32_to_bf16(r.standard_normal((H * d, R)) / np.sqrt(R)), a2b=f(r.uniform(-6, 9, H * d)), norm=f(1 + 0.3 * r.standard_normal(dv)), tau=8.0, q_scale=d ** -0.5, eps=1e-5)


def plain_gla(a, S, t0, t1):
    H, d = a["q"].shape[1:]
    ys, outs = [], []
    for t in range(t0, t1):
        al = so.gla_decay(so.bf16_to_f32(a["a2"]).astype(np.float64) @ a["low"][t] + a["a2b"], a["tau"]).reshape(H, d)
        y = np.zeros(a["v"].shape[1:])
        for h in range(H):
            S[h], y[h] = so.gla_step(S[h], al[h], a["k"][t, h].astype(np.float64), a["v"][t, h].astype(np.float64), a["q"][t, h] * a["q_scale"])
        ys.append(y)
        outs.append(np.stack([so.rms(y[h], a["eps"]) * a["norm"] * so.silu(a["gate"][t, h].astype(np.float64)) for h in range(H)]))
    return np.array(ys), np.array(outs), S


def part(a, t0, t1):
    return dict(a, **{k: a[k][t0:t1] for k in ("q", "k", "v", "gate", "low")})


@pytest.mark.parametrize("H,d,dv,R", [(1, 1, 1, 1), (3, 10, 14, 5), (5, 17, 33, 16), (2, 64, 64, 3), (2, 130, 70, 8), (1, 256, 20, 40), (40, 24, 16, 2), (1, 4, 200, 1)])
def test_gated_linear(bamd, H, d, dv, R):
    """portions from one token up, the state handed from portion to portion, channels that forget at once and channels that keep"""
    a = gla_case(H, d, dv, R, 75, H * d + dv)
    S, pos = np.zeros((H, d, dv)), 0
    gs = np.full((H, d, dv), 7, np.float32)               # what a fresh sequence finds in its place must not matter
    for n in (1, 1, 2, 7, 8, 9, 15, 32):
        y, out, S = plain_gla(a, S, pos, pos + n)
        gy, go, gs = bamd.op_gated_linear(pos0=pos, state=gs, dtype="float32", **part(a, pos, pos + n))
        assert rel(gy, y) < 1e-5 and rel(gs, S) < 1e-5, pos
        assert np.abs(go - out).max() < (3e-4 if dv < 4 else 1e-4) * (1 + np.abs(out).max()), pos      # (a norm over few columns magnifies)
        pos += n


@pytest.mark.parametrize("H,d,dv", [(2, 20, 24), (1, 130, 70), (3, 64, 16)])
@pytest.mark.parametrize("segment", [8, 16, 40, 104])
def test_gated_linear_in_segments(bamd, H, d, dv, segment):
    """a prompt scanned in segments gives what one scan gives, from a fresh state and from one that earlier tokens left"""
    a = gla_case(H, d, dv, 4, 230, 9)
    S = np.zeros((H, d, dv))
    gs = np.full((H, d, dv), 5, np.float32)
    for t0, t1 in ((0, 107), (107, 230)):
        y, out, S = plain_gla(a, S, t0, t1)
        gy, go, gs = bamd.op_gated_linear(pos0=t0, state=gs, dtype="float32", segment=segment, **part(a, t0, t1))
        assert rel(gy, y) < 1e-5 and rel(gs, S) < 1e-5
        for rows, ref in zip(gy, y):
            assert rel(rows, ref) < 1e-4


def test_a_long_memory(bamd):
    """decays next to one and strongly different ones per channel: a key of the first token is still read hundreds of tokens later, and only through the channels that keep it"""
    H, d, dv, T = 1, 8, 12, 400
    a = gla_case(H, d, dv, 1, T, 4)
    a["low"][:], a["a2b"][:] = 0, [14, 14, 14, 14, -8, -8, -8, -8]
    a["k"][1:] = 0; a["k"][0] = 1
    a["q"][:] = 0; a["q"][::2, :, :4] = 1; a["q"][1::2, :, 4:] = 1
    y, _, S = plain_gla(a, np.zeros((H, d, dv)), 0, T)
    for segment in (0, 64):
        gy, _, gs = bamd.op_gated_linear(pos0=0, state=np.zeros((H, d, dv)), dtype="float32", segment=segment, **a)
        assert rel(gy[::2], y[::2]) < 1e-4 and np.abs(gy[101::2]).max() < 1e-6 and rel(gs, S) < 1e-4


@pytest.mark.parametrize("dtype", DTYPES)
def test_head_norm_and_gate(bamd, dtype):
    a = gla_case(3, 12, 37, 2, 20, 8)
    _, out, _ = plain_gla(a, np.zeros((3, 12, 37)), 0, 20)
    _, go, _ = bamd.op_gated_linear(pos0=0, state=np.zeros((3, 12, 37)), dtype=dtype, out_scale=-0.6, **a)
    near(go.reshape(20, -1), -0.6 * out.reshape(20, -1), dtype)
    gy, go, _ = bamd.op_gated_linear(pos0=0, state=np.zeros((3, 12, 37)), dtype=dtype, **dict(a, gate=None))
    near(go, np.stack([[so.rms(y, 1e-5) * a["norm"] for y in row] for row in gy.astype(np.float64)]), dtype)
