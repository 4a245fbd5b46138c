"""CPU: the configured layer stacks without a device — the plain statement of the mechanisms against itself, what a fault in it would change, configuration and weight
files, the registry, and the request scheduler."""
import json
import os

import numpy as np
import pytest

from oracle import stack_oracle as so
from stack_cases import CONFIGS, tokens, weights


def rel(a, b):
    a, b = np.asarray(a, np.float64), np.asarray(b, np.float64)
    return float(np.sqrt(np.mean((a - b) ** 2) / np.mean(b ** 2)))


@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_portions_of_the_plain_statement(name):
    cfg = CONFIGS[name]
    m = so.StackModel(cfg, weights(name, 1))
    t = tokens(cfg, 21, 2)
    whole = m.forward(t)
    st = m.new_state()
    parts = np.concatenate([m.forward(t[a:b], st) for a, b in ((0, 2), (2, 3), (3, 11), (11, 21))])
    assert rel(parts, whole) < 1e-12


class Rounded:
    """a matrix whose products round their operand to bfloat16"""

    def __init__(self, w):
        self.w = w

    def __matmul__(self, x):
        return self.w @ so.round_bf16(x).astype(np.float64)

    def __getitem__(self, i):
        return self.w[i]


@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_rounding_alone_stays_small(name):
    """what bfloat16 operands cost in the test models: less than half of the tolerance the GPU tests allow, at every position"""
    cfg = CONFIGS[name]
    m = so.StackModel(cfg, weights(name))
    t = tokens(cfg, 150, 1)
    exact = m.forward(t)
    for ly, mix, mlp, _ in m.layers:
        for part, keys in ((mix, ("in", "q", "dkv", "g", "o", "left.q", "left.k", "left.v", "left.g", "left.o", "right.q", "right.k", "right.v", "right.g", "right.o", "right.a1")), (mlp, ("gate", "up", "down"))):
            part.update({k: Rounded(part[k]) for k in keys if k in part})
    head = "head" if "head" in m.w else "embed"
    m.w[head] = Rounded(m.w[head])
    e = np.sqrt(((m.forward(t) - exact) ** 2).mean(-1) / (exact ** 2).mean(-1))
    assert 0.001 < e.max() < 0.015


FAULTS = {
    "no sink": ("sink_softmax", lambda s, sink: np.exp(s - s.max()) / np.exp(s - s.max()).sum()),
    "shift from the token itself": ("token_shift", lambda h, prev, mu: h),
    "shift the other way round": ("token_shift", lambda h, prev, mu: prev + (h - prev) * mu),
    "taps reversed": ("causal_conv", lambda taps, bias, hist, x: (np.sum(taps.T[::-1] * np.concatenate([hist, x[None]]), 0) + bias, np.concatenate([hist, x[None]])[1:])),
    "one norm group": ("grouped_norm", lambda y, groups, g, eps: so.rms(y, eps) * g),
    "no constant term": ("poly_norm", lambda z, a, b, c, e, eps: a * so.rms(z, eps) + b * so.rms(z ** 2, eps) + c * so.rms(z ** 3, eps)),
    "step size not in the input": ("ssd_step", lambda S, dt, A, D, B, C, x: ((lambda n: (n, n.T @ C + D * x))(np.exp(-np.exp(A) * dt) * S + np.outer(B, x)))),
    "state not carried": ("ssd_step", lambda S, dt, A, D, B, C, x: ((lambda n: (n, n.T @ C + D * x))(dt * np.outer(B, x)))),
}


SIDE_FAULTS = {
    "window one longer": ("visible", lambda i, j, m: j <= i and (i - j <= m["size"] or j < m["keep_first"])),
    "window one shorter": ("visible", lambda i, j, m: j <= i and (i - j < m["size"] - 1 or j == i or j < m["keep_first"])),
    "first tokens not kept": ("visible", lambda i, j, m: j <= i and i - j < m["size"]),
    "one first token too many": ("visible", lambda i, j, m: j <= i and (i - j < m["size"] or j <= m["keep_first"])),
    "scores not capped": ("softcap", lambda s, cap: s),
    "bias in front of the cap": ("biased_softmax", lambda s, bias: (lambda e: e / e.sum())(np.exp(6 * np.tanh((s + bias) / 6)))),
    "no bias": ("biased_softmax", lambda s, bias: np.exp(s) / np.exp(s).sum()),
    "distances one off": ("distance_bucket", lambda n, rows, top, f=so.distance_bucket: f(n + 1, rows, top)),
    "no logarithmic steps": ("distance_bucket", lambda n, rows, top: min(n, rows - 1)),
    "no tau": ("gla_decay", lambda z, tau: so.sigmoid(z)),
    "one decay per head": ("gla_step", lambda S, al, k, v, q: ((lambda n: (n, n.T @ q))(al.mean() * S + np.outer(k, v)))),
    "decay on the columns": ("gla_step", lambda S, al, k, v, q: ((lambda n: (n, n.T @ q))(np.resize(al, len(v))[None] * S + np.outer(k, v)))),
    "own token not decayed in": ("gla_step", lambda S, al, k, v, q: (al[:, None] * S + np.outer(k, v), (al[:, None] * S).T @ q)),
    "state not carried": ("gla_step", lambda S, al, k, v, q: (np.outer(k, v), np.outer(k, v).T @ q)),
    "mean not taken off": ("layer_norm", lambda x, w, eps: so.rms(x, eps) * w),
    "no one behind up": ("clamped_glu", lambda g, u, limit: (lambda a: a * so.sigmoid(1.702 * a) * np.clip(u, -limit, limit))(np.minimum(g, limit))),
    "gate clamped below": ("clamped_glu", lambda g, u, limit: (lambda a: a * so.sigmoid(1.702 * a) * (np.clip(u, -limit, limit) + 1))(np.clip(g, -limit, limit))),
    "up not clamped": ("clamped_glu", lambda g, u, limit: (lambda a: a * so.sigmoid(1.702 * a) * (u + 1))(np.minimum(g, limit))),
}


@pytest.mark.parametrize("name,fault", [("odd", f) for f in sorted(FAULTS)] + [("side", f) for f in sorted(SIDE_FAULTS)])
def test_a_fault_shows_in_the_logits(name, fault, monkeypatch):
    """every mechanism matters in the test models: a fault planted in the plain statement moves the logits far beyond the tolerances of the GPU tests"""
    cfg = CONFIGS[name]
    w = weights(name, 3)
    t = tokens(cfg, 70 if name == "side" else 24, 4)
    good = so.StackModel(cfg, w).forward(t)
    monkeypatch.setattr(so, *(FAULTS if name == "odd" else SIDE_FAULTS)[fault])
    assert rel(so.StackModel(cfg, w).forward(t), good) > (0.1 if name == "odd" else 0.02)


def test_buckets():
    """the distances of every row: exact ones, then steps that grow, the last row from its start to infinity"""
    got = [so.distance_bucket(n, 8, 32) for n in range(40)]
    assert got[:4] == [0, 1, 2, 3] and got[4:7] == [4, 4, 4] and got[31:] == [7] * 9 and got == sorted(got)
    assert [so.distance_bucket(n, 2, 9) for n in range(4)] == [0, 1, 1, 1]
    m = {"size": 3, "keep_first": 2}
    assert [[j for j in range(9) if so.visible(i, j, m)] for i in (0, 2, 4, 5, 8)] == [[0], [0, 1, 2], [0, 1, 2, 3, 4], [0, 1, 3, 4, 5], [0, 1, 6, 7, 8]]


def test_weights_survive_the_file(tmp_path):
    cfg = CONFIGS["ones"]
    w = weights("ones", 5)
    so.write_model(str(tmp_path / "m"), cfg, w)
    m = so.StackModel.load(str(tmp_path / "m"))
    assert m.cfg == cfg and set(m.w) == set(w) and all(np.array_equal(m.w[k], np.asarray(w[k], np.float64)) for k in w)


# ---- the product's side that needs no device -------------------------------------------------------------------------------------------------------------
def load_error(path, **kw):
    import booster_amd
    with pytest.raises(booster_amd.BamdError) as e:
        booster_amd.Model(str(path), **kw)
    return str(e.value)


def test_registry_and_configuration_errors(tmp_path):
    cfg = CONFIGS["ones"]
    w = so.random_model(cfg, 6)
    d = tmp_path / "m"
    so.write_model(str(d), dict(cfg, architecture="Nope"), w)
    assert all(n in load_error(d) for n in ("Tupitar", "Mafurax", "Nope"))
    so.write_model(str(d), {k: v for k, v in cfg.items() if k != "width"}, w)
    assert "width" in load_error(d)
    so.write_model(str(d), dict(cfg, layers=[]), w)
    assert "layers" in load_error(d)
    (d / "config.json").write_text('{"architecture": "Tupitar", ')
    assert "config.json" in load_error(d)
    (d / "config.json").write_text(json.dumps(cfg))
    blob = (d / "model.safetensors").read_bytes()
    (d / "model.safetensors").write_bytes(blob[:len(blob) // 2])
    assert "does not fit" in load_error(d)
    (d / "model.safetensors").write_bytes(b"\xff" * 16)
    assert "header" in load_error(d)
    os.remove(d / "model.safetensors")
    assert "cannot open" in load_error(d)
    os.remove(d / "config.json")
    assert "cannot open" in load_error(d)
    from conftest import GOLDEN
    assert "dtype" in load_error(os.path.join(GOLDEN, "tiny_a.gguf"), dtype="float32")


class FakeContext:
    """counts what it is given: the 'logits' of a place point at (token + length of the sequence) % vocab"""

    def __init__(self, n_ctx, n_seq, vocab=11):
        self.n_ctx, self.n_seq, self.vocab, self.seqs, self.widest = n_ctx, n_seq, vocab, {}, 0

    def decode_batch(self, entries):
        out = []
        for seq, t, want in entries:
            q = self.seqs.setdefault(seq, [])
            for i, tok in enumerate(t):
                q.append(tok)
                if i in want:
                    l = np.zeros(self.vocab, np.float32); l[(tok + len(q)) % self.vocab] = 1
                    out.append(l)
        assert sum((len(q) + 63) // 64 for q in self.seqs.values()) <= (self.n_ctx + 63) // 64 + self.n_seq - 1, "pages"
        self.widest = max(self.widest, len(entries))
        return np.array(out)

    def seq_free(self, seq):
        self.seqs.pop(seq, None)


def alone(prompt, n, vocab=11):
    q, out = list(prompt), []
    for _ in range(n):
        out.append((q[-1] + len(q)) % vocab)
        q.append(out[-1])
    return out


@pytest.mark.parametrize("n_seq,n_ctx", [(1, 128), (3, 192), (8, 1024)])
def test_scheduler_serves_every_request(n_seq, n_ctx):
    from booster_amd.scheduler import Scheduler
    prompts = [[int(t) for t in np.random.default_rng(i).integers(0, 11, 1 + 7 * i % 60)] for i in range(9)]
    c = FakeContext(n_ctx, n_seq)
    s = Scheduler(c)
    assert s.generate(prompts, 17) == [alone(p, 17) for p in prompts]
    assert not c.seqs and not s.slot and len(s.free) == n_seq and c.widest == min(n_seq, c.widest) and (n_seq == 1 or c.widest > 1)
    out = s.generate(prompts, 17, stop=(3,))
    assert all(o == a[:a.index(3) + 1] if 3 in a else o == a for o, a in zip(out, (alone(p, 17) for p in prompts)))


def test_scheduler_refuses_what_does_not_fit():
    import booster_amd
    from booster_amd.scheduler import Scheduler
    s = Scheduler(FakeContext(64, 1))
    with pytest.raises(booster_amd.BamdError):
        s.generate([[1] * 60], 8)
    s.step([("a", [1], [])])
    with pytest.raises(booster_amd.BamdError):
        s.step([("b", [1], [])])
    s.close("a")
    s.step([("b", [1], [])])
