"""Plain numpy statement of the configured layer stacks the product runs (booster_amd/csrc/bamd_stack*.{cpp,hip}): one function per mechanism, one token
or one score row at a time, float64 throughout.  Test infrastructure: it shares no code with the product path and is written for reading, not for speed.

A model is (cfg, w): cfg the parsed config.json, w a dict of tensor name -> numpy array.  A sequence's state is a plain dict that `forward` creates and
advances; feeding the tokens in any number of portions gives the same numbers.
"""
import json
import math
import struct

import numpy as np


# ---- files ---------------------------------------------------------------------------------------------------------------------------------
def bf16_to_f32(u16):
    return (np.atleast_1d(np.asarray(u16, np.uint32)) << 16).view(np.float32).reshape(np.shape(u16))


def f32_to_bf16(x):
    """round to nearest even"""
    u = np.ascontiguousarray(x, np.float32).view(np.uint32)
    return ((u + 0x7fff + ((u >> 16) & 1)) >> 16).astype(np.uint16).reshape(np.shape(x))


def round_bf16(x):
    return bf16_to_f32(f32_to_bf16(x))


def read_safetensors(path):
    raw = open(path, "rb").read()
    n = struct.unpack("<Q", raw[:8])[0]
    head = json.loads(raw[8:8 + n])
    out = {}
    for name, t in head.items():
        if name == "__metadata__":
            continue
        a, b = t["data_offsets"]
        buf = raw[8 + n + a:8 + n + b]
        if t["dtype"] == "BF16":
            v = bf16_to_f32(np.frombuffer(buf, np.uint16))
        else:
            v = np.frombuffer(buf, {"F32": np.float32, "F16": np.float16, "I32": np.int32}[t["dtype"]])
        out[name] = v.reshape(t["shape"])
    return out


# ---- mechanisms ----------------------------------------------------------------------------------------------------------------------------
def rms(x, eps):
    return x / np.sqrt(np.mean(x * x) + eps)


def scalar_norm(x, g, eps):
    return rms(x, eps) * g


def sigmoid(x):
    return 1.0 / (1.0 + np.exp(-x))


def silu(x):
    return x * sigmoid(x)


def softplus(x):
    return np.logaddexp(0.0, x)


def token_shift(h, prev, mu):
    """every coordinate moves towards the previous token's value by its own share mu"""
    return h + (prev - h) * mu


def causal_conv(taps, bias, history, x):
    """history: the inputs of the taps - 1 tokens before x, oldest first; returns the filtered token and the new history"""
    rows = np.concatenate([history, x[None]], 0)
    return np.sum(taps.T * rows, 0) + bias, rows[1:]


def ssd_step(S, dt, A_log, D, B, C, x):
    """one token of one head: S [N, vdim] decays by exp(-exp(A_log) dt), takes dt B x^T and is read by C"""
    S = math.exp(-math.exp(A_log) * dt) * S + dt * np.outer(B, x)
    return S, S.T @ C + D * x


def grouped_norm(y, groups, g, eps):
    parts = np.split(y, groups)
    return np.concatenate([rms(p, eps) for p in parts]) * g


def mamba2(h, st, mx, w, eps):
    """one token through the state-space mixer; st = {conv, S}"""
    H, P, N, G, K = mx["heads"], mx["vdim"], mx["state"], mx["groups"], mx["conv"]
    inner = H * P
    if not st:
        st["conv"] = np.zeros((K - 1, inner + 2 * G * N))
        st["S"] = np.zeros((H, N, P))
    z, xbc, dt = np.split(w["in"] @ h, [inner, 2 * inner + 2 * G * N])
    xbc, st["conv"] = causal_conv(w["conv"], w["conv.b"], st["conv"], xbc)
    x, B, C = np.split(silu(xbc), [inner, inner + G * N])
    dt = softplus(dt + w["dt_bias"])
    y = np.zeros(inner)
    for i in range(H):
        g = i // (H // G)
        st["S"][i], y[i * P:(i + 1) * P] = ssd_step(st["S"][i], dt[i], w["A_log"][i], w["D"][i], B[g * N:(g + 1) * N], C[g * N:(g + 1) * N], x[i * P:(i + 1) * P])
    return w["o"] @ grouped_norm(y * silu(z), mx["norm_groups"], w["norm"], eps)


def sink_softmax(s, sink):
    """weights of the keys when the denominator also holds exp(sink)"""
    m = max(np.max(s), sink)
    e = np.exp(s - m)
    return e / (np.sum(e) + math.exp(sink - m))


def latent_attention(h, st, mx, w, eps):
    """one token through the latent attention; st = {c: the latents so far}"""
    H, d, dv = mx["heads"], mx["dim"], mx["vdim"]
    c = rms(w["dkv"] @ h, eps) * w["dkv.norm"]
    st["c"] = np.concatenate([st["c"], c[None]], 0) if st else c[None]
    k = (st["c"] @ w["uk"].T).reshape(-1, H, d)
    v = (st["c"] @ w["uv"].T).reshape(-1, H, dv)
    q = (w["q"] @ h).reshape(H, d)
    gate = sigmoid(w["g"] @ h)
    o = np.zeros((H, dv))
    for i in range(H):
        o[i] = gate[i] * (sink_softmax((k[:, i] @ q[i]) * mx["scale"], w["sink"][i]) @ v[:, i])
    return w["o"] @ o.reshape(-1)


def poly_norm(z, a, b, c, e, eps):
    return a * rms(z, eps) + b * rms(z ** 2, eps) + c * rms(z ** 3, eps) + e


def dense_mlp(x, w, eps):
    return w["down"] @ poly_norm(w["up"] @ x, *w["act"], eps)


def layer_norm(x, w, eps):
    d = x - np.mean(x)
    return d / np.sqrt(np.mean(d * d) + eps) * w


def distance_bucket(n, rows, top):
    """the first half of the rows: one distance each; the second half: logarithmic steps up to `top`, the last row beyond"""
    half = rows // 2
    if n < half:
        return n
    return min(rows - 1, half + math.floor(math.log(n / half) / math.log(top / half) * (rows - half)))


def visible(i, j, mask):
    """position i sees position j: behind it, and within the window or among the first tokens that are kept"""
    return j <= i and (i - j < mask["size"] or j < mask["keep_first"])


def softcap(s, cap):
    return cap * np.tanh(s / cap)


def biased_softmax(s, bias):
    e = np.exp(s + bias - np.max(s + bias))
    return e / np.sum(e)


def window_attention(h, st, mx, w, eps):
    """one token through grouped-query attention over a window and the first tokens: unit-RMS queries and keys, capped scores, a bias per distance and head, a gate per
    head; st = {k, v: every key and value so far}"""
    H, G, d, dv = mx["heads"], mx["kv_heads"], mx["dim"], mx["vdim"]
    q = (w["q"] @ h).reshape(H, d)
    k = np.stack([rms(x, eps) for x in (w["k"] @ h).reshape(G, d)])
    v = (w["v"] @ h).reshape(G, dv)
    st["k"] = st.get("k", []) + [k]
    st["v"] = st.get("v", []) + [v]
    i = len(st["k"]) - 1
    seen = [j for j in range(i + 1) if visible(i, j, mx["mask"])]
    buckets = [distance_bucket(i - j, len(w["rel"]), mx["bias_max"]) for j in seen]
    gate = sigmoid(w["g"] @ h)
    K, V = np.stack([st["k"][j] for j in seen]), np.stack([st["v"][j] for j in seen])
    o = np.zeros((H, dv))
    for a in range(H):
        g = a // (H // G)
        s = softcap((K[:, g] @ rms(q[a], eps)) * mx["scale"], mx["softcap"])
        o[a] = gate[a] * (biased_softmax(s, w["rel"][buckets, a]) @ V[:, g])
    return w["o"] @ o.reshape(-1)


def gla_decay(z, tau):
    return sigmoid(z) ** (1.0 / tau)


def gla_step(S, alpha, k, v, q):
    """one token of one head: every row (key channel) of S [dim, vdim] decays by its own alpha, takes k v^T and is read by q"""
    S = alpha[:, None] * S + np.outer(k, v)
    return S, S.T @ q


def gated_linear(h, st, mx, w, eps):
    """one token through gated linear attention; st = {S}"""
    H, d, dv = mx["heads"], mx["dim"], mx["vdim"]
    if not st:
        st["S"] = np.zeros((H, d, dv))
    q, k, v = (w["q"] @ h).reshape(H, d) / math.sqrt(d), (w["k"] @ h).reshape(H, d), (w["v"] @ h).reshape(H, dv)
    alpha = gla_decay(w["a2"] @ (w["a1"] @ h) + w["a2.b"], mx["tau"]).reshape(H, d)
    o = np.zeros((H, dv))
    for a in range(H):
        st["S"][a], y = gla_step(st["S"][a], alpha[a], k[a], v[a], q[a])
        o[a] = rms(y, eps) * w["norm"]
    return w["o"] @ (o.reshape(-1) * silu(w["g"] @ h))


def parallel(h, st, mx, w, eps):
    """both mixers read the same input; their results are added with a scale each"""
    part = lambda side: {k[len(side):]: v for k, v in w.items() if k.startswith(side)}
    st.setdefault("left", {}); st.setdefault("right", {})
    return mx["left_scale"] * window_attention(h, st["left"], mx["left"], part("left."), eps) + mx["right_scale"] * gated_linear(h, st["right"], mx["right"], part("right."), eps)


def clamped_glu(gate, up, limit):
    g, u = np.minimum(gate, limit), np.clip(up, -limit, limit)
    return g * sigmoid(1.702 * g) * (u + 1)


def glu_mlp(x, w, limit):
    return w["down"] @ clamped_glu(w["gate"] @ x, w["up"] @ x, limit)


MIXERS = {"mamba2": mamba2, "latent_attention": latent_attention, "parallel": parallel}


# ---- model ---------------------------------------------------------------------------------------------------------------------------------
class StackModel:
    def __init__(self, cfg, w):
        self.cfg = cfg
        self.w = {k: np.asarray(v, np.float64) for k, v in w.items()}
        self.part = lambda prefix: {k[len(prefix):]: v for k, v in self.w.items() if k.startswith(prefix)}
        self.layers = []
        for i, ly in enumerate(cfg["layers"]):
            p = "l%d." % i
            self.layers.append((ly, self.part(p + "mix."), self.part(p + "mlp."), self.part(p)))

    @classmethod
    def load(cls, folder):
        return cls(json.load(open(folder + "/config.json")), read_safetensors(folder + "/model.safetensors"))

    def tupitar_layer(self, x, ly, mix, mlp, top, st, eps):
        """one number scales the norm of every sublayer's output; mixers read a blend of this token and the previous one"""
        h = token_shift(x, st["prev"], top["shift"])
        st["prev"] = x
        x = x + scalar_norm(MIXERS[ly["type"]](h, st["mix"], ly["mixer"], mix, eps), top["norm1"], eps)
        if ly["mlp"] is not None:
            x = x + scalar_norm(dense_mlp(x, mlp, eps), top["norm2"], eps)
        return x

    def mafurax_layer(self, x, ly, mix, mlp, top, st, eps):
        """a layer norm in front of every sublayer, another on its output, and a scale per element on that"""
        x = x + layer_norm(MIXERS[ly["type"]](layer_norm(x, top["norm1"], eps), st["mix"], ly["mixer"], mix, eps), top["norm1b"], eps) * top["ls1"]
        if ly["mlp"] is not None:
            x = x + layer_norm(glu_mlp(layer_norm(x, top["norm2"], eps), mlp, ly["mlp"]["limit"]), top["norm2b"], eps) * top["ls2"]
        return x

    def new_state(self):
        return {"n": 0, "layers": [{"prev": np.zeros(self.cfg["width"]), "mix": {}} for _ in self.layers]}

    def token(self, tok, state, trace=None):
        """one token; returns its logits and advances the state"""
        eps = self.cfg["norm"]["eps"]
        mafurax = self.cfg["architecture"] == "Mafurax"
        x = self.w["embed"][tok] if mafurax else self.w["embed"][tok] * self.cfg["embedding"]["scale"] + self.w["pos"][state["n"]]
        for (ly, mix, mlp, top), st in zip(self.layers, state["layers"]):
            x = (self.mafurax_layer if mafurax else self.tupitar_layer)(x, ly, mix, mlp, top, st, eps)
            if trace is not None:
                trace.append(x)
        state["n"] += 1
        if mafurax:
            return self.w["embed"] @ layer_norm(x, self.w["final.norm"], eps) * self.cfg["logit_scale"]
        return self.w["head"] @ scalar_norm(x, self.w["final.norm"], eps)

    def forward(self, tokens, state=None, trace=None):
        """logits [n, vocab] of `tokens` behind `state` (a fresh sequence when None)"""
        state = self.new_state() if state is None else state
        return np.stack([self.token(int(t), state, trace) for t in tokens])


# ---- small random models ---------------------------------------------------------------------------------------------------------------------
def random_model(cfg, seed, rows=None):
    """bfloat16-representable weights of unit gain; decays, biases and gates spread so that no mechanism is idle"""
    r = np.random.default_rng(seed)
    E, V = cfg["width"], cfg["vocab"]
    lin = lambda o, i, s=1.0: r.standard_normal((o, i)) * s / math.sqrt(i)
    mafurax = cfg["architecture"] == "Mafurax"
    if mafurax:
        w = {"embed": lin(V, E, math.sqrt(E)), "final.norm": 1 + 0.2 * r.standard_normal(E)}
    else:
        w = {"embed": r.standard_normal((V, E)) / cfg["embedding"]["scale"], "pos": r.standard_normal((cfg["max_positions"], E)) * 0.3,
             "final.norm": np.array(1.1), "head": lin(V, E)}
    for i, ly in enumerate(cfg["layers"]):
        p, mx = "l%d." % i, ly["mixer"]
        m = {}
        if ly["type"] == "mamba2":
            H, P, N, G, K = mx["heads"], mx["vdim"], mx["state"], mx["groups"], mx["conv"]
            ch = H * P + 2 * G * N
            m = {"in": lin(H * P + ch + H, E), "conv": r.standard_normal((ch, K)) / math.sqrt(K), "conv.b": r.standard_normal(ch) * 0.1,
                 "dt_bias": r.uniform(-4, 0, H), "A_log": r.uniform(-1, 1.5, H), "D": r.standard_normal(H), "norm": 1 + 0.2 * r.standard_normal(H * P), "o": lin(E, H * P)}
        elif ly["type"] == "latent_attention":
            H, d, dv, R = mx["heads"], mx["dim"], mx["vdim"], mx["kv_rank"]
            m = {"q": lin(H * d, E), "dkv": lin(R, E), "dkv.norm": 1 + 0.2 * r.standard_normal(R), "uk": lin(H * d, R, 2.0), "uv": lin(H * dv, R), "sink": r.standard_normal(H) + 1,
                 "g": lin(H, E), "o": lin(E, H * dv)}
        else:
            # sizes that the configuration does not name: bias rows, rank of the decays
            a, b = mx["left"], mx["right"]
            B, R = (rows or {}).get("rel", 8), (rows or {}).get("rank", 5)
            H, G, d, dv = a["heads"], a["kv_heads"], a["dim"], a["vdim"]
            m = {"left.q": lin(H * d, E), "left.k": lin(G * d, E), "left.v": lin(G * dv, E), "left.rel": r.standard_normal((B, H)), "left.g": lin(H, E), "left.o": lin(E, H * dv)}
            H, d, dv = b["heads"], b["dim"], b["vdim"]
            m.update({"right.q": lin(H * d, E), "right.k": lin(H * d, E, 0.5), "right.v": lin(H * dv, E), "right.g": lin(H * dv, E), "right.o": lin(E, H * dv), "right.norm": 1 + 0.2 * r.standard_normal(dv),
                      "right.a1": lin(R, E), "right.a2": lin(H * d, R, 2.0), "right.a2.b": r.uniform(-3, 6, H * d)})
        w.update({p + "mix." + k: v for k, v in m.items()})
        if mafurax:
            n = lambda: 1 + 0.2 * r.standard_normal(E)
            w.update({p + "norm1": n(), p + "norm1b": n(), p + "ls1": r.uniform(0.3, 0.9, E) * r.choice([-1, 1], E)})
            if ly["mlp"] is not None:
                F = ly["mlp"]["ff"]
                w.update({p + "norm2": n(), p + "norm2b": n(), p + "ls2": r.uniform(0.3, 0.9, E), p + "mlp.gate": lin(F, E), p + "mlp.up": lin(F, E), p + "mlp.down": lin(E, F)})
            continue
        w[p + "norm1"] = np.array(r.uniform(0.4, 0.9)); w[p + "shift"] = r.uniform(0, 1, E)
        if ly["mlp"] is not None:
            F = ly["mlp"]["ff"]
            w[p + "norm2"] = np.array(r.uniform(0.4, 0.9))
            w.update({p + "mlp.up": lin(F, E), p + "mlp.down": lin(E, F), p + "mlp.act": r.standard_normal(4) * np.array([1, 0.5, 0.5, 0.2])})
    return {k: round_bf16(v) for k, v in w.items()}


def write_model(folder, cfg, w):
    """config.json + model.safetensors (bfloat16) of a model"""
    import os
    os.makedirs(folder, exist_ok=True)
    with open(os.path.join(folder, "config.json"), "w") as f:
        json.dump(cfg, f)
    head, blobs, at = {}, [], 0
    for k, v in w.items():
        b = f32_to_bf16(np.asarray(v, np.float32)).tobytes()
        head[k] = {"dtype": "BF16", "shape": list(np.shape(v)), "data_offsets": [at, at + len(b)]}
        blobs.append(b); at += len(b)
    h = json.dumps(head).encode()
    h += b" " * (-len(h) % 8)
    with open(os.path.join(folder, "model.safetensors"), "wb") as f:
        f.write(struct.pack("<Q", len(h)) + h + b"".join(blobs))
