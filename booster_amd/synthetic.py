"""Random weights for configured layer stacks (config.json + model.safetensors) of any size: for benchmarks and probes, the counterpart of gguf.write_synthetic_llama."""
import json
import math
import os
import struct

import numpy as np


def stack_tensors(cfg, bias_rows=32, decay_rank=16):
    """name -> (shape, kind); kind: a standard deviation, or the range of a uniform vector.  bias_rows, decay_rank: sizes that only tensors have"""
    E, V = cfg["width"], cfg["vocab"]
    sandwich = cfg["architecture"] == "Mafurax"
    lin = lambda o, i: ((o, i), 1 / math.sqrt(i))
    if sandwich:
        t = {"embed": ((V, E), 1.0), "final.norm": ((E,), (0.8, 1.2))}
    else:
        t = {"embed": ((V, E), 1.0 / cfg["embedding"]["scale"]), "pos": ((cfg["max_positions"], E), 0.3), "final.norm": ((), (1, 1)), "head": ((V, E), 1 / math.sqrt(E))}
    for n, ly in enumerate(cfg["layers"]):
        p, mx = "l%d." % n, ly["mixer"]
        if ly["type"] == "mamba2":
            H = mx["heads"]
            inner, gn = H * mx["vdim"], 2 * mx["groups"] * mx["state"]
            m = {"in": lin(2 * inner + gn + H, E), "conv": lin(inner + gn, mx["conv"]), "conv.b": ((inner + gn,), 0.1), "dt_bias": ((H,), (-4, 0)), "A_log": ((H,), (-1, 1.5)), "D": ((H,), 1.0),
                 "norm": ((inner,), (0.8, 1.2)), "o": lin(E, inner)}
        elif ly["type"] == "latent_attention":
            H, R, d, dv = mx["heads"], mx["kv_rank"], mx["dim"], mx["vdim"]
            m = {"q": lin(H * d, E), "dkv": lin(R, E), "dkv.norm": ((R,), (0.8, 1.2)), "uk": lin(H * d, R), "uv": lin(H * dv, R), "sink": ((H,), 1.0), "g": lin(H, E), "o": lin(E, H * dv)}
        else:
            a, b = mx["left"], mx["right"]
            H, G, d, dv = a["heads"], a["kv_heads"], a["dim"], a["vdim"]
            m = {"left.q": lin(H * d, E), "left.k": lin(G * d, E), "left.v": lin(G * dv, E), "left.rel": ((bias_rows, H), 1.0), "left.g": lin(H, E), "left.o": lin(E, H * dv)}
            H, d, dv = b["heads"], b["dim"], b["vdim"]
            m.update({"right.q": lin(H * d, E), "right.k": lin(H * d, E), "right.v": lin(H * dv, E), "right.g": lin(H * dv, E), "right.o": lin(E, H * dv), "right.norm": ((dv,), (0.8, 1.2)),
                      "right.a1": lin(decay_rank, E), "right.a2": lin(H * d, decay_rank), "right.a2.b": ((H * d,), (-3, 6))})
        t.update({p + "mix." + k: v for k, v in m.items()})
        F = ly["mlp"]["ff"] if ly["mlp"] is not None else 0
        if sandwich:
            t.update({p + "norm1": ((E,), (0.8, 1.2)), p + "norm1b": ((E,), (0.8, 1.2)), p + "ls1": ((E,), (0.4, 0.6))})
            if F:
                t.update({p + "norm2": ((E,), (0.8, 1.2)), p + "norm2b": ((E,), (0.8, 1.2)), p + "ls2": ((E,), (0.4, 0.6)), p + "mlp.gate": lin(F, E), p + "mlp.up": lin(F, E), p + "mlp.down": lin(E, F)})
            continue
        t[p + "norm1"] = ((), (0.5, 0.5)); t[p + "shift"] = ((E,), (0, 1))
        if F:
            t.update({p + "norm2": ((), (0.5, 0.5)), p + "mlp.up": lin(F, E), p + "mlp.down": lin(E, F), p + "mlp.act": ((4,), 0.5)})
    return t


def write_synthetic_stack(folder, cfg, seed=7):
    """matrices are cut from one block of normal values at a random place (no two rows of a matrix alike); writes a few GB in seconds"""
    r = np.random.default_rng(seed)
    base = r.standard_normal((1 << 22) + 12345).astype(np.float32)
    os.makedirs(folder, exist_ok=True)
    with open(os.path.join(folder, "config.json"), "w") as f:
        json.dump(cfg, f)
    tensors = stack_tensors(cfg)
    head, at = {}, 0
    for k, (shape, _) in tensors.items():
        n = 2 * int(np.prod(shape, dtype=np.int64))
        head[k] = {"dtype": "BF16", "shape": list(shape), "data_offsets": [at, at + n]}
        at += n
    h = json.dumps(head).encode()
    h += b" " * (-len(h) % 8)
    with open(os.path.join(folder, "model.safetensors"), "wb") as f:
        f.write(struct.pack("<Q", len(h)) + h)
        for shape, kind in tensors.values():
            n = int(np.prod(shape, dtype=np.int64))
            if isinstance(kind, tuple):
                v = r.uniform(kind[0], kind[1], n).astype(np.float32)
                f.write((v.view(np.uint32) >> 16).astype(np.uint16).tobytes())
                continue
            b = ((base * np.float32(kind)).view(np.uint32) >> 16).astype(np.uint16)
            off = int(r.integers(0, b.size))
            b = np.concatenate([b[off:], b[:off]])
            for i in range(0, n, b.size):
                f.write(b[:min(b.size, n - i)].tobytes())
    return sum(2 * int(np.prod(s, dtype=np.int64)) for s, _ in tensors.values())
