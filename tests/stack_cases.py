"""Small configurations of the layer-stack designs (Tupitar, Mafurax) for the tests: sizes that are no multiples of any tile, values that are 1, and layers that differ from one another."""
import numpy as np


def mamba(heads, vdim, state, groups, norm_groups, conv, ff=None):
    return {"type": "mamba2", "mixer": dict(heads=heads, vdim=vdim, state=state, groups=groups, norm_groups=norm_groups, conv=conv), "mlp": None if ff is None else {"kind": "dense", "ff": ff}}


def latent(heads, dim, vdim, kv_rank, scale, ff=None):
    return {"type": "latent_attention", "mixer": dict(heads=heads, dim=dim, vdim=vdim, kv_rank=kv_rank, scale=scale), "mlp": None if ff is None else {"kind": "dense", "ff": ff}}


def config(width, vocab, layers, max_positions=700, scale=3.0, eps=1e-5):
    return {"architecture": "Tupitar", "vocab": vocab, "width": width, "max_positions": max_positions, "embedding": {"scale": scale}, "norm": {"eps": eps}, "layers": layers}


def attend(heads, kv_heads, dim, vdim, scale, softcap, bias_max, size, keep_first):
    return dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, scale=scale, softcap=softcap, bias_max=bias_max, mask=dict(size=size, keep_first=keep_first))


def parallel(left, left_scale, right, right_scale, ff=None, limit=None):
    """right: (heads, dim, vdim, tau)"""
    return {"type": "parallel", "mixer": dict(left=left, left_scale=left_scale, right=dict(zip(("heads", "dim", "vdim", "tau"), right)), right_scale=right_scale),
            "mlp": None if ff is None else {"kind": "dense", "ff": ff, "limit": limit}}


def mafurax(width, vocab, layers, logit_scale=0.7, eps=1e-5):
    return {"architecture": "Mafurax", "vocab": vocab, "width": width, "logit_scale": logit_scale, "norm": {"eps": eps}, "layers": layers}


CONFIGS = {
    # both mixers, nothing a multiple of 16, a layer without a feed-forward
    "odd": config(75, 131, [mamba(3, 20, 24, 1, 5, 3, ff=90), latent(3, 24, 40, 36, 0.31, ff=101), mamba(4, 10, 12, 4, 2, 2), latent(5, 33, 12, 20, 0.2)]),
    # heads, groups, taps and ranks of 1 where that is possible
    "ones": config(48, 67, [latent(1, 16, 16, 8, 0.25, ff=40), mamba(1, 16, 8, 1, 1, 1, ff=33), mamba(2, 8, 1, 2, 1, 4)], scale=1.0),
    # more than 16 heads, more than 64 value columns, more than 64 states, a wide latent
    "wide": config(160, 259, [latent(18, 32, 20, 144, 0.18, ff=200), mamba(2, 80, 100, 1, 4, 4, ff=160), latent(2, 72, 130, 40, 0.12)], scale=8.0),
    # one mixer only; head sizes of different classes, layers that differ in every size
    "recurrent": config(52, 80, [mamba(6, 9, 17, 3, 3, 3, ff=70), mamba(2, 33, 65, 2, 6, 5)], eps=1e-4),
    "attending": config(64, 90, [latent(2, 200, 16, 28, 0.07, ff=50), latent(3, 16, 24, 65, 0.3), latent(16, 8, 8, 16, 0.4, ff=77)], scale=0.5),
    # a window and a recurrence side by side, layers that differ in every size, nothing a multiple of 16, a layer without a feed-forward
    "side": mafurax(75, 131, [parallel(attend(6, 2, 24, 20, 0.4, 6.0, 50, 19, 3), 0.7, (3, 10, 14, 8.0), 1.3, ff=90, limit=0.8),
                              parallel(attend(5, 5, 33, 40, 0.3, 9.0, 13, 64, 0), 1.1, (1, 17, 33, 16.0), 0.6)]),
    # heads, columns, ranks, windows and kept tokens of 1 where no norm makes a sign of it
    "side_ones": mafurax(48, 67, [parallel(attend(1, 1, 8, 8, 0.5, 4.0, 2, 1, 1), 1.0, (1, 3, 6, 1.0), 1.0, ff=33, limit=1.0),
                                  parallel(attend(2, 1, 16, 1, 0.4, 3.0, 7, 2, 0), 1.0, (2, 2, 8, 2.0), 0.5, ff=5, limit=2.0)], logit_scale=1.0),
    # more than 16 query heads per key head, a window and kept tokens beyond a page, more than 64 channels and columns
    "side_wide": mafurax(160, 259, [parallel(attend(34, 2, 40, 72, 0.25, 12.0, 100, 65, 66), 0.5, (5, 70, 80, 16.0), 1.4, ff=200, limit=1.5),
                                    parallel(attend(4, 4, 32, 32, 0.35, 20.0, 64, 63, 64), 1.2, (2, 64, 64, 4.0), 0.9, ff=96, limit=0.5)]),
    # the widest head class, a window longer than any sequence, more than 128 channels
    "side_long": mafurax(64, 90, [parallel(attend(4, 2, 130, 16, 0.15, 15.0, 140, 1000, 5), 0.9, (2, 132, 70, 16.0), 1.1, ff=50, limit=1.0),
                                  parallel(attend(3, 1, 16, 200, 0.4, 8.0, 33, 7, 130), 0.8, (3, 24, 5, 16.0), 1.2, ff=77, limit=1.2)], logit_scale=0.25, eps=1e-6),
}
# sizes that only the tensors have: rows of the bias tables, rank of the decays
ROWS = {"side": dict(rel=8, rank=5), "side_ones": dict(rel=2, rank=1), "side_wide": dict(rel=32, rank=18), "side_long": dict(rel=12, rank=16)}

# weights for which no position of the tests' sequences is badly conditioned: operands rounded to bfloat16 move every row of logits by little (test_stack.py measures it)
SEEDS = {"attending": 11, "odd": 25, "ones": 21, "recurrent": 15, "wide": 14, "side": 10, "side_ones": 12, "side_wide": 1, "side_long": 9}


def weights(name, seed=None):
    from oracle import stack_oracle
    return stack_oracle.random_model(CONFIGS[name], SEEDS[name] if seed is None else seed, ROWS.get(name))


def tokens(cfg, n, seed):
    return [int(t) for t in np.random.default_rng(seed).integers(0, cfg["vocab"], n)]
