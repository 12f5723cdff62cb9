"""Shared pieces of the Feditar tests: small configurations made here (none of them a real model's sizes),
the engine or single kernels on one side, oracle/feditar_oracle.py on the other. Replay, step and comparison
helpers are the ones of tests/_kagalorn.py."""
from __future__ import annotations

import random

from tests._kagalorn import TOL, assert_close, make_step, rel_err, replay, tokens_for, write_model  # noqa: F401

MEM_A = {"heads": 3, "dim": 8, "vdim": 12, "gate_cap": 6.0}
MEM_B = {"heads": 2, "dim": 20, "vdim": 6, "gate_cap": 15.0}
SSM_A = {"heads": 4, "vdim": 8, "state": 12, "groups": 2, "conv": 4, "norm_groups": 2}
SSM_B = {"heads": 3, "vdim": 10, "state": 7, "groups": 1, "conv": 2, "norm_groups": 3}
LEFT_A = {"heads": 4, "kv_heads": 2, "dim": 12, "vdim": 10, "scale": 0.4, "conv": 3, "softcap": 4.0, "q_temp": {"coef": 0.4, "every": 7}}
LEFT_B = {"heads": 3, "kv_heads": 3, "dim": 8, "vdim": 16, "scale": 0.5, "conv": 5, "softcap": 9.0, "q_temp": {"coef": -0.1, "every": 20}}
RIGHT_A = {"heads": 3, "dim": 8}
RIGHT_B = {"heads": 2, "dim": 14, "decay_rank": 3}
DENSE = {"kind": "dense", "ff": 40}
PAIRS = {"buckets": 31, "mul_prev": 7, "mul_cur": 3}

# every kind of layer, with and without a feed-forward
CFG_MAIN = {
    "architecture": "Feditar", "vocab": 67, "width": 48, "norm": {"eps": 1e-5}, "max_positions": 192,
    "embedding": {"scale": 5.0, "bigram": PAIRS},
    "layers": [
        {"type": "mlstm", "mixer": MEM_A, "mlp": DENSE},
        {"type": "mamba2", "mixer": SSM_A, "mlp": None},
        {"type": "parallel", "mixer": {"left": LEFT_A, "right": RIGHT_A}, "mlp": DENSE},
        {"type": "mamba2", "mixer": SSM_B, "mlp": DENSE},
        {"type": "mlstm", "mixer": MEM_B, "mlp": None},
        {"type": "parallel", "mixer": {"left": LEFT_B, "right": RIGHT_B}, "mlp": None},
    ],
}
# values that a model may happen to make 1 or equal: one head everywhere, one kv head under five, filters of one tap, of two and
# longer than a register window, a group and a norm part for every head and one for all, rank 1, one hash bucket, a factor that
# changes with every position, no factor, no cap, a gate cap far below 1, value sizes above one wave, key sizes 40 and 70, no
# embedding factor
CFG_ODD = {
    "architecture": "Feditar", "vocab": 37, "width": 40, "norm": {"eps": 1e-6}, "max_positions": 64,
    "embedding": {"bigram": {"buckets": 1, "mul_prev": 1, "mul_cur": 1}},
    "layers": [
        {"type": "parallel", "mixer": {"left": {"heads": 5, "kv_heads": 1, "dim": 6, "vdim": 70, "scale": 0.5, "conv": 1, "softcap": 1.5,
                                                "q_temp": {"coef": 0.2, "every": 1}},
                                       "right": {"heads": 1, "dim": 70, "decay_rank": 1}}, "mlp": None},
        {"type": "mamba2", "mixer": {"heads": 4, "vdim": 6, "state": 70, "groups": 4, "conv": 1, "norm_groups": 4}, "mlp": DENSE},
        {"type": "mlstm", "mixer": {"heads": 1, "dim": 40, "vdim": 130, "gate_cap": 0.5}, "mlp": DENSE},
        {"type": "mamba2", "mixer": {"heads": 1, "vdim": 66, "state": 5, "groups": 1, "conv": 11, "norm_groups": 1}, "mlp": None},
        {"type": "parallel", "mixer": {"left": {"heads": 2, "kv_heads": 2, "dim": 5, "vdim": 3, "scale": 0.6, "conv": 9},
                                       "right": {"heads": 5, "dim": 3}}, "mlp": DENSE},
    ],
}
# no hashed pairs; a single layer after which the model ends with a pair of mixers
CFG_ONE = {
    "architecture": "Feditar", "vocab": 41, "width": 36, "norm": {"eps": 1e-4}, "max_positions": 96, "embedding": {"scale": 0.5},
    "layers": [{"type": "parallel", "mixer": {"left": LEFT_B, "right": RIGHT_A}, "mlp": None}],
}
CFG_ONE_MEM = {
    "architecture": "Feditar", "vocab": 41, "width": 33, "norm": {"eps": 1e-5}, "max_positions": 96,
    "embedding": {"scale": 3.0, "bigram": {"buckets": 1 << 20 >> 13, "mul_prev": 1 << 40, "mul_cur": 3}},
    "layers": [{"type": "mlstm", "mixer": {"heads": 2, "dim": 7, "vdim": 9, "gate_cap": 3.0}, "mlp": None}],
}
# sizes in multiples of 16 and 64 (in bf16 the attention then runs on the matrix cores), five query heads a kv head
CFG_WIDE = {
    "architecture": "Feditar", "vocab": 83, "width": 64, "norm": {"eps": 1e-6}, "max_positions": 128,
    "embedding": {"scale": 8.0, "bigram": PAIRS},
    "layers": [
        {"type": "mamba2", "mixer": {"heads": 8, "vdim": 16, "state": 16, "groups": 4, "conv": 4, "norm_groups": 1},
         "mlp": {"kind": "dense", "ff": 128}},
        {"type": "parallel", "mixer": {"left": {"heads": 5, "kv_heads": 1, "dim": 32, "vdim": 48, "scale": 0.25, "conv": 4, "softcap": 8.0,
                                                "q_temp": {"coef": 0.25, "every": 16}},
                                       "right": {"heads": 4, "dim": 16, "decay_rank": 8}}, "mlp": {"kind": "dense", "ff": 96}},
        {"type": "mlstm", "mixer": {"heads": 4, "dim": 16, "vdim": 32, "gate_cap": 10.0}, "mlp": None},
    ],
}
# prompts of a few hundred tokens over several 64-token pages and 64-key tiles, head sizes of a real model's order
CFG_LONG = {
    "architecture": "Feditar", "vocab": 211, "width": 96, "norm": {"eps": 1e-6}, "max_positions": 400,
    "embedding": {"scale": 9.0, "bigram": {"buckets": 97, "mul_prev": 19, "mul_cur": 5}},
    "layers": [
        {"type": "mlstm", "mixer": {"heads": 2, "dim": 64, "vdim": 96, "gate_cap": 12.0}, "mlp": None},
        {"type": "parallel", "mixer": {"left": {"heads": 6, "kv_heads": 3, "dim": 64, "vdim": 32, "scale": 0.15, "conv": 3, "softcap": 6.0,
                                                "q_temp": {"coef": 0.3, "every": 65}},
                                       "right": {"heads": 2, "dim": 48, "decay_rank": 6}}, "mlp": {"kind": "dense", "ff": 160}},
        {"type": "mamba2", "mixer": {"heads": 3, "vdim": 64, "state": 48, "groups": 3, "conv": 4, "norm_groups": 3}, "mlp": None},
    ],
}


def random_config(seed: int) -> dict:
    """A configuration drawn from lists of sizes: layer count and kinds, head counts and sizes, filters, groups, caps, factors,
    ranks, feed-forwards and the embedding's parts all vary."""
    r = random.Random(seed)
    layers = []
    for _ in range(r.randint(2, 4)):
        kind = r.choice(["mlstm", "mamba2", "parallel"])
        if kind == "mlstm":
            m = {"heads": r.choice([1, 2, 3]), "dim": r.choice([4, 8, 20, 36]), "vdim": r.choice([6, 16, 72]), "gate_cap": r.choice([1.0, 5.0, 15.0])}
        elif kind == "mamba2":
            G = r.choice([1, 2, 3])
            H = G * r.choice([1, 2])
            m = {"heads": H, "vdim": r.choice([6, 8, 16]), "state": r.choice([4, 16, 33]), "groups": G, "conv": r.choice([1, 2, 3, 4, 6]),
                 "norm_groups": r.choice([1, H])}
        else:
            G = r.choice([1, 2])
            left = {"heads": G * r.choice([1, 2, 3]), "kv_heads": G, "dim": r.choice([8, 12, 16, 24]), "vdim": r.choice([8, 16, 20]),
                    "scale": r.choice([0.2, 0.4]), "conv": r.choice([1, 2, 3, 4])}
            if r.random() < 0.8:
                left["softcap"] = r.choice([2.0, 7.0, 30.0])
            if r.random() < 0.8:
                left["q_temp"] = {"coef": r.choice([0.1, 0.5]), "every": r.choice([1, 16, 64, 100])}
            m = {"left": left, "right": {"heads": r.choice([1, 2, 3]), "dim": r.choice([4, 8, 20]), "decay_rank": r.choice([1, 4, 9])}}
        layers.append({"type": kind, "mixer": m, "mlp": r.choice([None, {"kind": "dense", "ff": r.choice([24, 40, 65])}])})
    emb = {"scale": r.choice([1.0, 4.0])}
    if r.random() < 0.8:
        emb["bigram"] = {"buckets": r.choice([1, 13, 101]), "mul_prev": r.choice([1, 31, 1009]), "mul_cur": r.choice([1, 17])}
    return {"architecture": "Feditar", "vocab": r.choice([53, 97]), "width": r.choice([32, 48, 60]), "norm": {"eps": r.choice([1e-6, 1e-5])},
            "max_positions": 224, "embedding": emb, "layers": layers}
