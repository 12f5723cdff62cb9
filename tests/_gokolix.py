"""Shared pieces of the Gokolix tests: small configurations made here (none of them a real model's sizes),
the engine or single kernels on one side, oracle/gokolix_oracle.py on the other. Replay, step and comparison
helpers are the ones of tests/_kagalorn.py."""
from __future__ import annotations

import random

from tests._kagalorn import TOL, assert_close, make_step, rel_err, replay, tokens_for, write_model  # noqa: F401

LAT_A = {"heads": 3, "dim": 12, "vdim": 10, "kv_rank": 24, "rot_dim": 8, "scale": 0.3, "mask": {"size": 11},
         "rot": {"dims": 8, "base": 100.0, "scaling": {"factor": 8.0, "original": 64, "fast": 4.0, "slow": 0.5}}}
LAT_B = {"heads": 5, "dim": 6, "vdim": 7, "kv_rank": 9, "rot_dim": 6, "scale": 0.4, "mask": {"size": 20},
         "rot": {"dims": 6, "base": 5000.0, "scaling": {"factor": 2.5, "original": 300, "fast": 8.0, "slow": 1.0}}}
ATT_A = {"heads": 4, "kv_heads": 2, "dim": 12, "vdim": 12, "scale": 0.5, "mask": {"size": 19}, "bias_max": 15, "rel_rows": 8}
ATT_B = {"heads": 3, "kv_heads": 3, "dim": 10, "vdim": 10, "scale": 0.35, "mask": {"size": 7}, "bias_max": 40, "rel_rows": 12}
LRU_A = {"width": 40, "blocks": 4, "conv": 4}
LRU_B = {"width": 33, "blocks": 3, "conv": 2}
DENSE = {"kind": "dense", "ff": 40}

# every kind of layer, with and without a feed-forward; three passes over the middle of the stack
CFG_MAIN = {
    "architecture": "Gokolix", "vocab": 61, "width": 48, "norm": {"eps": 1e-5}, "embedding": {"scale": 3.0},
    "loop": {"start": 1, "stop": 4, "times": 3},
    "layers": [
        {"type": "attention", "mixer": ATT_B, "mlp": DENSE},
        {"type": "latent_attention", "mixer": LAT_A, "mlp": DENSE},
        {"type": "rglru", "mixer": LRU_A, "mlp": None},
        {"type": "attention", "mixer": ATT_A, "mlp": DENSE},
        {"type": "rglru", "mixer": LRU_B, "mlp": DENSE},
        {"type": "latent_attention", "mixer": LAT_B, "mlp": None},
    ],
}
# values that a model may happen to make 1 or equal: one head everywhere, one kv head under five, a window of one and one of
# two, a pair of rotated entries, a scaling by 1 and none at all, no rotated part, one block and a block a channel, filters of one
# tap and longer than a register window, a bias table of two rows, a single pass, no factor on the embeddings
CFG_ODD = {
    "architecture": "Gokolix", "vocab": 37, "width": 40, "norm": {"eps": 1e-6}, "loop": {"start": 0, "stop": 6, "times": 1},
    "layers": [
        {"type": "attention", "mixer": {"heads": 5, "kv_heads": 1, "dim": 6, "vdim": 6, "scale": 0.6, "mask": {"size": 30}, "bias_max": 3,
                                        "rel_rows": 2}, "mlp": None},
        {"type": "rglru", "mixer": {"width": 6, "blocks": 6, "conv": 1}, "mlp": {"kind": "dense", "ff": 1}},
        {"type": "latent_attention", "mixer": {"heads": 1, "dim": 5, "vdim": 70, "kv_rank": 3, "rot_dim": 2, "scale": 0.5, "mask": {"size": 2},
                                               "rot": {"dims": 2, "base": 30.0, "scaling": {"factor": 1.0, "original": 16, "fast": 2.0, "slow": 1.0}}},
         "mlp": {"kind": "dense", "ff": 17}},
        {"type": "rglru", "mixer": {"width": 70, "blocks": 1, "conv": 9}, "mlp": None},
        {"type": "attention", "mixer": {"heads": 1, "kv_heads": 1, "dim": 66, "vdim": 66, "scale": 0.2, "mask": {"size": 1}, "bias_max": 33,
                                        "rel_rows": 5}, "mlp": DENSE},
        {"type": "latent_attention", "mixer": {"heads": 2, "dim": 8, "vdim": 4, "kv_rank": 12, "rot_dim": 4, "scale": 0.4, "mask": {"size": 9},
                                               "rot": {"dims": 4, "base": 10.0}}, "mlp": None},
    ],
}
# no loop; windows no request reaches
CFG_ONE = {
    "architecture": "Gokolix", "vocab": 41, "width": 36, "norm": {"eps": 1e-4}, "embedding": {"scale": 0.3},
    "layers": [{"type": "latent_attention", "mixer": {**LAT_A, "mask": {"size": 500}}, "mlp": DENSE},
               {"type": "attention", "mixer": {**ATT_A, "mask": {"size": 500}}, "mlp": None}],
}
# the loop is the whole model, one recurrent layer in two passes
CFG_ONE_LRU = {
    "architecture": "Gokolix", "vocab": 41, "width": 33, "norm": {"eps": 1e-5}, "embedding": {"scale": 2.0},
    "loop": {"start": 0, "stop": 1, "times": 2}, "layers": [{"type": "rglru", "mixer": LRU_B, "mlp": None}],
}
# sizes in multiples of 16 and 32 (in bf16 attention and gates then run on the matrix cores), five query heads a kv head
CFG_WIDE = {
    "architecture": "Gokolix", "vocab": 83, "width": 64, "norm": {"eps": 1e-6}, "embedding": {"scale": 4.0},
    "loop": {"start": 0, "stop": 2, "times": 2},
    "layers": [
        {"type": "rglru", "mixer": {"width": 96, "blocks": 3, "conv": 4}, "mlp": {"kind": "dense", "ff": 128}},
        {"type": "attention", "mixer": {"heads": 5, "kv_heads": 1, "dim": 32, "vdim": 32, "scale": 0.2, "mask": {"size": 18}, "bias_max": 30,
                                        "rel_rows": 16}, "mlp": {"kind": "dense", "ff": 96}},
        {"type": "latent_attention", "mixer": {"heads": 4, "dim": 16, "vdim": 32, "kv_rank": 48, "rot_dim": 16, "scale": 0.2, "mask": {"size": 33},
                                               "rot": {"dims": 16, "base": 1000.0, "scaling": {"factor": 4.0, "original": 128, "fast": 8.0,
                                                                                               "slow": 1.0}}}, "mlp": None},
    ],
}
# prompts of a few hundred tokens over several 64-token pages and 64-key tiles, windows around tile and page sizes
CFG_LONG = {
    "architecture": "Gokolix", "vocab": 211, "width": 96, "norm": {"eps": 1e-6}, "embedding": {"scale": 5.0},
    "loop": {"start": 1, "stop": 3, "times": 2},
    "layers": [
        {"type": "attention", "mixer": {"heads": 6, "kv_heads": 3, "dim": 48, "vdim": 48, "scale": 0.15, "mask": {"size": 65}, "bias_max": 100,
                                        "rel_rows": 20}, "mlp": {"kind": "dense", "ff": 160}},
        {"type": "rglru", "mixer": {"width": 128, "blocks": 2, "conv": 3}, "mlp": None},
        {"type": "latent_attention", "mixer": {"heads": 4, "dim": 32, "vdim": 24, "kv_rank": 64, "rot_dim": 32, "scale": 0.15,
                                               "mask": {"size": 130},
                                               "rot": {"dims": 32, "base": 20000.0, "scaling": {"factor": 16.0, "original": 512, "fast": 16.0,
                                                                                                "slow": 2.0}}}, "mlp": None},
        {"type": "attention", "mixer": {"heads": 2, "kv_heads": 1, "dim": 64, "vdim": 64, "scale": 0.12, "mask": {"size": 200}, "bias_max": 64,
                                        "rel_rows": 32}, "mlp": {"kind": "dense", "ff": 96}},
    ],
}


def random_config(seed: int) -> dict:
    """A configuration drawn from lists of sizes: layer count, kinds and order, the loop, head counts and sizes, windows, biases,
    rotations, blocks, filters, feed-forwards and the embedding's factor all vary."""
    r = random.Random(seed)
    layers = []
    for _ in range(r.randint(2, 5)):
        kind = r.choice(["latent_attention", "attention", "rglru"])
        window = {"size": r.choice([3, 16, 33, 64, 65, 128, 400])}
        if kind == "latent_attention":
            d = r.choice([4, 8, 16])
            m = {"heads": r.choice([1, 2, 3, 5]), "dim": r.choice([8, 12, 16, 24]), "vdim": r.choice([8, 10, 16]), "kv_rank": r.choice([12, 16, 48]),
                 "rot_dim": d, "scale": r.choice([0.2, 0.4]), "mask": window,
                 "rot": {"dims": d, "base": r.choice([50.0, 10000.0]),
                         "scaling": {"factor": r.choice([2.0, 10.0]), "original": r.choice([32, 256, 4096]), "fast": r.choice([4.0, 32.0]),
                                     "slow": r.choice([0.5, 1.0])}}}
        elif kind == "attention":
            G, D, B = r.choice([1, 2]), r.choice([8, 12, 16, 36, 48]), r.choice([4, 8, 32])
            m = {"heads": G * r.choice([1, 2, 3]), "kv_heads": G, "dim": D, "vdim": D, "scale": r.choice([0.2, 0.5]), "mask": window,
                 "bias_max": r.choice([20, 64, 150]), "rel_rows": B}
        else:
            B = r.choice([1, 2, 3])
            m = {"width": B * r.choice([8, 20, 32, 64]), "blocks": B, "conv": r.choice([1, 2, 3, 4, 6])}
        layers.append({"type": kind, "mixer": m, "mlp": r.choice([None, {"kind": "dense", "ff": r.choice([24, 40, 65])}])})
    cfg = {"architecture": "Gokolix", "vocab": r.choice([53, 97]), "width": r.choice([32, 48, 60]), "norm": {"eps": r.choice([1e-6, 1e-5])},
           "embedding": {"scale": r.choice([0.7, 1.0, 4.0])}, "layers": layers}
    start = r.randint(0, len(layers) - 1)
    cfg["loop"] = {"start": start, "stop": r.randint(start + 1, len(layers)), "times": r.choice([1, 2, 3])}
    return cfg
