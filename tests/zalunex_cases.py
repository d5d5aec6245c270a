"""Small Zalunex configurations with random weights for the tests, none of them of a served model's sizes.  They differ
from one another in every size and constant; between them they cover a layer without a feed-forward, dense and routed
feed-forwards with other limits, expert sizes that are and are not multiples of 8, one expert, as many experts a token as
there are, one head, as many KV heads as query heads and one for all, values wider and narrower than keys in both halves, head
sizes that the matrix-core kernels take and sizes that they refuse, windows of one token, shorter and longer than a page, off
the pages' borders and none, decays from 0 over slow ones to 1, factors of one, below zero and others on both halves and on the
residual, logits with and without a cap, and a stretch that runs again in the middle, three times at the start, at the end, once
only, over the whole model, and none.
"""
import copy

import numpy as np
import torch


def _layer(left, right, left_scale, right_scale, mlp=None):
    heads, kv, dim, vdim, scale, window = left
    a = {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim, "scale": scale}
    if window:
        a["mask"] = {"size": window}
    r = {"heads": len(right[2]), "dim": right[0], "vdim": right[1], "decay": list(right[2])}
    return {"type": "parallel", "mixer": {"left": a, "right": r, "left_scale": left_scale, "right_scale": right_scale}, "mlp": mlp}


def _dense(ff, limit):
    return {"kind": "dense", "ff": ff, "limit": limit}


def _moe(experts, top, ff):
    return {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top}}


CONFIGS = {
    # a stretch of three in the middle runs twice; values of other sizes than keys; a layer without a feed-forward
    "P": {"architecture": "Zalunex", "vocab": 97, "width": 48, "max_positions": 333, "norm": {"eps": 1e-5}, "residual_mult": 0.6,
          "logit_softcap": 12.0, "loop": {"start": 1, "stop": 4, "times": 2},
          "layers": [_layer((4, 2, 16, 12, 0.4, 20), (12, 20, (0.9, 0.5, 0.99)), 0.7, 1.3, _dense(40, 0.8)),
                     _layer((6, 3, 8, 24, 0.6, 33), (20, 8, (0.97, 0.7)), 1.2, 0.5, _moe(5, 4, 20)),
                     _layer((2, 2, 10, 10, 0.5, 7), (6, 14, (0.8, 1.0, 0.95, 0.3)), -0.9, 0.6),
                     _layer((3, 1, 20, 8, 0.35, 50), (16, 16, (0.999,)), 1.1, -0.8, _moe(3, 1, 7))]},
    # sizes of the matrix-core kernels; windows of less than a page and of several
    "Q": {"architecture": "Zalunex", "vocab": 130, "width": 64, "max_positions": 1000, "norm": {"eps": 1e-6}, "residual_mult": 1.3,
          "logit_softcap": 25.0, "loop": {"start": 1, "stop": 2, "times": 2},
          "layers": [_layer((4, 2, 64, 40, 0.11, 37), (32, 64, (0.99, 0.9, 0.6, 0.97)), 1.25, 0.75, _moe(4, 2, 32)),
                     _layer((2, 2, 32, 64, 0.2, 5), (64, 32, (0.98, 0.93)), 0.5, 2.0, _dense(96, 2.0)),
                     _layer((8, 1, 24, 32, 0.2, 100), (40, 48, (0.995, 0.4)), 0.9, 1.1, _moe(6, 3, 48))]},
    # one head, one expert, as many experts a token as there are, a window of one token, no window, pages of 8, no loop, no cap
    "R": {"architecture": "Zalunex", "vocab": 64, "width": 32, "max_positions": 400, "norm": {"eps": 3e-6}, "residual_mult": 1.0,
          "layers": [_layer((1, 1, 10, 6, 0.35, 1), (6, 10, (0.0, 0.9, 0.3)), 1.0, 1.0, _moe(1, 1, 12)),
                     _layer((3, 3, 16, 16, 0.3, 0), (8, 12, (0.9, 1.0, 0.99, 0.5)), 0.3, -1.5, _moe(2, 2, 8)),
                     _layer((2, 1, 12, 20, 0.4, 17), (7, 1, (0.85, 0.95, 0.6, 0.99, 0.9, 0.7, 0.8, 0.3)), 0.8, 0.4, _dense(24, 0.3))]},
    # pages of 32, heads of 128 with three query heads per KV head, one layer three times at the start
    "S": {"architecture": "Zalunex", "vocab": 200, "width": 96, "max_positions": 512, "norm": {"eps": 1e-5}, "residual_mult": 0.45,
          "logit_softcap": 40.0, "loop": {"start": 0, "stop": 1, "times": 3},
          "layers": [_layer((6, 2, 128, 128, 0.06, 70), (96, 48, (0.99, 0.8)), 0.8, 1.4, _moe(8, 3, 48)),
                     _layer((2, 1, 32, 32, 0.2, 0), (24, 24, (0.9, 0.99, 0.7, 0.997)), 1.6, 0.4, _dense(64, 7.0)),
                     _layer((3, 1, 48, 136, 0.12, 128), (130, 72, (0.96,)), 1.0, 1.0, _dense(80, 1.5))]},
    # nothing a multiple of 8: a width of 100, an odd vocabulary, five heads of 20; the last layer runs again
    "T": {"architecture": "Zalunex", "vocab": 451, "width": 100, "max_positions": 321, "norm": {"eps": 1e-5}, "residual_mult": 0.85,
          "logit_softcap": 9.0, "loop": {"start": 1, "stop": 2, "times": 2},
          "layers": [_layer((5, 5, 20, 28, 0.25, 23), (14, 9, (0.9, 0.99, 0.6)), 1.7, 0.9, _moe(6, 3, 50)),
                     _layer((6, 3, 12, 20, 0.4, 64), (22, 13, (0.97, 0.8)), 0.45, 1.15, _moe(3, 2, 33))]},
    # the whole model runs twice
    "U": {"architecture": "Zalunex", "vocab": 75, "width": 56, "max_positions": 700, "norm": {"eps": 1e-5}, "residual_mult": 0.5,
          "logit_softcap": 18.0, "loop": {"start": 0, "stop": 2, "times": 2},
          "layers": [_layer((4, 4, 24, 16, 0.3, 16), (10, 30, (0.99, 0.9)), 1.0, 0.5, _dense(30, 1.0)),
                     _layer((4, 2, 8, 8, 0.7, 90), (20, 16, (0.995, 0.75)), 0.6, 1.0, _moe(4, 3, 24))]},
    # a loop that runs once only
    "V": {"architecture": "Zalunex", "vocab": 81, "width": 40, "max_positions": 350, "norm": {"eps": 2e-5}, "residual_mult": 0.9,
          "logit_softcap": 15.0, "loop": {"start": 0, "stop": 1, "times": 1},
          "layers": [_layer((5, 1, 16, 8, 0.45, 9), (16, 8, (0.9, 0.98, 0.3, 0.999, 0.6)), 1.3, 0.7, _dense(33, 0.5))]},
}
BLOCK_SIZE = {"P": 16, "Q": 16, "R": 8, "S": 32, "T": 16, "U": 8, "V": 16}


def tensors_for(raw, seed, sharpen=3.0):
    """Checkpoint names -> tensors (float32 on the bfloat16 grid, so that both storage modes hold the same numbers).
    Matrices N(0, 1 / fan-in), the gated feed-forward's first ones wider so that its limits act; norm weights stored around zero
    0.2 N, plain ones 1 + 0.1 N; sinks spread over -1 .. 3, so that they take a good part of the weight."""
    from kvcm_amd.config.zalunex_config import ZalunexConfig
    from kvcm_amd.weights.random_init import expected_tensors
    cfg = ZalunexConfig.from_dict(raw)
    rng = np.random.default_rng(seed)
    out = {}
    for name, (shape, role) in sorted(expected_tensors("Zalunex", cfg).items()):
        leaf = name.rsplit(".", 1)[-1]
        a = rng.normal(size=shape)
        if name in ("embed", "pos"):
            a = a * 0.7
        elif leaf == "sink":
            a = a + 1.0
        elif leaf in ("norm1", "norm1b", "norm2", "norm2b") or name == "final.norm":
            a = a * 0.2
        elif role == "vector":
            a = 1.0 + 0.1 * a
        elif len(shape) == 2:
            a = a / np.sqrt(shape[1])
            if leaf == "router":
                a = a * sharpen
            elif leaf in ("gate", "up"):
                a = a * 1.5
        out[name] = torch.from_numpy(np.asarray(a, dtype=np.float64)).to(torch.bfloat16).to(torch.float32)
    return cfg, out


def as_numpy(tensors):
    return {k: v.double().numpy() for k, v in tensors.items()}


def requests_for(raw, lengths, seed):
    rng = np.random.default_rng(seed)
    return {f"r{i}": rng.integers(0, raw["vocab"], size=n).tolist() for i, n in enumerate(lengths)}


def with_every_expert_chosen(raw):
    """The configuration with ``top`` raised to the number of experts in every routed layer: nothing is chosen, so no choice
    hangs on rounding.  (Where 8-bit rounding decides between two experts of nearly equal scores, the other expert's output
    enters that token's keys and states and stays there for every later token: a test of long decoding should not rest on it.)"""
    out = copy.deepcopy(raw)
    for layer in out["layers"]:
        if layer["mlp"] and layer["mlp"]["kind"] == "moe":
            layer["mlp"]["router"]["top"] = layer["mlp"]["router"]["experts"]
    return out
