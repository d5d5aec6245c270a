"""Small Vugotar configurations with random weights for the tests, none of them of a served model's sizes.  They differ
from one another in every size and constant; between them they cover each mixer first and last, a layer without a
feed-forward, dense and routed feed-forwards with and without a shared expert, expert sizes that are and are not
multiples of 16, one expert, as many experts a token as there are, one head, as many KV heads as query heads and one
for all, in the attention and in the delta rule, values wider and narrower than keys, no / partial / whole rotation,
head sizes that the matrix-core kernels take and sizes that they refuse, chunks of one token, shorter and longer than a
page, off the pages' borders and none, convolutions of one to five taps, one and several groups, norm parts that differ
from the groups, factors of one, below zero and others, and a stretch that runs again in the middle, three times at the
start, at the end, once only, and none.
"""
import copy

import numpy as np
import torch


def _parallel(left, right, left_scale, right_scale):
    heads, kv, dim, vdim, scale, chunk, rot = left
    a = {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim, "scale": scale}
    if chunk:
        a["mask"] = {"size": chunk}
    if rot:
        a["rot"] = {"dims": rot[0], "base": rot[1]}
    d = dict(zip(("heads", "kv_heads", "dim", "vdim", "conv"), right))
    return "parallel", {"left": a, "right": d, "left_scale": left_scale, "right_scale": right_scale}


def _mamba2(heads, vdim, state, groups, norm_groups, conv):
    return "mamba2", {"heads": heads, "vdim": vdim, "state": state, "groups": groups, "norm_groups": norm_groups, "conv": conv}


def _dense(ff):
    return {"kind": "dense", "ff": ff}


def _moe(experts, top, ff, scale, shared=0):
    d = {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top, "scale": scale}}
    if shared:
        d["shared"] = {"ff": shared}
    return d


def _layer(mixer, mlp=None):
    return {"type": mixer[0], "mixer": mixer[1], "mlp": mlp}


CONFIGS = {
    # a stretch of three in the middle runs twice; values of other sizes than keys; a layer without a feed-forward
    "P": {"architecture": "Vugotar", "vocab": 97, "width": 48, "norm": {"eps": 1e-5}, "loop": {"start": 1, "stop": 4, "times": 2},
          "layers": [_layer(_mamba2(4, 12, 10, 2, 3, 3), _dense(40)),
                     _layer(_parallel((4, 2, 16, 12, 0.4, 20, (8, 100.0)), (6, 3, 12, 20, 4), 0.7, 1.3), _moe(5, 2, 20, 1.6, shared=24)),
                     _layer(_mamba2(3, 16, 24, 1, 2, 2)),
                     _layer(_parallel((3, 1, 10, 24, 0.5, 7, (10, 5000.0)), (2, 1, 20, 8, 2), -0.9, 0.6), _dense(56)),
                     _layer(_parallel((2, 2, 8, 8, 0.6, 33, None), (3, 3, 16, 16, 3), 1.1, 0.8), _moe(3, 1, 7, 0.5, shared=9))]},
    # sizes of the matrix-core kernels; several chunks a page and several pages a chunk; no shared expert in one layer
    "Q": {"architecture": "Vugotar", "vocab": 130, "width": 64, "norm": {"eps": 1e-6}, "loop": {"start": 2, "stop": 4, "times": 2},
          "layers": [_layer(_parallel((4, 2, 64, 40, 0.11, 33, (32, 10000.0)), (4, 2, 32, 64, 4), 1.25, 0.75), _moe(4, 2, 32, 2.0, shared=16)),
                     _layer(_mamba2(4, 32, 64, 4, 2, 4), _moe(6, 3, 48, 1.0)),
                     _layer(_parallel((2, 2, 32, 64, 0.2, 5, (32, 500000.0)), (2, 1, 64, 32, 2), 0.5, 2.0), _dense(96)),
                     _layer(_mamba2(2, 64, 32, 1, 1, 2), _dense(72))]},
    # one head, one expert, as many experts a token as there are, one tap, a chunk of one token, pages of 8, no loop
    "R": {"architecture": "Vugotar", "vocab": 64, "width": 32, "norm": {"eps": 3e-6},
          "layers": [_layer(_parallel((1, 1, 10, 6, 0.35, 1, (2, 50.0)), (1, 1, 6, 10, 1), 1.0, 1.0), _moe(1, 1, 12, 1.0, shared=8)),
                     _layer(_mamba2(1, 8, 5, 1, 1, 1), _moe(2, 2, 8, 3.0)),
                     _layer(_parallel((3, 3, 16, 16, 0.3, 40, (16, 20000.0)), (4, 1, 8, 12, 5), 0.3, -1.5))]},
    # pages of 32, heads of 128 with three query heads per KV head, no chunks in the second, one layer three times at the start
    "S": {"architecture": "Vugotar", "vocab": 200, "width": 96, "norm": {"eps": 1e-5}, "loop": {"start": 0, "stop": 1, "times": 3},
          "layers": [_layer(_parallel((6, 2, 128, 128, 0.06, 70, (64, 25000.0)), (2, 2, 96, 48, 4), 0.8, 1.4), _moe(8, 3, 48, 2.2, shared=64)),
                     _layer(_parallel((2, 1, 32, 32, 0.2, 0, (16, 1000.0)), (4, 4, 24, 24, 3), 1.6, 0.4), _dense(64)),
                     _layer(_mamba2(6, 24, 130, 3, 6, 4), _dense(80))]},
    # nothing a multiple of 8: a width of 100, an odd vocabulary, five heads of 20; the last layer runs again; a mixer first that
    # has no feed-forward beside it
    "T": {"architecture": "Vugotar", "vocab": 451, "width": 100, "norm": {"eps": 1e-5}, "loop": {"start": 2, "stop": 3, "times": 2},
          "layers": [_layer(_mamba2(5, 7, 11, 5, 7, 3)),
                     _layer(_parallel((5, 5, 20, 28, 0.25, 23, (12, 30000.0)), (3, 3, 14, 9, 3), 1.7, 0.9), _moe(6, 3, 50, 1.3, shared=70)),
                     _layer(_parallel((6, 3, 12, 20, 0.4, 64, (4, 70.0)), (6, 2, 22, 13, 4), 0.45, 1.15), _moe(3, 2, 33, 0.8, shared=21))]},
    # a loop that runs once only: no embedding is added again
    "U": {"architecture": "Vugotar", "vocab": 75, "width": 56, "norm": {"eps": 1e-5}, "loop": {"start": 0, "stop": 2, "times": 1},
          "layers": [_layer(_parallel((4, 4, 24, 16, 0.3, 16, (24, 900.0)), (2, 2, 10, 30, 3), 1.0, 0.5), _dense(30)),
                     _layer(_mamba2(2, 20, 16, 2, 4, 3), _moe(4, 1, 24, 1.0, shared=40))]},
}
BLOCK_SIZE = {"P": 16, "Q": 16, "R": 8, "S": 32, "T": 16, "U": 8}


def tensors_for(raw, seed, sharpen=3.0):
    """Checkpoint names -> tensors (float32 on the bfloat16 grid, so that both storage modes hold the same numbers).
    Matrices N(0, 1 / fan-in); norm weights stored around zero 0.2 N, plain ones 1 + 0.1 N; biases 0.3 N; decays slow enough
    that a state reaches back over tens of tokens; the delta rule's rates spread over (0, 1)."""
    from kvcm_amd.config.vugotar_config import VugotarConfig
    from kvcm_amd.weights.random_init import expected_tensors
    cfg = VugotarConfig.from_dict(raw)
    rng = np.random.default_rng(seed)
    out = {}
    for name, (shape, role) in sorted(expected_tensors("Vugotar", cfg).items()):
        leaf = name.rsplit(".", 1)[-1]
        a = rng.normal(size=shape)
        if name == "embed":
            a = a * 0.7
        elif leaf == "A_log":
            a = a * 0.7 - 1.5
        elif leaf == "dt_bias":
            a = a * 0.5 - 1.0
        elif leaf in ("norm1",) or name == "final.norm":
            a = a * 0.2
        elif role == "vector":
            a = 1.0 + 0.1 * a
        elif len(shape) == 2:
            a = a / np.sqrt(shape[1])
            if leaf == "router":
                a = a * sharpen
        else:
            a = a * 0.3
        out[name] = torch.from_numpy(np.asarray(a, dtype=np.float64)).to(torch.bfloat16).to(torch.float32)
    return cfg, out


def as_numpy(tensors):
    return {k: v.double().numpy() for k, v in tensors.items()}


def requests_for(raw, lengths, seed):
    rng = np.random.default_rng(seed)
    return {f"r{i}": rng.integers(0, raw["vocab"], size=n).tolist() for i, n in enumerate(lengths)}


def with_every_expert_chosen(raw):
    """The configuration with ``top`` raised to the number of experts in every routed layer: nothing is chosen, so no choice
    hangs on rounding.  (Where 8-bit rounding decides between two experts of nearly equal logits, the other expert's output
    enters that token's keys and states and stays there for every later token: a test of long decoding should not rest on it.)"""
    out = copy.deepcopy(raw)
    for layer in out["layers"]:
        if layer["mlp"] and layer["mlp"]["kind"] == "moe":
            layer["mlp"]["router"]["top"] = layer["mlp"]["router"]["experts"]
    return out
