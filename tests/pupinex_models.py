"""Tiny Pupinex configurations for the tests, and their model folders.

Sizes differ from layer to layer and between the configurations: one to eight heads, grouped and ungrouped, keys
wider and narrower than values, windows of one token to many, a part of a head rotated and all of it, loops of two
layers, of the whole model and of one pass, a layer without a feed-forward, one group of experts to many (groups of a
single expert among them), shared experts smaller and larger than the others.  The random weights are made *sharp*
after they are drawn so that a wrong key, a lost state or sink, a window that is one token off or a wrong
expert moves the logits by far more than bfloat16 rounding.  The norms' eps are large: a recurrence's first outputs are
multiples of one value row, whose sign alone would be left of a small one.
"""
from __future__ import annotations

import functools
import json
import os

import torch


def attn(heads, kv_heads, dim, vdim, scale, size, rot):
    return {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale, "mask": {"size": size},
            "rot": {"dims": rot[0], "base": rot[1]}}


def gla(heads, dim, vdim, tau, rank):
    return {"heads": heads, "dim": dim, "vdim": vdim, "tau": tau, "decay_rank": rank}


def pair(left, factor, right, scales):
    """left: as ``attn``; right: heads, dim, vdim, the gates' cap."""
    m = attn(*left)
    m["rot"]["scaling"] = {"factor": factor}
    h, d, e, cap = right
    return {"left": m, "right": {"heads": h, "dim": d, "vdim": e, "gate_cap": cap}, "left_scale": scales[0], "right_scale": scales[1]}


def dense(ff, limit):
    return {"kind": "dense", "ff": ff, "limit": limit}


def moe(experts, top, groups, keep, ff, shared, scale):
    return {"kind": "moe", "expert": {"ff": ff}, "shared": {"ff": shared},
            "router": {"experts": experts, "top": top, "groups": {"count": groups, "keep": keep}, "scale": scale}}


def layer(kind, mixer, mlp):
    return {"type": kind, "mixer": mixer, "mlp": mlp}


def model(width, vocab, eps, bigram, loop, layers):
    m = {"architecture": "Pupinex", "width": width, "vocab": vocab, "norm": {"eps": eps},
         "embedding": {"bigram": dict(zip(("buckets", "mul_prev", "mul_cur"), bigram))}, "layers": layers}
    if loop:
        m["loop"] = dict(zip(("start", "stop", "times"), loop))
    return m


# every kind of layer, a loop over two of them, a layer without a feed-forward, pages of which a window spans two
PX_A = model(64, 300, 1e-2, (211, 31, 7), (1, 3, 3), [
    layer("attention", attn(4, 2, 16, 24, 0.2, 20, (8, 500.0)), dense(72, 1.5)),
    layer("gla", gla(3, 8, 12, 4.0, 6), moe(8, 2, 4, 2, 24, 24, 2.5)),
    layer("parallel", pair((4, 2, 16, 8, 0.5, 13, (8, 900.0)), 3.0, (3, 8, 12, 10.0), (0.7, 0.4)), moe(6, 2, 3, 2, 16, 40, 1.0)),
    layer("attention", attn(2, 1, 24, 32, 0.15, 33, (24, 300.0)), None),
    layer("gla", gla(2, 16, 16, 1.0, 3), dense(40, 3.0)),
])
# the parallel layer first and the whole model twice; a window of one token, heads that are not grouped, one head; every
# expert chosen, one group, groups of a single expert
PX_B = model(96, 257, 3e-3, (64, 5, 3), (0, 3, 2), [
    layer("parallel", pair((6, 6, 8, 8, 0.6, 9, (4, 50.0)), 1.0, (1, 24, 40, 15.0), (1.0, 1.0)), moe(3, 3, 1, 1, 16, 8, 0.5)),
    layer("attention", attn(2, 2, 32, 48, 0.2, 1, (32, 1000000.0)), moe(5, 2, 5, 3, 8, 20, 1.5)),
    layer("gla", gla(1, 40, 24, 16.0, 20), None),
])
# sizes that are no multiples of 8, five heads on one kv head; no loop
PX_C = model(132, 500, 5e-3, (997, 701, 13), None, [
    layer("gla", gla(3, 10, 14, 8.0, 5), moe(6, 4, 2, 2, 28, 12, 2.0)),
    layer("attention", attn(5, 1, 12, 20, 0.25, 37, (12, 777.0)), dense(52, 1.0)),
    layer("parallel", pair((3, 1, 20, 12, 0.7, 16, (10, 2000.0)), 8.0, (2, 36, 20, 6.0), (0.3, 1.2)), dense(36, 2.0)),
    layer("parallel", pair((2, 2, 12, 36, 0.4, 50, (12, 100.0)), 2.0, (5, 6, 10, 12.0), (0.5, 0.5)), moe(12, 3, 6, 3, 20, 44, 2.5)),
])
# head sizes of real models: prompts run on the blocks of the matrix-core attention, keys and values over several tiles
PX_D = model(320, 400, 1e-2, (4093, 127, 31), (1, 2, 1), [
    layer("attention", attn(8, 2, 128, 128, 0.03, 40, (64, 10000.0)), dense(128, 2.0)),
    layer("gla", gla(2, 64, 160, 16.0, 16), moe(8, 3, 4, 2, 32, 64, 2.0)),
    layer("parallel", pair((8, 2, 64, 128, 0.2, 65, (32, 50000.0)), 4.0, (3, 128, 72, 15.0), (0.6, 0.5)), dense(96, 4.0)),
    layer("gla", gla(2, 130, 64, 12.0, 40), moe(4, 2, 2, 1, 64, 32, 1.5)),
])
PUPINEX_CONFIGS = {"pxA": (PX_A, 3), "pxB": (PX_B, 5), "pxC": (PX_C, 7), "pxD": (PX_D, 9)}
PUPINEX_PAGE = {"pxA": 16, "pxB": 8, "pxC": 32, "pxD": 16}
PUPINEX_LENGTHS = {"pxA": [1, 2, 15, 16, 17, 40, 75], "pxB": [3, 8, 9, 17, 75, 130], "pxC": [5, 31, 33, 64, 100],
                   "pxD": [1, 2, 33, 190]}

#: factors on the drawn weights by the tensor's last name (matrices only)
SHARP = {"q": 9.0, "k": 9.0, "v": 10.0, "g": 8.0, "o": 5.0, "up": 8.0, "down": 6.0, "gate": 10.0, "sg": 6.0, "a1": 8.0,
         "a2": 12.0, "i": 8.0, "f": 6.0, "embed": 12.0, "bigram": 12.0}
#: factors on vectors by the end of their names, and what is added to them
SHARP_VECTORS = {"q.b": (5.0, 0.0), "k.b": (5.0, 0.0), "v.b": (5.0, 0.0), "o.b": (3.0, 0.0), ".sink": (4.0, 1.0), ".f.b": (1.0, 2.0)}
#: the smallest gap that a choice of experts or groups rests on in the test sequences
MIN_MARGIN = 0.01


def make_pupinex_dir(path: str, cfg: dict, seed: int, sharp: bool = True) -> str:
    from safetensors import safe_open
    from safetensors.torch import save_file
    from tffinfer_amd.weights import write_random_model
    write_random_model(path, json.loads(json.dumps(cfg)), seed, dtype="bfloat16")
    if sharp:
        f = os.path.join(path, "model.safetensors")
        W = {}
        with safe_open(f, "pt") as fh:
            for k in fh.keys():
                W[k] = fh.get_tensor(k)
        for k in list(W):
            last = k.split(".")[-1]
            if last == "router":        # (scores of the same spread whatever the width)
                W[k] = (W[k].float() * 50.0 * cfg["width"] ** -0.5).to(W[k].dtype)
            if last in SHARP and W[k].dim() == 2:
                W[k] = (W[k].float() * SHARP[last]).to(W[k].dtype)
            for tail, (f_, add) in SHARP_VECTORS.items():
                if k.endswith(tail):
                    W[k] = (W[k].float() * f_ + add).to(W[k].dtype)
        save_file(W, f)
    return path


@functools.lru_cache(maxsize=None)
def clear_tokens(model_dir: str, n: int, vocab: int, seed: int) -> tuple:
    """``n`` random tokens whose sequence makes no close call in any mixture of experts.  A token's routers see
    the tokens up to it and no later one, so the first token with a close call is drawn again until none is left."""
    import plain_pupinex as plain
    from helpers import random_tokens
    cfg, W = plain.load(model_dir)
    toks = random_tokens(n, vocab, seed)
    g = torch.Generator().manual_seed(seed + 1)
    for _ in range(60 + 6 * n):
        margins = []
        plain.forward(cfg, W, toks, margins=margins)
        if not margins:
            return tuple(toks)
        close = (torch.stack(margins, 0).min(0).values < MIN_MARGIN).nonzero()
        if close.numel() == 0:
            return tuple(toks)
        toks[int(close[0])] = int(torch.randint(0, vocab, (1,), generator=g))
    raise AssertionError(f"no sequence of {n} tokens without a close call")
