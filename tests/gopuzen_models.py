"""Tiny Gopuzen configurations for the tests, and their model folders.

Sizes differ from layer to layer and between the configurations: one to eight heads, grouped and ungrouped, keys
wider and narrower than values, windows of one token to many with blocks shorter and longer than the window, a
borrowed cache read with windows and blocks of other sizes than its owner's, a part of a head rotated and all of
it, convolutions of one to four taps, a layer without a feed-forward, experts with and without ones that hand their
input on, one of them chosen to all of them.  The random weights are made *sharp* after they are drawn so that a
wrong key, a lost block or state, a window that is one token off or a wrong expert moves the logits by far more
than bfloat16 rounding.
"""
from __future__ import annotations

import functools
import json
import os

import torch


def attn(heads, kv_heads, dim, vdim, scale, mask, rot, kv_from=None):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale,
         "mask": {"size": mask[0], "pool": mask[1]}, "rot": {"dims": rot[0], "base": rot[1]}}
    if kv_from is not None:
        m["kv_from"] = kv_from
    return m


def pair(left, right):
    """left: heads, kv heads, dim, vdim, scale, (coef, every); right: dim, vdim, decays."""
    h, g, d, e, s, (coef, every) = left
    rd, re, dec = right
    return {"left": {"heads": h, "kv_heads": g, "dim": d, "vdim": e, "scale": s, "q_temp": {"coef": coef, "every": every}},
            "right": {"heads": len(dec), "dim": rd, "vdim": re, "decay": list(dec)}}


def dense(ff):
    return {"kind": "dense", "ff": ff}


def moe(experts, identity, top, ff):
    return {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "identity": identity, "top": top}}


def layer(kind, mixer, mlp):
    return {"type": kind, "mixer": mixer, "mlp": mlp}


def model(width, vocab, eps, taps, emb, layers):
    return {"architecture": "Gopuzen", "width": width, "vocab": vocab, "norm": {"eps": eps}, "canon": {"taps": taps},
            "embedding": {"scale": emb}, "layers": layers}


# one cache with two readers whose windows and blocks differ from its owner's (one larger, one smaller, blocks longer
# than a window); a layer without a feed-forward; four taps
GZ_A = model(64, 300, 1e-6, 4, 8.0, [
    layer("attention", attn(4, 2, 16, 24, 0.08, (20, 6), (8, 500.0)), dense(72)),
    layer("parallel", pair((4, 2, 16, 8, 0.25, (0.5, 7)), (8, 12, (0.6, 0.9, 0.99))), moe(5, 3, 2, 24)),
    layer("attention", attn(4, 2, 16, 24, 0.07, (33, 4), (8, 500.0), kv_from=0), moe(3, 1, 1, 16)),
    layer("parallel", pair((2, 1, 24, 32, 0.2, (1.0, 16)), (16, 16, (0.5, 0.95))), None),
    layer("attention", attn(4, 2, 16, 24, 0.1, (5, 12), (8, 500.0), kv_from=0), dense(40)),
])
# the recurrence first; a window of one token with blocks of one; heads that are not grouped; two taps; every expert
# chosen and none that hands its input on; one head, a temperature that rises with every token
GZ_B = model(96, 257, 1e-5, 2, 1.0, [
    layer("parallel", pair((1, 1, 32, 16, 0.15, (0.3, 1)), (24, 40, (0.97,))), moe(3, 0, 3, 16)),
    layer("attention", attn(2, 2, 32, 48, 0.2, (1, 1), (32, 1000000.0)), dense(40)),
    layer("attention", attn(6, 6, 8, 8, 0.1, (9, 3), (4, 50.0)), None),
])
# sizes that are no multiples of 8, five heads on one kv head, three taps, every expert without matrices may be chosen
GZ_C = model(132, 500, 1e-4, 3, 20.0, [
    layer("attention", attn(5, 1, 12, 20, 0.06, (37, 5), (12, 777.0)), moe(4, 3, 3, 28)),
    layer("parallel", pair((3, 1, 20, 12, 0.3, (0.7, 10)), (10, 14, (0.8, 0.3, 0.998))), dense(52)),
    layer("attention", attn(3, 1, 12, 20, 0.06, (16, 8), (12, 777.0), kv_from=0), moe(2, 2, 4, 20)),
    layer("parallel", pair((6, 2, 10, 36, 0.3, (0.2, 40)), (36, 20, (0.9, 0.99))), dense(36)),
])
# head sizes of real models: prompts run on the blocks of the matrix-core attention, with and without keys of blocks;
# one tap (nothing to carry over)
GZ_D = model(256, 400, 1e-5, 1, 16.0, [
    layer("attention", attn(8, 2, 128, 128, 0.012, (40, 16), (64, 10000.0)), dense(128)),
    layer("parallel", pair((8, 2, 64, 128, 0.125, (0.5, 64)), (64, 64, (0.7, 0.9, 0.99, 0.999))), moe(8, 4, 3, 32)),
    layer("attention", attn(8, 2, 128, 128, 0.016, (65, 8), (64, 10000.0), kv_from=0), moe(4, 1, 2, 64)),
    layer("parallel", pair((4, 1, 32, 32, 0.2, (0.25, 32)), (128, 32, (0.98, 0.5))), dense(96)),
])
GOPUZEN_CONFIGS = {"gzA": (GZ_A, 3), "gzB": (GZ_B, 5), "gzC": (GZ_C, 7), "gzD": (GZ_D, 9)}
GOPUZEN_PAGE = {"gzA": 16, "gzB": 8, "gzC": 32, "gzD": 16}
GOPUZEN_LENGTHS = {"gzA": [1, 2, 15, 16, 17, 40, 75], "gzB": [3, 8, 9, 17, 75, 130], "gzC": [5, 31, 33, 64, 100],
                   "gzD": [1, 2, 33, 190]}

#: factors on the drawn weights by the tensor's last name (matrices only)
SHARP = {"q": 9.0, "k": 9.0, "v": 10.0, "g": 8.0, "o": 5.0, "up": 8.0, "down": 8.0, "gate": 10.0, "router": 3.0, "embed": 10.0,
         "head": 3.0, "canon1": 0.6, "canon2": 0.6}
#: factors on vectors by the end of their names
SHARP_VECTORS = {"gate.b": 5.0, "up.b": 5.0, "down.b": 5.0, ".correction": 0.2}
#: the smallest gap between a token's last chosen choice score and its first rejected one in the test sequences
MIN_MARGIN = 0.008


def make_gopuzen_dir(path: str, cfg: dict, seed: int, sharp: bool = True) -> str:
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
            if last in SHARP and W[k].dim() == 2 and W[k].is_floating_point():
                W[k] = (W[k].float() * SHARP[last]).to(W[k].dtype)
            for tail, f_ in SHARP_VECTORS.items():
                if k.endswith(tail):
                    W[k] = (W[k].float() * f_).to(W[k].dtype)
        save_file(W, f)
    return path


@functools.lru_cache(maxsize=None)
def clear_tokens(model_dir: str, n: int, vocab: int, seed: int) -> tuple:
    """``n`` random tokens whose sequence makes no close call in any mixture of experts.  A token's routers see
    the tokens up to it and no later one, so the first token with a close call is drawn again until none is left."""
    import plain_gopuzen as plain
    from helpers import random_tokens
    cfg, W = plain.load(model_dir)
    toks = random_tokens(n, vocab, seed)
    g = torch.Generator().manual_seed(seed + 1)
    for _ in range(60 + 4 * n):
        margins = []
        plain.forward(cfg, W, toks, margins=margins)
        if not margins:
            return tuple(toks)
        close = (torch.stack(margins, 0).min(0).values < MIN_MARGIN).nonzero()
        if close.numel() == 0:
            return tuple(toks)
        toks[int(close[0])] = int(torch.randint(0, vocab, (1,), generator=g))
    raise AssertionError(f"no sequence of {n} tokens without a close call")
