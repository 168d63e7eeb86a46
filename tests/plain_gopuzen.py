"""Plain, slow implementation of the Gopuzen decoder, used only by tests.

Whole sequences, no cache, no batching, one function per mechanism, float64.  It shares no code
with the package: config.json is read with ``json``, the weights with the ``safetensors`` library,
the recurrence goes token by token, and a window with blocks before it is one softmax over all
tokens and all blocks' means with what a position does not see masked out.
"""
from __future__ import annotations

import json
import math
import os

import torch


# ---------------------------------------------------------------- small pieces ---
def unit_rms(x: torch.Tensor, eps: float) -> torch.Tensor:
    """x / sqrt(mean(x^2) + eps) over the last dimension."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def layer_norm(x: torch.Tensor, w: torch.Tensor, b: torch.Tensor, eps: float) -> torch.Tensor:
    """Centred, divided by the root of (mean squared deviation + eps), times w, plus b."""
    d = x - x.mean(-1, keepdim=True)
    return d / torch.sqrt((d * d).mean(-1, keepdim=True) + eps) * w + b


def sigmoid(z):
    return 1.0 / (1.0 + torch.exp(-z))


def silu(z):
    return z * sigmoid(z)


def rotate_pairs(x: torch.Tensor, dims: int, base: float, first_pos: int = 0) -> torch.Tensor:
    """x [T, ..., D]: elements 2i and 2i + 1 (2i < dims) turn by the angle pos * base^(-2i/dims); the
    other elements stay."""
    T = x.shape[0]
    y = x.clone()
    for i in range(dims // 2):
        f = base ** (-2.0 * i / dims)
        a = (torch.arange(first_pos, first_pos + T, dtype=torch.float64) * f).reshape([T] + [1] * (x.dim() - 2))
        u, v = x[..., 2 * i], x[..., 2 * i + 1]
        y[..., 2 * i] = u * torch.cos(a) - v * torch.sin(a)
        y[..., 2 * i + 1] = v * torch.cos(a) + u * torch.sin(a)
    return y


def with_input_conv(h: torch.Tensor, w: torch.Tensor) -> torch.Tensor:
    """h plus a causal convolution of it over time, per channel: the last tap is the token itself."""
    T, taps = h.shape[0], w.shape[1]
    out = h.clone()
    for j in range(taps):
        back = taps - 1 - j
        if back < T:
            out[back:] += w[:, j] * h[:T - back]
    return out


# ---------------------------------------------------------------- attention ---
def query_temperature(T: int, coef: float, every: int) -> torch.Tensor:
    """The factor on the query of each position."""
    return torch.tensor([1.0 + coef * math.log((p + 1) // every + 1) for p in range(T)], dtype=torch.float64)


def block_means(x: torch.Tensor, pool: int) -> torch.Tensor:
    """x [T, ...] -> the means over its whole blocks of ``pool`` rows, [T // pool, ...]."""
    n = x.shape[0] // pool
    return x[:n * pool].reshape(n, pool, *x.shape[1:]).mean(1)


def visible(T: int, size: int, pool: int):
    """(what position i sees of the tokens [T, T], of the blocks [T, T // pool]): tokens j <= i with
    i - j < size; blocks whose last token lies before that window.  size 0: every token j <= i."""
    i, j = torch.arange(T)[:, None], torch.arange(T)[None, :]
    tokens = (j <= i) & ((i - j < size) if size else True)
    if not (size and pool):
        return tokens, torch.zeros(T, 0, dtype=torch.bool)
    last = torch.arange(T // pool)[None, :] * pool + pool - 1
    return tokens, last <= i - size


def grouped_attention(q, k, v, scale: float, size: int = 0, pool: int = 0) -> torch.Tensor:
    """q [T, H, D] on k [T, G, D], v [T, G, E]; head h reads kv head h // (H / G); one softmax over
    everything that is visible."""
    T, H, _ = q.shape
    G, E = k.shape[1], v.shape[2]
    sees = torch.cat(visible(T, size, pool), 1)
    if size and pool:
        k, v = torch.cat([k, block_means(k, pool)]), torch.cat([v, block_means(v, pool)])
    out = torch.zeros(T, H, E, dtype=q.dtype)
    for a in range(H):
        g = a // (H // G)
        s = (q[:, a] @ k[:, g].T) * scale
        out[:, a] = torch.softmax(s.masked_fill(~sees, -math.inf), -1) @ v[:, g]
    return out


def attention_cache(m: dict, P: dict, h: torch.Tensor):
    """The rotated keys [T, G, D] and the values [T, G, E] that a layer keeps."""
    T, G = h.shape[0], m["kv_heads"]
    k = rotate_pairs((h @ P["k"].T).reshape(T, G, m["dim"]), m["rot"]["dims"], m["rot"]["base"])
    return k, (h @ P["v"].T).reshape(T, G, m["vdim"])


def window_attention(m: dict, P: dict, h: torch.Tensor, cache) -> torch.Tensor:
    """``cache``: the keys and values of this layer or of the one it borrows from."""
    T, H = h.shape[0], m["heads"]
    q = rotate_pairs((h @ P["q"].T).reshape(T, H, m["dim"]), m["rot"]["dims"], m["rot"]["base"])
    o = grouped_attention(q, cache[0], cache[1], m["scale"], m["mask"]["size"], m["mask"]["pool"])
    o = o * sigmoid(h @ P["g"].T)[:, :, None]
    return o.reshape(T, -1) @ P["o"].T


def tempered_attention(m: dict, P: dict, h: torch.Tensor) -> torch.Tensor:
    T, H, G = h.shape[0], m["heads"], m["kv_heads"]
    q = (h @ P["q"].T).reshape(T, H, m["dim"])
    q = q * query_temperature(T, m["q_temp"]["coef"], m["q_temp"]["every"])[:, None, None]
    k = (h @ P["k"].T).reshape(T, G, m["dim"])
    v = (h @ P["v"].T).reshape(T, G, m["vdim"])
    return grouped_attention(q, k, v, m["scale"]).reshape(T, -1) @ P["o"].T


# ---------------------------------------------------------------- the recurrence ---
def lightning_states(q, k, v, decay) -> torch.Tensor:
    """q, k [T, H, D], v [T, H, E]: S <- decay S + k v^T, o = S^T q, S zero at the start; o [T, H, E]."""
    T, H, D = q.shape
    E = v.shape[2]
    S = torch.zeros(H, D, E, dtype=q.dtype)
    dec = torch.as_tensor(decay, dtype=torch.float64)[:, None, None]
    out = torch.zeros(T, H, E, dtype=q.dtype)
    for t in range(T):
        S = dec * S + k[t][:, :, None] * v[t][:, None, :]
        out[t] = torch.einsum("hde,hd->he", S, q[t])
    return out


def lightning(m: dict, P: dict, h: torch.Tensor, eps: float) -> torch.Tensor:
    T, H = h.shape[0], m["heads"]
    q = silu(h @ P["q"].T).reshape(T, H, m["dim"])
    k = silu(h @ P["k"].T).reshape(T, H, m["dim"])
    v = silu(h @ P["v"].T).reshape(T, H, m["vdim"])
    o = lightning_states(q, k, v, m["decay"]).reshape(T, -1)
    return (unit_rms(o, eps) * P["norm"] * sigmoid(h @ P["g"].T)) @ P["o"].T


def parallel(m: dict, P: dict, h: torch.Tensor, eps: float) -> torch.Tensor:
    a = tempered_attention(m["left"], sub(P, "left."), h)
    b = lightning(m["right"], sub(P, "right."), h, eps)
    return 0.5 * (unit_rms(a, eps) * P["left.out"] + unit_rms(b, eps) * P["right.out"])


# ---------------------------------------------------------------- feed-forwards ---
def dense_ff(P: dict, h: torch.Tensor) -> torch.Tensor:
    return (silu(h @ P["gate"].T + P["gate.b"]) * (h @ P["up"].T + P["up.b"])) @ P["down"].T + P["down.b"]


def router_scores(P: dict, h: torch.Tensor):
    """(scores, choice scores): a softmax over all experts, and the same with the correction added."""
    s = torch.softmax(h @ P["router"].T, -1)
    return s, s + P["correction"]


def routed_experts(m: dict, P: dict, h: torch.Tensor) -> torch.Tensor:
    """The chosen experts' outputs times their scores; an expert beyond the ones with matrices hands its
    input on."""
    r = m["router"]
    s, c = router_scores(P, h)
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e in torch.topk(c[t], r["top"]).indices.tolist():
            if e >= r["experts"]:
                y = h[t]
            else:
                y = P[f"e{e}.down"] @ (silu(P[f"e{e}.gate"] @ h[t]) * (P[f"e{e}.up"] @ h[t]))
            out[t] += s[t, e] * y
    return out


def router_margins(m: dict, P: dict, h: torch.Tensor) -> torch.Tensor:
    """Per token, the gap between its last chosen choice score and its first rejected one."""
    top, E = m["router"]["top"], m["router"]["experts"] + m["router"]["identity"]
    if top >= E:
        return torch.full((h.shape[0],), math.inf, dtype=h.dtype)
    c = torch.sort(router_scores(P, h)[1], -1, descending=True).values
    return c[:, top - 1] - c[:, top]


def feed_forward(m, P: dict, h: torch.Tensor):
    if m["kind"] == "dense":
        return dense_ff(P, h)
    if m["kind"] == "moe":
        return routed_experts(m, P, h)
    raise ValueError(m["kind"])


# ---------------------------------------------------------------- the model ---
def load(model_dir: str):
    from safetensors import safe_open
    with open(os.path.join(model_dir, "config.json")) as f:
        cfg = json.load(f)
    P = {}
    with safe_open(os.path.join(model_dir, "model.safetensors"), "pt") as f:
        for name in f.keys():
            t = f.get_tensor(name)
            P[name] = t.to(torch.float64) if t.is_floating_point() else t.to(torch.int64)
    return cfg, P


def sub(P: dict, prefix: str) -> dict:
    return {k[len(prefix):]: v for k, v in P.items() if k.startswith(prefix)}


def norm(P: dict, name: str, x: torch.Tensor, eps: float) -> torch.Tensor:
    return layer_norm(x, P[name], P[name + ".b"], eps)


def forward(cfg: dict, P: dict, tokens: list, streams: list | None = None, margins: list | None = None) -> torch.Tensor:
    """float64 logits [T, vocab] of a whole sequence; ``streams`` collects the stream after every
    layer, ``margins`` every router's gaps, a tensor [T] per mixture of experts."""
    eps = cfg["norm"]["eps"]
    x = P["embed"][torch.tensor(tokens)] * cfg["embedding"]["scale"]
    caches = {}
    for i, L in enumerate(cfg["layers"]):
        W = sub(P, f"l{i}.")
        M, m = sub(W, "mix."), L["mixer"]
        h = with_input_conv(norm(W, "norm1", x, eps), W["canon1"])
        if L["type"] == "attention":
            src = m.get("kv_from")
            if src is None:
                caches[i] = attention_cache(m, M, h)
                src = i
            a = window_attention(m, M, h, caches[src])
        elif L["type"] == "parallel":
            a = parallel(m, M, h, eps)
        else:
            raise ValueError(L["type"])
        x = x + norm(W, "norm1b", a, eps) * W["ls1"]
        if L.get("mlp") is not None:
            z = with_input_conv(norm(W, "norm2", x, eps), W["canon2"])
            if margins is not None and L["mlp"]["kind"] == "moe":
                margins.append(router_margins(L["mlp"], sub(W, "mlp."), z))
            x = x + norm(W, "norm2b", feed_forward(L["mlp"], sub(W, "mlp."), z), eps) * W["ls2"]
        if streams is not None:
            streams.append(x.clone())
    return norm(P, "final.norm", x, eps) @ P["head"].T
