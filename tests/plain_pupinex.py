"""Plain, slow implementation of the Pupinex decoder, used only by tests.

Whole sequences, no cache, no batching, one function per mechanism, float64.  It shares no code
with the package: config.json is read with ``json``, the weights with the ``safetensors`` library,
both recurrences go token by token, and what a position does not see is masked out of one softmax.
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


def layer_norm(x: torch.Tensor, w: torch.Tensor, eps: float) -> torch.Tensor:
    """Centred, divided by the root of (mean squared deviation + eps), times w."""
    d = x - x.mean(-1, keepdim=True)
    return d / torch.sqrt((d * d).mean(-1, keepdim=True) + eps) * w


def sigmoid(z):
    return 1.0 / (1.0 + torch.exp(-z))


def log_sigmoid(z):
    return -torch.logaddexp(torch.zeros_like(z), -z)


def silu(z):
    return z * sigmoid(z)


def project(P: dict, name: str, h: torch.Tensor) -> torch.Tensor:
    """h times the matrix ``name``, plus its bias where there is one."""
    y = h @ P[name].T
    return y + P[name + ".b"] if name + ".b" in P else y


def rotate(x: torch.Tensor, dims: int, base: float, interleaved: bool, slower: float = 1.0) -> torch.Tensor:
    """x [T, heads, D]: the first ``dims`` elements of every head turn in pairs by pos * base^(-2i/dims) / slower;
    pair i is (2i, 2i + 1), or (i, i + dims / 2)."""
    T = x.shape[0]
    y = x.clone()
    pos = torch.arange(T, dtype=torch.float64)[:, None]
    for i in range(dims // 2):
        a = pos * (base ** (-2.0 * i / dims) / slower)
        j, k = (2 * i, 2 * i + 1) if interleaved else (i, i + dims // 2)
        u, v = x[:, :, j], x[:, :, k]
        y[:, :, j] = u * torch.cos(a) - v * torch.sin(a)
        y[:, :, k] = v * torch.cos(a) + u * torch.sin(a)
    return y


# ---------------------------------------------------------------- the embedding ---
def bigram_rows(tokens: list, buckets: int, mul_prev: int, mul_cur: int) -> list:
    """The row of the table of pairs that each token adds: the last one for the first token."""
    return [buckets if t == 0 else (tokens[t - 1] * mul_prev + tokens[t] * mul_cur) % buckets for t in range(len(tokens))]


def embedding(cfg: dict, P: dict, tokens: list) -> torch.Tensor:
    b = cfg["embedding"]["bigram"]
    return P["embed"][torch.tensor(tokens)] + P["bigram"][torch.tensor(bigram_rows(tokens, b["buckets"], b["mul_prev"], b["mul_cur"]))]


# ---------------------------------------------------------------- attention ---
def windowed_attention(q, k, v, scale: float, size: int, sinks=None) -> torch.Tensor:
    """q [T, H, D] on k [T, G, D], v [T, G, E]; head h reads kv head h // (H / G); position i sees the j with
    0 <= i - j < size (0: every j <= i); ``sinks`` [H]: a logit without a value."""
    T, H, _ = q.shape
    G, E = k.shape[1], v.shape[2]
    i, j = torch.arange(T)[:, None], torch.arange(T)[None, :]
    sees = (j <= i) & ((i - j < size) if size else True)
    out = torch.zeros(T, H, E, dtype=q.dtype)
    for a in range(H):
        g = a // (H // G)
        s = ((q[:, a] @ k[:, g].T) * scale).masked_fill(~sees, -math.inf)
        if sinks is not None:
            s = torch.cat([s, sinks[a].expand(T, 1)], 1)
        out[:, a] = torch.softmax(s, -1)[:, :T] @ v[:, g]
    return out


def attention(m: dict, P: dict, h: torch.Tensor, eps: float, interleaved: bool, qk_norm: bool) -> torch.Tensor:
    T, H, G = h.shape[0], m["heads"], m["kv_heads"]
    q, k, v = (project(P, n, h) for n in "qkv")
    if qk_norm:
        q, k = unit_rms(q, eps) * P["q.norm"], unit_rms(k, eps) * P["k.norm"]
    q, k, v = q.reshape(T, H, m["dim"]), k.reshape(T, G, m["dim"]), v.reshape(T, G, m["vdim"])
    r = m["rot"]
    slower = r["scaling"]["factor"] if r.get("scaling") else 1.0
    q, k = (rotate(x, r["dims"], r["base"], interleaved, slower) for x in (q, k))
    o = windowed_attention(q, k, v, m["scale"], m["mask"]["size"], P.get("sink"))
    return project(P, "o", o.reshape(T, -1))


# ---------------------------------------------------------------- the recurrences ---
def gla_states(q, k, v, alpha) -> torch.Tensor:
    """q, k, alpha [T, H, D], v [T, H, E]: S <- diag(alpha) S + k v^T, o = S^T q; o [T, H, E]."""
    T, H, D = q.shape
    S = torch.zeros(H, D, v.shape[2], dtype=q.dtype)
    out = torch.zeros(T, H, v.shape[2], dtype=q.dtype)
    for t in range(T):
        S = alpha[t][:, :, None] * S + k[t][:, :, None] * v[t][:, None, :]
        out[t] = torch.einsum("hde,hd->he", S, q[t])
    return out


def gla_decay(m: dict, P: dict, h: torch.Tensor) -> torch.Tensor:
    z = (h @ P["a1"].T) @ P["a2"].T + P["a2.b"]
    return torch.exp(log_sigmoid(z) / m["tau"]).reshape(h.shape[0], m["heads"], m["dim"])


def gla(m: dict, P: dict, h: torch.Tensor, eps: float) -> torch.Tensor:
    T, H, D = h.shape[0], m["heads"], m["dim"]
    q = (h @ P["q"].T).reshape(T, H, D) * D ** -0.5
    k = (h @ P["k"].T).reshape(T, H, D)
    v = (h @ P["v"].T).reshape(T, H, m["vdim"])
    o = unit_rms(gla_states(q, k, v, gla_decay(m, P, h)), eps) * P["norm"]
    return (o.reshape(T, -1) * silu(h @ P["g"].T)) @ P["o"].T


def mlstm_states(q, k, v, i, f, floor: bool = True) -> torch.Tensor:
    """q, k [T, H, D], v [T, H, E], log gates i, f [T, H]: the matrix S and the vector n kept relative to exp(m),
    m the running maximum (zero at the start); ``floor`` False: the denominator without its floor; o [T, H, E]."""
    T, H, D = q.shape
    S = torch.zeros(H, D, v.shape[2], dtype=q.dtype)
    n = torch.zeros(H, D, dtype=q.dtype)
    m = torch.zeros(H, dtype=q.dtype)
    out = torch.zeros(T, H, v.shape[2], dtype=q.dtype)
    for t in range(T):
        new = torch.maximum(f[t] + m, i[t])
        keep, put = torch.exp(f[t] + m - new), torch.exp(i[t] - new)
        m = new
        S = keep[:, None, None] * S + put[:, None, None] * k[t][:, :, None] * v[t][:, None, :]
        n = keep[:, None] * n + put[:, None] * k[t]
        den = (n * q[t]).sum(-1).abs()
        den = (torch.maximum(den, torch.exp(-m)) if floor else den) + 1e-6
        out[t] = torch.einsum("hde,hd->he", S, q[t]) / den[:, None]
    return out


def mlstm_gates(m: dict, P: dict, h: torch.Tensor):
    """(log input gate, log forget gate), both [T, H]."""
    cap = m["gate_cap"]
    return cap * torch.tanh(project(P, "i", h) / cap), log_sigmoid(cap * torch.tanh(project(P, "f", h) / cap))


def mlstm(m: dict, P: dict, h: torch.Tensor, eps: float) -> torch.Tensor:
    T, H, D = h.shape[0], m["heads"], m["dim"]
    q = (h @ P["q"].T).reshape(T, H, D) * D ** -0.5
    k = (h @ P["k"].T).reshape(T, H, D)
    v = (h @ P["v"].T).reshape(T, H, m["vdim"])
    o = unit_rms(mlstm_states(q, k, v, *mlstm_gates(m, P, h)), eps).reshape(T, -1)
    return (o * P["norm"] * sigmoid(h @ P["g"].T)) @ P["o"].T


def mix(kind: str, m: dict, P: dict, h: torch.Tensor, eps: float) -> torch.Tensor:
    if kind == "attention":
        return attention(m, P, h, eps, True, False)
    if kind == "gla":
        return gla(m, P, h, eps)
    if kind == "parallel":
        return (m["left_scale"] * attention(m["left"], sub(P, "left."), h, eps, False, True)
                + m["right_scale"] * mlstm(m["right"], sub(P, "right."), h, eps))
    raise ValueError(kind)


# ---------------------------------------------------------------- feed-forwards ---
def dense_ff(P: dict, h: torch.Tensor, limit: float) -> torch.Tensor:
    g, u = (h @ P["gate"].T).clamp(max=limit), (h @ P["up"].T).clamp(-limit, limit)
    return (g * sigmoid(1.702 * g) * (u + 1.0)) @ P["down"].T


def gated_ff(P: dict, h: torch.Tensor) -> torch.Tensor:
    return (silu(h @ P["gate"].T) * (h @ P["up"].T)) @ P["down"].T


def router_choice(r: dict, s: torch.Tensor):
    """Scores s [E] of one token -> (chosen experts, smallest gap that the choice rests on).  Groups of neighbours
    compete by the sum of their two largest scores; only experts of the best groups take part."""
    E, count, keep = s.numel(), r["groups"]["count"], r["groups"]["keep"]
    size = E // count
    by_group = torch.sort(s.reshape(count, size), 1, descending=True).values[:, :2].sum(1)
    order = torch.sort(by_group, descending=True)
    gap = math.inf if keep == count else float(order.values[keep - 1] - order.values[keep])
    allowed = torch.zeros(E, dtype=torch.bool)
    for g in order.indices[:keep].tolist():
        allowed[g * size:(g + 1) * size] = True
    c = torch.sort(s.masked_fill(~allowed, -math.inf), descending=True)
    if r["top"] < keep * size:
        gap = min(gap, float(c.values[r["top"] - 1] - c.values[r["top"]]))
    return c.indices[:r["top"]].tolist(), gap


def routed_experts(m: dict, P: dict, h: torch.Tensor, gaps: list | None = None) -> torch.Tensor:
    r = m["router"]
    s = sigmoid(h @ P["router"].T)
    out = torch.zeros_like(h)
    gap = []
    for t in range(h.shape[0]):
        chosen, g = router_choice(r, s[t])
        gap.append(g)
        w = s[t, chosen] / (s[t, chosen].sum() + 1e-20) * r["scale"]
        for e, we in zip(chosen, w):
            out[t] += we * gated_ff(sub(P, f"e{e}."), h[t])
    if gaps is not None:
        gaps.append(torch.tensor(gap))
    return out + sigmoid(h @ P["shared.sg"].T) * gated_ff(sub(P, "shared."), h)


def feed_forward(m: dict, P: dict, h: torch.Tensor, gaps: list | None = None) -> torch.Tensor:
    if m["kind"] == "dense":
        return dense_ff(P, h, m["limit"])
    if m["kind"] == "moe":
        return routed_experts(m, P, h, gaps)
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


def run_order(cfg: dict) -> list:
    """(layer, whether the embedding's output is added before it) for every layer that runs."""
    n, loop = len(cfg["layers"]), cfg.get("loop")
    if not loop:
        return [(i, False) for i in range(n)]
    a, b = loop["start"], loop["stop"]
    order = [(i, False) for i in range(a)]
    for t in range(loop["times"]):
        order += [(i, t > 0 and i == a) for i in range(a, b)]
    return order + [(i, False) for i in range(b, n)]


def forward(cfg: dict, P: dict, tokens: list, streams: list | None = None, margins: list | None = None) -> torch.Tensor:
    """float64 logits [T, vocab] of a whole sequence; ``streams`` collects the stream after every layer that runs,
    ``margins`` every router's gaps, a tensor [T] per mixture of experts."""
    eps = cfg["norm"]["eps"]
    start = embedding(cfg, P, tokens)
    x = start.clone()
    for i, again in run_order(cfg):
        L, W = cfg["layers"][i], sub(P, f"l{i}.")
        if again:
            x = x + start
        x = x + mix(L["type"], L["mixer"], sub(W, "mix."), layer_norm(x, W["norm1"], eps), eps)
        if L.get("mlp") is not None:
            x = x + feed_forward(L["mlp"], sub(W, "mlp."), layer_norm(x, W["norm2"], eps), margins)
        if streams is not None:
            streams.append(x.clone())
    return layer_norm(x, P["final.norm"], eps) @ P["embed"].T
