"""The Pupinex design in the engine against the plain implementation: each mechanism alone at the
level of its op or part, then whole models through the step function (whole prompts, decoding
token by token, portions down to two tokens, mixed batches on a pool whose pages and slots are
used again), and greedy generation through the engine's own entry point and scheduler."""
import math

import pytest
import torch

import plain_pupinex as plain
import replay_lib as rl
from helpers import note_error, oracle_logits, rel_err, read_config, tol
from pupinex_models import PUPINEX_LENGTHS, PUPINEX_PAGE, clear_tokens

pytestmark = pytest.mark.gpu
DEV = "cuda:0"
DTYPES = {"float32": torch.float32, "bfloat16": torch.bfloat16}
NAMES = ["pxA", "pxB", "pxC", "pxD"]
BF = torch.bfloat16
F32 = torch.float32


def _ops():
    from tffinfer_amd.kernels import ops
    return ops


def _err(got, ref):
    got, ref = _ops().as_tensor(got).double().cpu(), ref.double().cpu()
    return float((got - ref).abs().max() / ref.abs().max().clamp_min(1e-30))


def _i32(v):
    return torch.tensor(v, dtype=torch.int32, device=DEV)


def _rand(*shape, seed=0, scale=1.0):
    return torch.randn(*shape, generator=torch.Generator().manual_seed(seed)) * scale


def _cuts(T):
    """Ways to bring T tokens: at once, in portions down to two tokens, a portion and then single tokens."""
    rest = T - 3 - 2 - 61
    return [[T], [3, 2, 61] + ([rest] if rest else []), [T - 40] + [1] * 40]


def _steps(cache, plan):
    """Batches of the steps in ``plan``, each a list of (request, tokens or their number); commits after each."""
    from tffinfer_amd.engine.batch import StepEntry, build_step_batch
    for parts in plan:
        parts = [(r, [0] * n if isinstance(n, int) else list(n)) for r, n in parts]
        for r, toks in parts:
            if not cache.has_request(r):
                cache.add_request(r)
            cache.reserve(r, len(toks))
        yield build_step_batch([StepEntry(r, toks, []) for r, toks in parts], cache, DEV)
        for r, toks in parts:
            cache.commit(r, len(toks))


def _view(cache, batch, cache_id):
    from tffinfer_amd.engine.batch import KVView
    gi = cache.group_index(cache_id)
    k, v = cache.kv_tensors(cache_id)
    gt = batch.groups[gi]
    return KVView(k, v, gt.block_tables, gt.slot_mapping, cache.page_size, gi, gt.key_runs, gt.run_start, gt.runs_window,
                  gt.runs_for_blocks, gt.runs_merge, gt.pool_tables)


def _ctx(batch, act_dtype, max_positions=2048):
    from tffinfer_amd.engine.runner import LayerContext
    return LayerContext(_ops(), act_dtype, batch, max_positions)


def _draw(part, seed, weights=None, scale=0.3):
    g = torch.Generator().manual_seed(seed)
    w = {}
    for k, s in part.weight_specs().items():
        t = torch.randn(s.shape, generator=g)
        w[k] = (1 + 0.2 * t) if s.init == "norm" else ((0.5 * t) if s.init in ("norm_offset", "vector") else (t * scale).to(BF))
    w.update(weights or {})
    return w


def _run(part, x, cuts, dtype, page=16):
    """The part over rows x of one request in portions ``cuts``; outputs [T, W].  The pool holds what the request
    needs and no more."""
    from tffinfer_amd.cache import CacheManager
    T = x.shape[0]
    kv = part.cache_spec()
    cache = CacheManager([(0, True, kv, part.state_spec())], page, -(-T // page), 2, dtype=dtype, device=DEV)
    outs, at = [], 0
    for n, batch in zip(cuts, _steps(cache, [[("r", n)] for n in cuts])):
        ctx = _ctx(batch, dtype)
        ctx.state = cache.state_tensors.get(0)
        if kv is not None:
            ctx.kv = _view(cache, batch, 0)
        outs.append(_ops().as_tensor(part.forward(ctx, x[at:at + n].to(dtype).to(DEV))).float())
        at += n
    assert at == T
    cache.check()
    return torch.cat(outs, 0)


# ---------------------------------------------------------------- the embedding ---

@pytest.mark.parametrize("dtype", [F32, BF])
@pytest.mark.parametrize("W,V,bigram", [(64, 50, (97, 13, 5)), (36, 301, (1, 3, 2)), (1032, 77, (4093, 2147483629, 2147483587))])
def test_rows_for_pairs_of_tokens_in_portions_and_batches(W, V, bigram, dtype):
    """Portions of any length and single tokens, requests side by side, slots that are used again: the token before a
    portion comes from the request's state; the first token takes the last row; factors far beyond 32 bits' products."""
    from tffinfer_amd.cache import CacheManager
    from tffinfer_amd.parts import BigramTable, Embedding
    b = BigramTable(bigram[0], W, *bigram[1:])
    emb = Embedding(V, W, bigram=b)
    P = {"embed": _rand(V, W, seed=1).to(BF), "bigram": _rand(bigram[0] + 1, W, seed=2).to(BF)}
    emb.load_weights({"weight": P["embed"]}, dtype, DEV)
    b.load_weights({"weight": P["bigram"]}, dtype, DEV)
    cfg = {"embedding": {"bigram": dict(zip(("buckets", "mul_prev", "mul_cur"), bigram))}}
    P = {k: v.double() for k, v in P.items()}
    cache = CacheManager([(0, True, None, emb.state_spec())], 16, 1, 3, device=DEV)
    g = torch.Generator().manual_seed(5)
    plan = [[("a", 40), ("b", 1)], [("b", 2), ("a", 1)], [("a", 1), ("b", 1)], [("c", 2), ("a", 3), ("b", 1)], [("c", 1)], [("c", 20), ("b", 5)]]
    for _ in range(2):
        total = {r: sum(n for p in plan for q, n in p if q == r) for r in "abc"}
        toks = {r: torch.randint(0, V, (n,), generator=g).tolist() for r, n in total.items()}
        refs = {r: plain.embedding(cfg, P, t) for r, t in toks.items()}
        at = dict.fromkeys("abc", 0)
        given = [[(r, toks[r][o:o + n]) for r, n, o in _spans(plan, i)] for i in range(len(plan))]
        for parts, batch in zip(plan, _steps(cache, given)):
            ctx = _ctx(batch, dtype)
            ctx.state = cache.state_tensors[0]
            out, kept = emb.forward_kept(ctx, batch.token_ids)
            ref = torch.cat([refs[r][at[r]:at[r] + n] for r, n in parts])
            assert _err(out, ref) < 1e-6, parts
            assert torch.equal(out, kept) and out.data_ptr() != kept.data_ptr()
            for r, n in parts:
                at[r] += n
        for r in "abc":
            cache.release(r)
    lone = plain.embedding(cfg, P, toks["a"][40:])      # (what went before a portion matters)
    assert bigram[0] == 1 or _err(lone[:1], refs["a"][40:41]) > 1e-2


def _spans(plan, i):
    """(request, tokens, first place) of step i's entries."""
    at = {}
    for p in plan[:i]:
        for r, n in p:
            at[r] = at.get(r, 0) + n
    return [(r, n, at.get(r, 0)) for r, n in plan[i]]


# ---------------------------------------------------------------- norms and products ---

@pytest.mark.parametrize("W", [48, 321, 1030, 2052, 4100, 4099, 12288])
def test_layer_norm_without_bias_and_rows_added_beside_the_term(W):
    """resid += term + extra (a row each, or one for all) and the layer norm of the sum without a bias; the term may be a
    second result with a factor per row."""
    ops = _ops()
    n, eps = 5, 1e-3
    x, one, rows = (_rand(n, W, seed=i, scale=s) for i, s in ((1, 3.0), (2, 0.7), (3, 2.0)))
    one = one + 2.0                 # (a mean far from zero)
    planes, w, vec, bias, fac = _rand(3, n, W, seed=4), _rand(W, seed=5), _rand(W, seed=6), _rand(W, seed=7), _rand(n, seed=8)
    d = lambda t: t.to(DEV)                  # noqa: E731
    dd = lambda t: t.double()                # noqa: E731
    for term, want in ((None, 0 * dd(x)), (d(one), dd(one)), (d(planes), dd(planes).sum(0)),
                       (ops.OutputTerm(d(planes), bias=d(bias)), dd(planes).sum(0) + dd(bias)),
                       (ops.OutputTerm(d(one), beside=(d(planes), d(fac))), dd(one) + dd(fac)[:, None] * dd(planes).sum(0))):
        for extra, add in ((None, 0 * dd(x)), (d(rows), dd(rows)), (d(vec), dd(vec))):
            total = dd(x) + want + add
            ref = plain.layer_norm(total, dd(w), eps)
            resid = d(x.clone())
            out = ops.add_layernorm(resid, term, d(w), None, eps, F32, extra=extra)
            assert _err(resid, total) < 2e-6 and _err(out, ref) < 5e-6
            assert _err(ops.add_layernorm(d(x.clone()), term, d(w), None, eps, BF, extra=extra).float(), ref) < 5e-3
            resid = d(x.clone())
            y = ops.add_layernorm(resid, term, d(w), None, eps, F32, rows=_i32([4, 0, 2]), extra=extra)
            assert _err(y, ref[[4, 0, 2]]) < 5e-6 and torch.equal(resid.cpu(), x)
    # many rows take another shape of block
    xm, em = _rand(600, W, seed=8), _rand(600, W, seed=9)
    r = d(xm.clone())
    out = ops.add_layernorm(r, None, d(w), None, eps, F32, extra=d(em))
    assert _err(r, dd(xm) + dd(em)) < 2e-6 and _err(out, plain.layer_norm(dd(xm) + dd(em), dd(w), eps)) < 5e-6


@pytest.mark.parametrize("limit", [0.7, 3.0, 1e4])
@pytest.mark.parametrize("M,I,K", [(1, 24, 64), (8, 200, 320), (16, 48, 132), (33, 1000, 256), (150, 136, 72), (300, 512, 1024), (40, 64, 4096),
                                   (12, 4200, 512)])
def test_clamps_in_the_gated_product(M, I, K, limit):
    """g sigmoid(1.702 g) (u + 1) of clamped g and u, whatever kernel the product's sizes select (few rows, tiles, K split
    over blocks); the slope and what is added to u are arguments."""
    ops = _ops()
    x, g, u = (_rand(*s, seed=i).to(BF) for i, s in ((1, (M, K)), (2, (I, K)), (3, (I, K))))
    g, u = (g.float() * 2 * K ** -0.5).to(BF), (u.float() * 2 * K ** -0.5).to(BF)
    a, b = (x.double() @ g.double().T).clamp(max=limit), (x.double() @ u.double().T).clamp(-limit, limit)
    for alpha, off in ((1.702, 1.0), (1.0, 0.0), (0.5, -2.0)):
        ref = a * plain.sigmoid(alpha * a) * (b + off)
        act = (limit, alpha, off)
        out = ops.linear(x.to(DEV), ops.pack_gate_up(g.to(DEV), u.to(DEV), act))
        assert _err(out.float(), ref) < 6e-3
        gu = ops.linear(x.float().to(DEV), torch.cat([g, u]).float().to(DEV))
        assert _err(ops.swiglu(gu, act=act), ref) < 8e-6
    plain_act = ops.linear(x.to(DEV), ops.pack_gate_up(g.to(DEV), u.to(DEV)))
    full = (x.double() @ g.double().T, x.double() @ u.double().T)
    assert _err(plain_act.float(), plain.silu(full[0]) * full[1]) < 6e-3


@pytest.mark.parametrize("E,top,groups,keep,ff,shared,scale", [
    (8, 2, 4, 2, 24, 24, 2.5), (6, 3, 1, 1, 16, 40, 1.0), (5, 2, 5, 3, 8, 20, 0.5), (12, 4, 4, 3, 32, 8, 2.0),
    (256, 8, 8, 4, 8, 16, 2.5), (3, 3, 1, 1, 16, 130, 1.0), (90, 1, 30, 1, 8, 8, 1.0)])
def test_experts_from_the_best_groups_beside_a_shared_one(E, top, groups, keep, ff, shared, scale):
    """The choice and its weights against the plain router (groups of one expert to many), the shared expert narrower,
    as wide and wider than the others, experts by pairs and by tiles; a token's result does not depend on its batch."""
    from tffinfer_amd.parts import RoutedExperts
    ops = _ops()
    T, W = 40, 48
    part = RoutedExperts(W, ff, E, top, None, act_alpha=1.0, up_offset=0.0, correction=False, groups=groups, keep_groups=keep,
                         weight_scale=scale, shared=shared)
    w, ws = _draw(part, E + top), _draw(part.shared_expert, E + top + 1)
    w["router"] = (w["router"].float() * 0.8).to(BF)
    P = {k: v.double() for k, v in w.items()} | {"shared." + k: v.double() for k, v in ws.items()}
    m = {"router": {"top": top, "experts": E, "groups": {"count": groups, "keep": keep}, "scale": scale}}
    x = _rand(400, W, seed=E).to(BF).float()
    # rows whose choice rests on no close call
    s = plain.sigmoid(x.double() @ P["router"].T)
    x = x[[i for i in range(400) if plain.router_choice(m["router"], s[i])[1] > 1e-4][:T]]
    assert x.shape[0] == T
    s = plain.sigmoid(x.double() @ P["router"].T)
    want = [plain.router_choice(m["router"], s[t])[0] for t in range(T)]
    ref = plain.routed_experts(m, P, x.double())
    idx, wts, gate = ops.route_topk(x.to(DEV), torch.cat([w["router"], w["shared.sg"]]).float().to(DEV), None, top, groups=groups,
                              keep_groups=keep, scale=scale, shared=True)
    assert torch.equal(idx.cpu().long(), torch.tensor(want))
    chosen = torch.gather(s, 1, torch.tensor(want))
    assert _err(wts, chosen / chosen.sum(1, keepdim=True) * scale) < 2e-6
    assert _err(gate, plain.sigmoid(x.double() @ P["shared.sg"].T)[:, 0]) < 2e-6
    if keep < groups < E:       # the groups matter
        free = dict(m["router"], groups={"count": groups, "keep": groups})
        assert any(set(plain.router_choice(free, s[t])[0]) != set(want[t]) for t in range(T))
    for dtype, limit in ((F32, 2e-5), (BF, 3e-2)):
        part.load_weights(w, dtype, DEV)
        part.shared_expert.load_weights(ws, dtype, DEV)
        ctx = _ctx(None, dtype)
        full = ops.as_tensor(part.forward(ctx, x.to(dtype).to(DEV)))
        assert _err(full, ref) < limit
        alone = ops.as_tensor(part.forward(ctx, x[7:8].to(dtype).to(DEV)))
        assert _err(alone[0], ref[7]) < limit


# ---------------------------------------------------------------- attention ---

def _attention(W, H, G, D, E, scale, size, rot, dtype, seed, interleaved=True, factor=None, qk_norm=False, sinks=True, out_bias=True,
               weights=None):
    """(part, the plain functions' mixer entry, the plain functions' weights)."""
    from tffinfer_amd.config.base import PartSpec
    from tffinfer_amd.parts import GroupedAttention
    args = {"head_dim": D, "theta": rot[1], "pairing": "interleaved" if interleaved else "half", "rotary_dim": rot[0]} if rot else None
    pos = None if not rot else PartSpec("rope", args) if factor is None else PartSpec("rope_linear", dict(args, factor=factor))
    att = GroupedAttention(hidden_size=W, num_heads=H, num_kv_heads=G, head_dim=D, value_dim=E, position=pos, scale=scale, window=size,
                           bias=True, output_bias=out_bias, qk_norm_eps=1e-3 if qk_norm else None, sinks=sinks)
    w = _draw(att, seed, weights)
    att.load_weights(w, dtype, DEV)
    m = {"heads": H, "kv_heads": G, "dim": D, "vdim": E, "scale": scale, "mask": {"size": size},
         "rot": {"dims": rot[0], "base": rot[1]} if rot else {"dims": 0, "base": 1.0}}
    if factor is not None:
        m["rot"]["scaling"] = {"factor": factor}
    return att, m, {k: v.double() for k, v in w.items()}


SIZES = [(4, 2, 16, 24, 20, (8, 500.0), 16),      # a part of a head rotated, values wider than keys
         (2, 2, 32, 48, 1, (32, 1e6), 8),         # a window of one token
         (5, 1, 12, 20, 37, (12, 777.0), 32),     # no multiples of 8, five heads on one kv head
         (6, 6, 9, 7, 9, (4, 50.0), 16),          # heads that are not grouped, odd sizes
         (8, 2, 128, 64, 64, (64, 1e4), 16),      # the sizes of real models
         (16, 1, 64, 64, 33, (64, 1e4), 16),
         (2, 1, 192, 64, 40, (32, 1e4), 16),
         (1, 1, 16, 288, 30, (16, 100.0), 16),    # values beyond the matrix-core attention's sizes
         (4, 2, 16, 24, 0, (16, 100.0), 8)]       # every key


@pytest.mark.parametrize("dtype,limit", [(F32, 3e-5), (BF, 4e-2)])
@pytest.mark.parametrize("H,G,D,E,size,rot,page", SIZES)
def test_attention_with_biases_and_sinks(H, G, D, E, size, rot, page, dtype, limit):
    """A prompt in one step, as portions down to two tokens, and as a portion followed by single tokens."""
    W, T = 48, 230
    att, m, P = _attention(W, H, G, D, E, 0.4 * D ** -0.5, size, rot, dtype, H * D + E)
    x = _rand(T, W, seed=7).to(BF).float()
    ref = plain.attention(m, P, x.double(), 1e-3, True, False)
    for cuts in _cuts(T):
        err = _err(_run(att, x, cuts, dtype, page), ref)
        assert err < limit, f"cut {cuts[:3]}: {err:.3e}"
    for lost in ("sink", "q.b", "k.b", "v.b", "o.b"):
        other = dict(P, **{lost: P[lost] * 0 - (30.0 if lost == "sink" else 0.0)})
        assert _err(plain.attention(m, other, x.double(), 1e-3, True, False), ref) > 5e-4, lost


@pytest.mark.parametrize("dtype,limit", [(F32, 3e-5), (BF, 4e-2)])
@pytest.mark.parametrize("H,G,D,E,size,rot,page", SIZES)
def test_attention_with_a_norm_over_the_whole_of_q_and_k(H, G, D, E, size, rot, page, dtype, limit):
    W, T = 48, 230
    att, m, P = _attention(W, H, G, D, E, 1.5 * D ** -0.5, size, rot, dtype, H + D + E, interleaved=False, factor=4.0, qk_norm=True,
                           sinks=False, out_bias=False)
    x = _rand(T, W, seed=8).to(BF).float()
    x = x * torch.linspace(0.2, 3.0, T)[:, None]            # (rows of unequal size)
    x = x.to(BF).float()
    ref = plain.attention(m, P, x.double(), 1e-3, False, True)
    for cuts in _cuts(T):
        err = _err(_run(att, x, cuts, dtype, page), ref)
        assert err < limit, f"cut {cuts[:3]}: {err:.3e}"
    if H > 1 and size != 1:     # the norm is one over all heads, not one a head
        q = plain.unit_rms((x.double() @ P["q"].T + P["q.b"]).reshape(T, H, D), 1e-3)
        assert _err(q.reshape(T, -1), plain.unit_rms(x.double() @ P["q"].T + P["q.b"], 1e-3)) > 1e-2


def _loud(T, i, loud, decode_tail, size, dtype, sink=-30.0):
    """An attention of one head without rotation on rows in which token ``loud``'s key stands out for query i only;
    returns (engine's row i, plain row i, plain row i without the loud key)."""
    W = D = 8
    eye, pick = torch.eye(D), torch.eye(D)
    pick[3], pick[4] = eye[4], 0            # (a query lies along the keys' axis 3 if its row does along axis 4)
    z = torch.zeros
    fixed = {"q": pick.to(BF), "k": eye.to(BF), "v": _rand(12, W, seed=3).to(BF), "o": _rand(W, 12, seed=4).to(BF), "q.b": z(D), "k.b": z(D),
             "v.b": z(12), "sink": torch.tensor([sink])}
    att, m, P = _attention(W, 1, 1, D, 12, 6.0, size, None, dtype, 1, out_bias=False, weights=fixed)
    x = _rand(T, W, seed=9, scale=0.05).to(BF).float()
    x[:, 3:5] = 0
    x[loud] = 0
    x[loud, 3], x[loud, 5], x[loud, 6] = 4.0, -4.0, 4.0
    x[i, 4] = 4.0
    without = x.clone()
    without[loud] = 0
    both = [plain.attention(m, P, y.double(), 1e-3, True, False)[i] for y in (x, without)]
    cuts = [i] + [1] * (T - i) if decode_tail else [T]
    return _run(att, x, cuts, dtype)[i], both[0], both[1]


@pytest.mark.parametrize("decode", [False, True])
@pytest.mark.parametrize("size", [1, 2, 7, 16, 24, 33, 150])
def test_a_loud_key_at_the_edges_of_the_window(size, decode):
    """One key whose score with the last query stands far out: the window's first and second key, the last key before it,
    keys at the borders of pages, the first tokens of the sequence.  Where the key is seen its loss moves the plain
    result; where it is not, the result is the one without it."""
    for i in (150, 159):
        lo = max(0, i - size + 1)
        for j in {lo, lo + 1, lo - 1, lo - 2, i - 1, 0, 1, 15, 16, 31, 32, 143, 144} - {i}:
            if not 0 <= j < i:
                continue
            out, ref, lost = _loud(160, i, j, decode, size, F32)
            assert _err(out, ref) < 3e-5, (i, j)
            moved = float((ref - lost).abs().max() / ref.abs().max())
            assert (moved > 0.5) if j >= lo else (moved < 1e-9), (i, j, moved)
    out, ref, _ = _loud(160, 155, max(0, 155 - size + 1) if size > 1 else 3, decode, size, BF)
    assert _err(out, ref) < 3e-2


@pytest.mark.parametrize("sink", [-5.0, 3.0, 90.0, 98.0])
def test_a_sink_as_loud_as_the_loudest_key(sink):
    """The sink's exponential stands beside the keys', counted once, whatever runs the keys are split into."""
    for decode in (False, True):
        for dtype, limit in ((F32, 3e-5), (BF, 3e-2)):
            out, ref, _ = _loud(160, 158, 140, decode, 24, dtype, sink=sink)        # (the loud key's score is 96)
            silent = _loud(160, 158, 140, decode, 24, dtype)[1]
            scale = max(float(ref.abs().max()), 1e-3 * float(silent.abs().max()))
            assert float((out.double().cpu() - ref).abs().max()) / scale < limit
    if sink > 80:
        assert float((ref - silent).abs().max() / silent.abs().max()) > 1e-3


# ---------------------------------------------------------------- the recurrences ---

def _gla(W, H, D, E, tau, rank, dtype, seed, weights=None, eps=1e-5):
    from tffinfer_amd.parts import GatedLinearAttention
    part = GatedLinearAttention(W, H, D, E, tau=tau, decay_rank=rank, norm_eps=eps)
    w = _draw(part, seed, weights)
    part.load_weights(w, dtype, DEV)
    return part, {"heads": H, "dim": D, "vdim": E, "tau": tau}, {k: v.double() for k, v in w.items()}


def _mlstm(W, H, D, E, cap, dtype, seed, weights=None, eps=1e-5, shift=0.0):
    from tffinfer_amd.parts import MatrixMemory
    part = MatrixMemory(W, H, D, E, gate_cap=cap, norm_eps=eps)
    w = _draw(part, seed, weights)
    w["f.b"] = w["f.b"] + shift
    part.load_weights(w, dtype, DEV)
    return part, {"heads": H, "dim": D, "vdim": E, "gate_cap": cap}, {k: v.double() for k, v in w.items()}


REC_CUTS = [[64, 65, 63, 38], [128, 102], [11, 12, 13, 16, 48, 130]]


@pytest.mark.parametrize("dtype,limit", [(F32, 5e-5), (BF, 4e-2)])
@pytest.mark.parametrize("H,D,E,tau,rank", [(3, 8, 12, 4.0, 6), (1, 24, 8, 1.0, 1), (2, 10, 14, 16.0, 33), (2, 64, 64, 16.0, 16),
                                            (1, 128, 40, 8.0, 70), (1, 32, 130, 16.0, 16), (2, 256, 16, 2.0, 4), (1, 130, 260, 16.0, 9),
                                            (1, 7, 1, 3.0, 2), (4, 1, 33, 1.0, 3)])
def test_recurrence_with_a_decay_per_key_channel(H, D, E, tau, rank, dtype, limit):
    W, T, eps = 48, 230, 1e-5 if E > 1 else 0.1       # (a norm over one channel leaves little but its sign)
    part, m, P = _gla(W, H, D, E, tau, rank, dtype, D + E, eps=eps)
    x = _rand(T, W, seed=6).to(BF).float()
    ref = plain.gla(m, P, x.double(), eps)
    for cuts in _cuts(T) + REC_CUTS:
        err = _err(_run(part, x, cuts, dtype), ref)
        assert err < limit, f"cut {cuts[:3]}: {err:.3e}"
    assert _err(plain.gla(dict(m, tau=tau * 1.3), P, x.double(), eps), ref) > 1e-3


@pytest.mark.parametrize("shift", [-60.0, -20.0, 30.0])
def test_decays_near_nothing_and_near_one(shift):
    """Channels that forget a token at once (sums of their logarithms far below what a 32-bit exponential holds) beside
    channels that forget nothing, in chunks and token by token."""
    W, T, eps, H, D, E = 32, 200, 1e-5, 2, 20, 12
    bias = _rand(H * D, seed=3)
    bias[::3] += shift
    bias[1::3] += 12.0
    part, m, P = _gla(W, H, D, E, 1.0, 5, F32, 2, weights={"a2.b": bias}, eps=eps)
    x = _rand(T, W, seed=4).to(BF).float()
    alpha = plain.gla_decay(m, P, x.double())
    assert float(alpha[:, :, 1::3].min()) > 0.9 or float(alpha.max()) > 0.999
    assert shift > 0 or float(alpha.min()) < 1e-8
    ref = plain.gla(m, P, x.double(), eps)
    for cuts in ([T], [3, 2, 61, 134], [100] + [1] * 100):
        out = _run(part, x, cuts, F32)
        assert torch.isfinite(out).all() and _err(out, ref) < 5e-5, cuts[:3]


@pytest.mark.parametrize("dtype,limit", [(F32, 5e-5), (BF, 4e-2)])
@pytest.mark.parametrize("H,D,E,cap,shift", [(3, 8, 12, 10.0, 2.0), (1, 24, 8, 1.0, 0.0), (2, 10, 14, 15.0, 4.0), (2, 64, 64, 15.0, 3.0),
                                             (1, 128, 40, 5.0, 6.0), (1, 32, 130, 15.0, 2.0), (2, 256, 16, 15.0, 1.0),
                                             (1, 130, 260, 15.0, 5.0), (1, 7, 1, 3.0, -2.0), (4, 1, 33, 8.0, 2.0)])
def test_recurrence_with_exponential_gates(H, D, E, cap, shift, dtype, limit):
    W, T, eps = 48, 230, 1e-5 if E > 1 else 0.1
    part, m, P = _mlstm(W, H, D, E, cap, dtype, D + E, eps=eps, shift=shift)
    x = _rand(T, W, seed=6).to(BF).float()
    ref = plain.mlstm(m, P, x.double(), eps)
    for cuts in _cuts(T) + REC_CUTS:
        err = _err(_run(part, x, cuts, dtype), ref)
        assert err < limit, f"cut {cuts[:3]}: {err:.3e}"
    assert _err(plain.mlstm(dict(m, gate_cap=cap * 0.7), P, x.double(), eps), ref) > 1e-3


@pytest.mark.parametrize("i_shift,f_shift", [(0.0, 60.0), (-40.0, 60.0), (40.0, 60.0), (0.0, -60.0), (40.0, -60.0), (-6.0, 3.0), (6.0, 3.0)])
def test_exponential_gates_at_their_limits(i_shift, f_shift):
    """Input gates at plus and minus the cap, forget gates that keep everything or nothing: the running maximum and the
    floor exp(-m) of the denominator show in the outputs before the norm."""
    from tffinfer_amd.kernels import lib, ops
    from tffinfer_amd.cache import CacheManager
    from tffinfer_amd.parts.base import StateSpec
    W, T, H, D, E, cap, eps = 1, 150, 2, 12, 8, 15.0, 3e-2
    q, k, v, g = (_rand(T, H, n, seed=s) for s, n in ((1, D), (2, D), (3, E), (4, E)))
    zi, zf = _rand(T, H, seed=5, scale=8.0) + i_shift, _rand(T, H, seed=6, scale=4.0) + f_shift
    dd = lambda t: t.double()                # noqa: E731
    i, f = cap * torch.tanh(dd(zi) / cap), plain.log_sigmoid(cap * torch.tanh(dd(zf) / cap))
    o = plain.mlstm_states(dd(q) * D ** -0.5, dd(k), dd(v), i, f)
    # (a norm with a large eps leaves the outputs' size in)
    ref = (plain.unit_rms(o, eps) * plain.sigmoid(dd(g))).reshape(T, -1)
    bare = plain.mlstm_states(dd(q) * D ** -0.5, dd(k), dd(v), i, f, floor=False)
    if i_shift < -1:
        assert _err((plain.unit_rms(bare, eps) * plain.sigmoid(dd(g))).reshape(T, -1), ref) > 0.05       # the floor matters
    proj = torch.cat([t.reshape(T, -1) for t in (q, k, v, g, zi, zf)], 1).to(DEV)
    cols = {"q": 0, "k": H * D, "v": 2 * H * D, "gate": 2 * H * D + H * E, "ig": 2 * H * D + 2 * H * E, "fg": 2 * H * D + 2 * H * E + H}
    n_state = H * (E + 1) * D + H
    cache = CacheManager([(0, True, None, StateSpec((n_state,)))], 16, 1, 2, device=DEV)
    z, one = torch.zeros(H, device=DEV), torch.ones(E, device=DEV)
    for chunked in (False, True, None):
        for cuts in ([T], [70, 2, 13, 65], [1] * 20 + [130]):
            outs, at = [], 0
            for n, batch in zip(cuts, _steps(cache, [[("r", n)] for n in cuts])):
                out = torch.empty(n, H * E, device=DEV)
                ops.exp_gate_recurrence(proj[at:at + n], cols, z, z, cap, one, eps, cache.state_tensors[0], batch, H, D, E, out,
                                        q_scale=D ** -0.5, chunked=chunked)
                outs.append(out)
                at += n
            cache.release("r")
            got = torch.cat(outs)
            assert torch.isfinite(got).all() and _err(got, ref) < 5e-5, (chunked, cuts[:3])
    assert lib.LR_EXP == 1


@pytest.mark.parametrize("kind", ["gla", "mlstm"])
def test_a_loud_token_far_back_in_a_recurrence(kind):
    """What a token far back wrote into the state is read by the last token, in a prompt and decoded, and a state lost
    at a portion's border would show."""
    W, D, E, T, eps = 16, 8, 8, 400, 1e-5
    if kind == "gla":
        part, m, P = _gla(W, 2, D, E, 16.0, 3, F32, 3, weights={"a2.b": torch.full((2 * D,), 9.0)}, eps=eps)
    else:
        part, m, P = _mlstm(W, 2, D, E, 15.0, F32, 3, weights={"f.b": torch.full((2,), 9.0)}, eps=eps)
    run = plain.gla if kind == "gla" else plain.mlstm
    x = _rand(T, W, seed=4, scale=0.1).to(BF).float()
    x[30] *= 60.0
    ref = run(m, P, x.double(), eps)
    calm = x.clone()
    calm[30] *= 0
    assert _err(run(m, P, calm.double(), eps)[-1], ref[-1]) > 0.1
    for cuts in ([T], [31] + [1] * (T - 31), [100, 2, 200, 98]):
        assert _err(_run(part, x, cuts, F32), ref) < 5e-5, cuts[:3]


@pytest.mark.parametrize("sizes", [((4, 2, 16, 24), (3, 12, 20)), ((3, 3, 9, 7), (5, 6, 10)), ((2, 1, 20, 12), (1, 64, 80))])
def test_two_mixers_side_by_side_and_batches_of_unequal_requests(sizes):
    """The scaled sum of an attention and a matrix memory: three requests of unequal length in shared steps give what
    each gives alone; pages and slots are freed and used again."""
    from tffinfer_amd.cache import CacheManager
    from tffinfer_amd.config.base import PartSpec
    from tffinfer_amd.parts import MixerPair
    W, eps, page, size = 40, 1e-4, 8, 11
    (H, G, D, E), (rh, rd, re) = sizes
    mixer = MixerPair(W, PartSpec("grouped_attention", {
        "hidden_size": W, "num_heads": H, "num_kv_heads": G, "head_dim": D, "value_dim": E, "scale": 0.4, "window": size, "bias": True,
        "qk_norm_eps": eps, "position": PartSpec("rope_linear", {"head_dim": D, "theta": 100.0, "factor": 3.0, "rotary_dim": D - D % 2})}),
        PartSpec("matrix_memory", {"hidden_size": W, "num_heads": rh, "head_dim": rd, "value_dim": re, "gate_cap": 9.0, "norm_eps": eps}),
        left_scale=0.7, right_scale=1.3)
    assert mixer.joint
    w = _draw(mixer, 17)
    m = {"left": {"heads": H, "kv_heads": G, "dim": D, "vdim": E, "scale": 0.4, "mask": {"size": size},
                  "rot": {"dims": D - D % 2, "base": 100.0, "scaling": {"factor": 3.0}}},
         "right": {"heads": rh, "dim": rd, "vdim": re, "gate_cap": 9.0}, "left_scale": 0.7, "right_scale": 1.3}
    P = {k: v.double() for k, v in w.items()}
    lengths = {"a": 60, "b": 41, "c": 7}
    xs = {r: _rand(n, W, seed=n).to(BF).float() for r, n in lengths.items()}
    refs = {r: plain.mix("parallel", m, P, x.double(), eps) for r, x in xs.items()}
    for dtype, limit in ((F32, 5e-5), (BF, 4e-2)):
        mixer.load_weights(w, dtype, DEV)
        cache = CacheManager([(0, True, mixer.cache_spec(), mixer.state_spec())], page, 15, 3, dtype=dtype, device=DEV)
        for plan in ([[("a", 35), ("b", 40)], [("a", 25), ("b", 1), ("c", 7)]],
                     [[("b", 2), ("a", 30)], [("c", 1), ("b", 20)], [("c", 1), ("a", 1), ("b", 1)], [("a", 29), ("b", 18), ("c", 5)]]):
            at = dict.fromkeys("abc", 0)
            for parts, batch in zip(plan, _steps(cache, plan)):
                ctx = _ctx(batch, dtype)
                ctx.kv, ctx.state = _view(cache, batch, 0), cache.state_tensors[0]
                rows = torch.cat([xs[r][at[r]:at[r] + n] for r, n in parts]).to(dtype).to(DEV)
                out = mixer.forward(ctx, rows)
                assert _err(out, torch.cat([refs[r][at[r]:at[r] + n] for r, n in parts])) < limit, parts
                for r, n in parts:
                    at[r] += n
            for r in "abc":
                cache.release(r)
            cache.check()


@pytest.mark.parametrize("dtype,limit", [(F32, 3e-5), (BF, 3e-2)])
def test_long_contexts_decode_beside_a_portion(dtype, limit):
    """Requests of 300 to 900 tokens that decode beside another's portion get the kernel that splits keys among waves: the
    sink counts once all the same."""
    from tffinfer_amd.cache import CacheManager
    W, page = 40, 16
    att, m, P = _attention(W, 8, 2, 64, 64, 0.04, 700, (64, 1000.0), dtype, 41, weights={"sink": torch.linspace(4.0, 9.0, 8)})
    lengths = {"a": 901, "b": 302, "c": 90}
    xs = {r: _rand(n, W, seed=n).to(BF).float() for r, n in lengths.items()}
    refs = {r: plain.attention(m, P, x.double(), 1e-3, True, False) for r, x in xs.items()}
    cache = CacheManager([(0, True, att.cache_spec(), None)], page, 90, 3, dtype=dtype, device=DEV)
    plan = [[("a", 899), ("b", 300)], [("a", 1), ("b", 1), ("c", 80)], [("b", 1), ("c", 9)], [("a", 1), ("c", 1)]]
    at = dict.fromkeys("abc", 0)
    for parts, batch in zip(plan, _steps(cache, plan)):
        ctx = _ctx(batch, dtype)
        ctx.kv = _view(cache, batch, 0)
        rows = torch.cat([xs[r][at[r]:at[r] + n] for r, n in parts]).to(dtype).to(DEV)
        out = _ops().as_tensor(att.forward(ctx, rows))
        assert _err(out, torch.cat([refs[r][at[r]:at[r] + n] for r, n in parts])) < limit, parts
        for r, n in parts:
            at[r] += n
    lost = plain.attention(m, dict(P, sink=P["sink"] - 30), xs["a"].double(), 1e-3, True, False)
    assert _err(lost[-1], refs["a"][-1]) > 0.05


# ---------------------------------------------------------------------- whole models ---

def requests_for(name, model_dir):
    V = read_config(model_dir)["vocab"]
    # (sequences in which no choice of experts is a close call that rounding could turn)
    return {f"{name}{i}": list(clear_tokens(model_dir, n, V, 3000 + n)) for i, n in enumerate(PUPINEX_LENGTHS[name])}


def make_runner(model_dir, dtype, page_size, num_pages, max_seqs=4, use_graphs=False):
    from tffinfer_amd.engine.runner import ModelRunner
    from tffinfer_amd.models import load_model
    model = load_model(model_dir, DTYPES[dtype], DEV)
    return ModelRunner(model, page_size=page_size, num_pages=num_pages, max_seqs=max_seqs, max_model_len=512,
                       use_graphs=use_graphs)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", NAMES)
def test_residual_stream_after_every_layer(pupinex_dirs, name, dtype):
    """Layer by layer, so that a fault names its layer.  A block leaves its last sublayer's output to the norm
    after it; the stream after a layer is the stream plus what is pending."""
    from tffinfer_amd.engine.batch import StepEntry, build_step_batch
    from tffinfer_amd.engine.runner import StepContext
    d = pupinex_dirs[name]
    toks = list(clear_tokens(d, PUPINEX_LENGTHS[name][-1], read_config(d)["vocab"], 3000 + PUPINEX_LENGTHS[name][-1]))[:70]
    want = []
    plain.forward(*plain.load(d), toks, want)
    runner = make_runner(d, dtype, PUPINEX_PAGE[name], 16)
    model, ops = runner.model, runner.ops
    runner.add_request("a")
    e = [StepEntry("a", toks, [])]
    runner.reserve(e)
    batch = build_step_batch(e, runner.cache, runner.device, runner._pinned)
    ctx = StepContext(ops, runner.act_dtype, batch, runner.max_model_len, runner._calls, runner.cache)
    resid, pending, _ = model.run_items(ctx, ["embed"], None, None)
    assert len(model.schedule) == len(want)
    for it in range(len(want)):
        resid, pending, _ = model.run_items(ctx, [it], resid, pending)
        after = resid + ops.as_tensor(pending) if pending is not None else resid
        err = _err(after, want[it])
        assert err < (4e-5 if dtype == "float32" else 5e-2), f"layer run {it}: {err:.3e}"


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", NAMES)
@pytest.mark.parametrize("mode", ["whole", "tail", "chunks", "mixed"])
def test_replay_modes(pupinex_dirs, name, dtype, mode):
    model_dir = pupinex_dirs[name]
    reqs = requests_for(name, model_dir)
    steps = {"whole": rl.trace_whole, "tail": rl.trace_tail, "chunks": rl.trace_chunks,
             "mixed": rl.trace_mixed}[mode](reqs)
    ps = PUPINEX_PAGE[name]
    # the pool holds what is live at the worst moment and no more, so pages and slots are used again
    num_pages = rl.max_live_tokens(steps, unit=ps) // ps
    runner = make_runner(model_dir, dtype, ps, num_pages)
    results = rl.run_steps_in_process(runner, steps)
    worst = rl.check_against_oracle(model_dir, reqs, steps, results, tol(dtype, name), dtype)
    print(f"{name} {dtype} {mode}: worst rel. error {worst:.3e} over {len(steps)} steps, {num_pages} pages")
    assert all(g.pool.num_used == 0 for g in runner.cache.groups)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", ["pxA", "pxD"])
@pytest.mark.parametrize("pieces", [False, True])
def test_long_decoding_through_captured_graphs(pupinex_dirs, name, dtype, pieces):
    """Three requests decode many tokens each as replays of captured HIP graphs beside eager prompt steps; also with a
    layer that cannot be captured, so that the step is cut into pieces around it and the embedding's output crosses them."""
    model_dir = pupinex_dirs[name]
    V = read_config(model_dir)["vocab"]
    lengths = (55, 61, 70) if name == "pxA" else (90, 101, 111)
    reqs = {f"g{i}": list(clear_tokens(model_dir, n, V, 300 + n)) for i, n in enumerate(lengths)}
    steps = rl.trace_mixed(reqs, max_live=3, prompt_frac=0.1, want_all=True)
    ps = PUPINEX_PAGE[name]
    from tffinfer_amd.engine.runner import ModelRunner
    from tffinfer_amd.models import load_model
    model = load_model(model_dir, DTYPES[dtype], DEV)
    if pieces:
        model.blocks[1].mixer.graph_safe = False
        assert len(model.graph_pieces()) > 2
    runner = ModelRunner(model, page_size=ps, num_pages=rl.max_live_tokens(steps, unit=ps) // ps, max_seqs=4, max_model_len=512,
                         use_graphs=True)
    results = rl.run_steps_in_process(runner, steps)
    rl.check_against_oracle(model_dir, reqs, steps, results, tol(dtype, name), dtype)
    assert runner._graphs, "no decode step ran as a graph"


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_trace_run_program(pupinex_dirs, tmp_path, dtype):
    """The program itself, as a user calls it, on a model of this architecture."""
    model_dir = pupinex_dirs["pxA"]
    reqs = requests_for("pxA", model_dir)
    steps = rl.trace_mixed(reqs, want_all=False)
    out = rl.run_steps_subprocess(model_dir, dtype, steps, str(tmp_path / "out"), rl.max_live_tokens(steps, 64))
    rl.check_against_oracle(model_dir, reqs, steps, out, tol(dtype, "pxA"), dtype)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", ["pxA", "pxC"])
def test_greedy_generation_through_the_engine(pupinex_dirs, name, dtype):
    """The engine's own entry point: scheduler, portions beside decoding requests, graphs, sampler (whose tokens the next
    step reads on the device), a cache too small for all requests at once.  Every kept row of logits matches the
    plain logits of the engine's own sequence (up to the first close call of a router), and every token is the first
    maximum of its row."""
    from tffinfer_amd import EngineOptions, LLMEngine
    from pupinex_models import MIN_MARGIN
    d = pupinex_dirs[name]
    V = read_config(d)["vocab"]
    prompts = [list(clear_tokens(d, n, V, 80 + n)) for n in (1, 9, 40, 60)]
    eng = LLMEngine.from_model_dir(d, EngineOptions(dtype=dtype, page_size=16, kv_tokens=192, max_num_seqs=3,
                                                    max_num_batched_tokens=48, prefill_chunk=24, max_model_len=256))
    eng.keep_logits = True
    res = eng.generate(prompts, max_new_tokens=40, ignore_eos=True)
    cfg, Wt = plain.load(d)
    for r in res:
        assert len(r.output) == 40 and r.finish_reason == "length"
        margins = []
        ref = plain.forward(cfg, Wt, r.prompt + r.output, margins=margins)
        gap = torch.stack(margins, 0).min(0).values if margins else torch.full((len(r.prompt) + 40,), math.inf)
        # a close call turns an expert for that token and, through the cache, may move every later row
        close = (gap < MIN_MARGIN).nonzero()
        upto = int(close[0]) if (close.numel() and dtype == "bfloat16") else len(gap)
        for i, (row, tok) in enumerate(zip(r.logits, r.output)):
            assert tok == int(torch.argmax(row))
            at = len(r.prompt) + i - 1
            if at >= upto:
                break
            err = rel_err(row, ref[at])
            note_error(dtype, d, err)
            assert err <= tol(dtype, d), f"output {i}: {err:.3e}"
    if dtype == "float32":
        toks = list(prompts[1])
        for _ in range(8):
            toks.append(int(torch.argmax(plain.forward(cfg, Wt, toks)[-1])))
        assert res[1].output[:8] == toks[len(prompts[1]):]


def test_the_command_line_with_a_configuration_file_of_this_architecture(tmp_path):
    """--config FILE --random-weights through bin/tffinfer: the weights are those of the folder that
    --save-model writes, the dumped rows are the logits that chose each token."""
    import json
    import os
    import subprocess
    import sys
    import numpy as np
    from pupinex_models import PX_B
    prog = os.path.join(os.path.dirname(os.path.dirname(os.path.abspath(__file__))), "bin", "tffinfer")
    cfg = tmp_path / "config.json"
    cfg.write_text(json.dumps(PX_B))
    folder, dump = str(tmp_path / "pxB"), str(tmp_path / "logits.f32")
    cmd = [sys.executable, prog, "--config", str(cfg), "--random-weights", "--seed", "5", "--fp32", "--n-ctx", "256",
           "--n-predict", "12", "--ignore-eos", "--json", "--random-prompts", "3:30", "--page-size", "8",
           "--max-batches", "3", "--save-model", folder, "--dump-logits", dump, "--kv-tokens", "512"]
    p = subprocess.run(cmd, capture_output=True, text=True, timeout=300)
    assert p.returncode == 0, p.stderr[-3000:]
    recs = [json.loads(ln) for ln in p.stdout.strip().splitlines()]
    meta = json.load(open(dump + ".json"))
    V = PX_B["vocab"]
    rows = np.fromfile(dump, dtype="<f4").reshape(meta["shape"])
    assert meta["shape"] == [36, V]
    for i, r in enumerate(recs):
        ref = oracle_logits(folder, r["prompt"] + r["output"])
        first = meta["requests"][i]["first_row"]
        for j, tok in enumerate(r["output"]):
            row = torch.from_numpy(rows[first + j].copy())
            assert rel_err(row, ref[len(r["prompt"]) - 1 + j]) <= tol("float32", "pxB")
            assert tok == int(torch.argmax(row))
