"""The Gopuzen design in the engine against the plain implementation: each mechanism alone at the
level of its op or part, then whole models through the step function (whole prompts, decoding
token by token, portions down to two tokens, mixed batches on a pool whose pages and slots are
used again), and greedy generation through the engine's own entry point and scheduler."""
import math

import pytest
import torch

import plain_gopuzen as plain
import replay_lib as rl
from gopuzen_models import GOPUZEN_LENGTHS, GOPUZEN_PAGE, clear_tokens
from helpers import note_error, oracle_logits, random_tokens, read_config, rel_err, tol

pytestmark = pytest.mark.gpu
DEV = "cuda:0"
DTYPES = {"float32": torch.float32, "bfloat16": torch.bfloat16}
NAMES = ["gzA", "gzB", "gzC", "gzD"]
BF = torch.bfloat16


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


# ---------------------------------------------------------------- mechanisms, one by one ---

@pytest.mark.parametrize("W", [48, 321, 1030, 2052, 4100, 4099])
def test_norms_before_and_after_a_sublayer(W):
    """resid += scale * layernorm(term) and the layer norm of the sum, the term being a tensor, planes, a tensor with a
    bias, or the half sum of two RMS-normed results; or the norm of chosen rows with the stream left as it is."""
    ops = _ops()
    n, eps, peps = 5, 1e-3, 1e-2
    x, one, two = (_rand(n, W, seed=i, scale=s) for i, s in ((1, 3.0), (2, 0.7), (3, 5.0)))
    one = one + 2.0                 # (a mean far from zero)
    planes, planes2 = _rand(3, n, W, seed=4), _rand(2, n, W, seed=5)
    w, b, nw, nb, sc, wa, wb, bias = (_rand(W, seed=10 + i) for i in range(8))
    d = lambda t: t.to(DEV)                  # noqa: E731
    dd = lambda t: t.double()                # noqa: E731
    norm, pair_w = (d(nw), d(nb), peps), (d(wa), d(wb), peps)
    pair = 0.5 * (plain.unit_rms(dd(one), peps) * dd(wa) + plain.unit_rms(dd(planes2).sum(0), peps) * dd(wb))
    normed = lambda t: plain.layer_norm(t, dd(nw), dd(nb), peps)     # noqa: E731
    O = ops.OutputTerm
    cases = [
        (None, 0 * dd(x)), (d(one), dd(one)), (d(planes), dd(planes).sum(0)),
        (O(d(one), bias=d(bias)), dd(one) + dd(bias)),
        (O(d(planes), bias=d(bias), norm=norm, scale=d(sc)), normed(dd(planes).sum(0) + dd(bias)) * dd(sc)),
        (O(d(one), pair=(d(planes2), *pair_w)), pair),
        (O(d(one), pair=(d(planes2), *pair_w), norm=norm, scale=d(sc)), normed(pair) * dd(sc)),
        (O(d(one), norm=norm), normed(dd(one))),
    ]
    for term, want in cases:
        total = dd(x) + want
        ref = plain.layer_norm(total, dd(w), dd(b), eps)
        resid = d(x.clone())
        out = ops.add_layernorm(resid, term, d(w), d(b), eps, torch.float32)
        assert _err(resid, total) < 2e-6 and _err(out, ref) < 5e-6
        assert _err(ops.add_layernorm(d(x.clone()), term, d(w), d(b), eps, BF).float(), ref) < 5e-3
        if term is not None:
            assert _err(term, want) < 2e-6
            resid = d(x.clone())
            y = ops.add_layernorm(resid, term, d(w), d(b), eps, torch.float32, rows=_i32([4, 0, 2]))
            assert _err(y, ref[[4, 0, 2]]) < 5e-6 and torch.equal(resid.cpu(), x)
    # many rows take another shape of block
    xm, om = _rand(600, W, seed=6), _rand(600, W, seed=7)
    r = d(xm.clone())
    out = ops.add_layernorm(r, O(d(om), norm=norm, scale=d(sc)), d(w), d(b), eps, torch.float32)
    total = dd(xm) + normed(dd(om)) * dd(sc)
    assert _err(r, total) < 2e-6 and _err(out, plain.layer_norm(total, dd(w), dd(b), eps)) < 5e-6


def _steps(cache, plan):
    """Batches of the steps in ``plan``, each a list of (request, tokens); commits after each."""
    from tffinfer_amd.engine.batch import StepEntry, build_step_batch
    for parts in plan:
        for r, n in parts:
            if not cache.has_request(r):
                cache.add_request(r)
            cache.reserve(r, n)
        yield build_step_batch([StepEntry(r, [0] * n, []) for r, n in parts], cache, DEV)
        for r, n in parts:
            cache.commit(r, n)


@pytest.mark.parametrize("W", [36, 35, 1032])
@pytest.mark.parametrize("taps", [1, 2, 3, 4, 5, 9])
def test_convolution_of_a_sublayers_input(taps, W):
    """out = h + conv(h) with h the norm's rows, for requests of unequal length in shared steps: portions down to two
    tokens, single tokens beside them, steps of single tokens only (one kernel), and slots that are used again."""
    from tffinfer_amd.cache import CacheManager
    from tffinfer_amd.parts.base import StateSpec
    ops = _ops()
    eps, off, n_state = 1e-5, 7, 7 + (taps - 1) * W + 3
    w, b = 1 + 0.2 * _rand(W, seed=1), _rand(W, seed=2)
    conv = _rand(W, taps, seed=3, scale=0.6)
    cw = conv.t().contiguous().to(DEV)
    cache = CacheManager([(0, True, None, StateSpec((n_state,)))], 16, 1, 3, device=DEV)
    state = cache.state_tensors[0]
    plan = [[("a", 40), ("b", 2)], [("b", 70), ("a", 1)], [("a", 1), ("b", 1)], [("a", 1), ("b", 1)], [("c", 2), ("a", 1), ("b", 3)],
            [("c", 2)], [("c", 1)], [("c", 33)], [("b", 1), ("c", 1)]]
    for _ in range(2):
        total = {r: sum(n for p in plan for q, n in p if q == r) for r in "abc"}
        xs = {r: _rand(n, W, seed=ord(r), scale=2.0) for r, n in total.items()}
        refs = {r: plain.with_input_conv(plain.layer_norm(x.double(), w.double(), b.double(), eps), conv.double()) for r, x in xs.items()}
        at = dict.fromkeys("abc", 0)
        for parts, batch in zip(plan, _steps(cache, plan)):
            rows = torch.cat([xs[r][at[r]:at[r] + n] for r, n in parts]).to(DEV)
            out = ops.add_layernorm(rows, None, w.to(DEV), b.to(DEV), eps, torch.float32, conv=(cw, state, off), batch=batch)
            ref = torch.cat([refs[r][at[r]:at[r] + n] for r, n in parts])
            assert _err(out, ref) < 5e-6, parts
            for r, n in parts:
                at[r] += n
        for r in "abc":
            cache.release(r)
        assert float(state[:, :off].abs().max()) == 0.0 and float(state[:, off + (taps - 1) * W:].abs().max()) == 0.0
    if taps > 1:        # what went before a portion matters
        lost = plain.with_input_conv(plain.layer_norm(xs["a"].double()[40:], w.double(), b.double(), eps), conv.double())
        assert _err(lost[:1], refs["a"][40:41]) > 1e-2


@pytest.mark.parametrize("M,I,K", [(1, 24, 64), (8, 200, 320), (16, 48, 132), (33, 1000, 256), (150, 136, 72), (300, 512, 1024), (40, 64, 4096)])
def test_biases_in_the_gated_product(M, I, K):
    """silu(x Wg + bg) * (x Wu + bu) whatever kernel the product's sizes select (few rows, tiles, K split over blocks)."""
    ops = _ops()
    x, g, u = (_rand(*s, seed=i).to(BF) for i, s in ((1, (M, K)), (2, (I, K)), (3, (I, K))))
    g, u = (g.float() * K ** -0.5).to(BF), (u.float() * K ** -0.5).to(BF)
    gb, ub = _rand(I, seed=4), _rand(I, seed=5, scale=2.0)
    ref = plain.silu(x.double() @ g.double().T + gb.double()) * (x.double() @ u.double().T + ub.double())
    out = ops.linear_swiglu_bias(x.to(DEV), ops.pack_gate_up(g.to(DEV), u.to(DEV)), ops.pack_gate_up_bias(gb.to(DEV), ub.to(DEV)))
    assert _err(out.float(), ref) < 6e-3
    out = ops.linear_swiglu_bias(x.float().to(DEV), torch.cat([g, u]).float().to(DEV), torch.cat([gb, ub]).to(DEV))
    assert _err(out, ref) < 3e-6
    # a plain product with a bias
    pw = ops.pack_weight(g.to(DEV))
    pad = torch.zeros(-(-I // 16) * 16)
    pad[:I] = gb
    out = ops.linear(x.to(DEV), pw, out_dtype=torch.float32, bias=pad.to(DEV))
    assert _err(out, x.double() @ g.double().T + gb.double()) < 3e-6


@pytest.mark.parametrize("E,I,top", [(8, 4, 3), (2, 2, 4), (5, 1, 1), (40, 8, 6), (1, 1, 2)])
def test_experts_that_hand_their_input_on(E, I, top):
    """A softmax over all experts, a correction that moves the choice only, weights that are not made to add up to
    one, and experts without matrices whose output is their input; by pairs and by tiles."""
    ops = _ops()
    T, W, ff = 40, 48, 24
    x = _rand(T, W, seed=E).to(BF).float()
    P = {"router": _rand(E + I, W, seed=E + 1, scale=0.25).double(), "correction": _rand(E + I, seed=E + 2, scale=0.2).double()}
    for e in range(E):
        for k, (n, shape) in enumerate((("gate", (ff, W)), ("up", (ff, W)), ("down", (W, ff)))):
            P[f"e{e}.{n}"] = _rand(*shape, seed=100 * e + k, scale=0.3).to(BF).double()
    m = {"router": {"top": top, "experts": E, "identity": I}}
    ref = plain.routed_experts(m, P, x.double())
    s, c = plain.router_scores(P, x.double())
    want = torch.topk(c, top).indices
    idx, wts = ops.route_topk(x.to(DEV), P["router"].float().to(DEV), P["correction"].float().to(DEV), top, softmax=True)
    assert torch.equal(idx.cpu().long(), want) and _err(wts, torch.gather(s, 1, want)) < 2e-6
    assert (want >= E).any() and ((want < E).any() or top <= I)
    stack = lambda n: ops.pad_expert_rows(torch.stack([P[f"e{e}.{n}"] for e in range(E)], 0).float()).to(DEV)   # noqa: E731
    args = (stack("gate"), stack("up"), stack("down"))
    run = lambda h, a, **kw: ops.routed_experts(h, *a, idx, wts, float("inf"), 1.0, up_offset=0.0, **kw)        # noqa: E731
    full = run(x.to(DEV), args, identity=I)
    assert _err(full, ref) < 2e-5
    for by_tiles in (False, True):
        out = run(x.to(BF).to(DEV), tuple(a.to(BF) for a in args), identity=I, by_tiles=by_tiles)
        assert _err(out, ref) < 3e-2
    alone = ops.routed_experts(x[7:8].to(DEV), *args, idx[7:8].contiguous(), wts[7:8].contiguous(), float("inf"), 1.0,
                               up_offset=0.0, identity=I)
    assert torch.equal(ops.as_tensor(alone)[0], ops.as_tensor(full)[7])


# ---------------------------------------------------------------- attention ---

def _view(cache, batch, cache_id, writes=True):
    from tffinfer_amd.engine.batch import KVView
    gi = cache.group_index(cache_id)
    k, v = cache.kv_tensors(cache_id)
    gt = batch.groups[gi]
    return KVView(k, v, gt.block_tables, gt.slot_mapping if writes else gt.no_slot_mapping, cache.page_size, gi, gt.key_runs,
                  gt.run_start, gt.runs_window, gt.runs_for_blocks, gt.runs_merge, gt.pool_tables)


def _ctx(batch, act_dtype, max_positions=2048):
    from tffinfer_amd.engine.runner import LayerContext
    return LayerContext(_ops(), act_dtype, batch, max_positions)


def _draw(part, seed, weights=None, scale=0.3):
    g = torch.Generator().manual_seed(seed)
    w = {}
    for k, s in part.weight_specs().items():
        t = torch.randn(s.shape, generator=g)
        w[k] = (1 + 0.2 * t) if s.init == "norm" else ((0.5 * t) if s.init == "norm_offset" else (t * scale).to(BF))
    w.update(weights or {})
    return w


def _attention(W, H, G, D, E, scale, mask, rot, dtype, seed, gate=True, temp=(0.0, 1), shared=False, keeps=None, weights=None):
    """(part, the plain functions' mixer entry, the plain functions' weights)."""
    from tffinfer_amd.config.base import PartSpec
    from tffinfer_amd.parts import GroupedAttention
    pos = PartSpec("rope", {"head_dim": D, "theta": rot[1], "pairing": "interleaved", "rotary_dim": rot[0]}) if rot else None
    size, pool = mask
    keeps = keeps or (size, (pool,) if pool else ())
    att = GroupedAttention(hidden_size=W, num_heads=H, num_kv_heads=G, head_dim=D, value_dim=E, position=pos, scale=scale,
                           window=size, pool=pool, cache_window=keeps[0], cache_pools=keeps[1], shared_cache=shared,
                           head_gate=gate, q_temp_coef=temp[0], q_temp_every=temp[1])
    w = _draw(att, seed, weights)
    att.load_weights(w, dtype, DEV)
    m = {"heads": H, "kv_heads": G, "dim": D, "vdim": E, "scale": scale, "mask": {"size": size, "pool": pool},
         "rot": {"dims": rot[0], "base": rot[1]} if rot else {"dims": 0, "base": 1.0},
         "q_temp": {"coef": temp[0], "every": temp[1]}}
    return att, m, {k: v.double() for k, v in w.items()}


def _run(parts, x, cuts, dtype, page, state=None):
    """The parts (the writer of a cache, then readers of it) over rows x of one request in portions ``cuts``; returns
    each part's outputs [T, W].  The pool of pages holds what the request needs and no more."""
    from tffinfer_amd.cache import CacheManager
    T = x.shape[0]
    kv = parts[0].cache_spec()
    reqs = [(0, not getattr(p, "shared_cache", False), p.cache_spec(), p.state_spec()) for p in parts]
    cache = CacheManager(reqs, page, -(-T // page), 2, dtype=dtype, device=DEV)
    outs, at = [[] for _ in parts], 0
    for n, batch in zip(cuts, _steps(cache, [[("r", n)] for n in cuts])):
        ctx = _ctx(batch, dtype)
        ctx.state = cache.state_tensors.get(0)
        rows = x[at:at + n].to(dtype).to(DEV)
        for i, part in enumerate(parts):
            if kv is not None:
                ctx.kv = _view(cache, batch, 0, writes=not getattr(part, "shared_cache", False))
            outs[i].append(_ops().as_tensor(part.forward(ctx, rows)).float())
        at += n
    assert at == T
    cache.check()
    return [torch.cat(o, 0) for o in outs]


@pytest.mark.parametrize("dtype,limit", [(torch.float32, 3e-5), (torch.bfloat16, 4e-2)])
@pytest.mark.parametrize("H,G,D,E,mask,rot,page", [
    (4, 2, 16, 24, (20, 6), (8, 500.0), 16),      # a part of a head rotated, blocks that are no divisor of a page
    (2, 2, 32, 48, (1, 1), (32, 1e6), 8),         # a window of one token, blocks of one
    (5, 1, 12, 20, (37, 5), (12, 777.0), 32),     # no multiples of 8, five heads on one kv head
    (6, 6, 8, 8, (9, 3), (4, 50.0), 16),          # heads that are not grouped
    (4, 1, 24, 16, (5, 12), (24, 300.0), 8),      # blocks longer than the window
    (8, 2, 128, 128, (64, 16), (64, 1e4), 16),    # the sizes of real models
    (16, 1, 64, 64, (33, 4), (64, 1e4), 16),
    (2, 1, 192, 64, (40, 8), (32, 1e4), 16),
    (2, 1, 64, 256, (40, 8), (64, 1e4), 16),
    (1, 1, 16, 288, (30, 10), (16, 100.0), 16),   # values beyond the matrix-core attention's sizes
    (4, 2, 16, 16, (25, 0), (16, 100.0), 8),      # a window without blocks
    (4, 2, 16, 24, (0, 0), (16, 100.0), 8)])      # every key
def test_attention_over_a_window_and_the_blocks_before_it(H, G, D, E, mask, rot, page, dtype, limit):
    """A prompt in one step, as portions down to two tokens, and as a portion followed by single tokens."""
    W, T = 48, 230
    att, m, P = _attention(W, H, G, D, E, 0.4 * D ** -0.5, mask, rot, dtype, H * D + E)
    x = _rand(T, W, seed=7).to(BF).float()
    ref = plain.window_attention(m, P, x.double(), plain.attention_cache(m, P, x.double()))
    for cuts in _cuts(T):
        err = _err(_run([att], x, cuts, dtype, page)[0], ref)
        assert err < limit, f"cut {cuts[:3]}: {err:.3e}"


@pytest.mark.parametrize("dtype,limit", [(torch.float32, 3e-5), (torch.bfloat16, 4e-2)])
@pytest.mark.parametrize("D,E,page", [(16, 24, 8), (64, 64, 16), (20, 12, 16)])
def test_readers_of_a_borrowed_cache_with_windows_of_their_own(D, E, page, dtype, limit):
    """Two readers whose windows and blocks are not the owner's: the cache keeps what any of them sees."""
    W, T, G = 48, 170, 2
    masks = [(20, 6), (33, 4), (5, 12)]
    keeps = (33, (4, 6, 12))
    parts, plains = [], []
    for i, (mask, H) in enumerate(zip(masks, (4, 2, 6))):
        att, m, P = _attention(W, H, G, D, E, 0.2, mask, (D - D % 4, 100.0), dtype, 20 + i, shared=i > 0, keeps=keeps)
        assert ("k" in att.weight_specs()) == (i == 0)
        parts.append(att)
        plains.append((m, P))
    assert len({p.cache_spec() for p in parts}) == 1
    x = _rand(T, W, seed=5).to(BF).float()
    cache = plain.attention_cache(*plains[0], x.double())
    refs = [plain.window_attention(m, P, x.double(), cache) for m, P in plains]
    for cuts in _cuts(T):
        for i, (out, ref) in enumerate(zip(_run(parts, x, cuts, dtype, page), refs)):
            assert _err(out, ref) < limit, (i, cuts[:3])


def _loud(T, i, loud, decode_tail, mask, dtype, page=16, P_weights=None):
    """An attention of one head without rotation on rows in which token ``loud``'s key stands out for query i only;
    returns (engine's row i, plain row i, plain row i without the loud key)."""
    W = D = 8
    eye, pick = torch.eye(D), torch.eye(D)
    pick[3], pick[4] = eye[4], 0            # (a query lies along the keys' axis 3 if its row does along axis 4)
    fixed = {"q": pick.to(BF), "k": eye.to(BF), "v": _rand(12, W, seed=3).to(BF), "g": torch.zeros(1, W).to(BF),
             "o": _rand(W, 12, seed=4).to(BF)}
    att, m, P = _attention(W, 1, 1, D, 12, 6.0, mask, None, dtype, 1, weights=fixed)
    x = _rand(T, W, seed=9, scale=0.05).to(BF).float()
    x[:, 3:5] = 0
    x[loud] = 0
    x[loud, 3], x[loud, 5], x[loud, 6] = 4.0, -4.0, 4.0
    x[i, 4] = 4.0
    without = x.clone()
    without[loud] = 0
    both = [plain.window_attention(m, P, y.double(), plain.attention_cache(m, P, y.double()))[i] for y in (x, without)]
    cuts = [i] + [1] * (T - i) if decode_tail else [T]
    return _run([att], x, cuts, dtype, page)[0][i], both[0], both[1]


@pytest.mark.parametrize("decode", [False, True])
@pytest.mark.parametrize("mask", [(24, 8), (40, 6), (7, 16)])
def test_a_loud_key_at_the_edges_of_window_and_blocks(mask, decode):
    """One key whose score with the last query stands far out: the window's first key, the key before it (its block
    not seen yet or just seen), the tokens of the last block that is seen, the block after it, the first tokens
    of the sequence.  Where the key is seen its loss moves the plain result; where it is not, the result is the one
    without it."""
    size, pool = mask
    for i in (150, 151, 155, 158):
        lo = i - size + 1
        nb = lo // pool                                # blocks that are seen
        spots = {i: True, lo: True, lo - 1: nb * pool > lo - 1, nb * pool - 1: True, (nb - 1) * pool: True, nb * pool: nb * pool >= lo,
                 0: True, 1: True, pool - 1: True, pool: True}
        for j, seen in spots.items():
            if j == i:
                continue
            out, ref, lost = _loud(160, i, j, decode, mask, torch.float32)
            assert _err(out, ref) < 3e-5, (i, j)
            moved = float((ref - lost).abs().max() / ref.abs().max())
            assert (moved > 0.02) if seen else (moved < 1e-9), (i, j, moved)


def test_a_loud_key_is_seen_through_its_block_in_bfloat16():
    for j in (3, 40, 101):
        out, ref, lost = _loud(160, 158, j, True, (24, 8), torch.bfloat16)
        assert _err(out, ref) < 3e-2 and float((ref - lost).abs().max() / ref.abs().max()) > 0.06


@pytest.mark.parametrize("dtype,limit", [(torch.float32, 3e-5), (torch.bfloat16, 3e-2)])
@pytest.mark.parametrize("H,G,D,E,temp,page", [(4, 2, 16, 8, (0.5, 7), 16), (1, 1, 32, 16, (0.3, 1), 8), (3, 1, 20, 12, (0.7, 10), 16),
                                              (8, 2, 64, 128, (0.5, 64), 16), (2, 2, 96, 192, (1.5, 40), 16)])
def test_attention_whose_queries_grow_with_the_position(H, G, D, E, temp, page, dtype, limit):
    W, T = 48, 200
    att, m, P = _attention(W, H, G, D, E, 0.3 * D ** -0.5, (0, 0), None, dtype, H * D, gate=False, temp=temp)
    x = _rand(T, W, seed=8).to(BF).float()
    ref = plain.tempered_attention(m, P, x.double())
    for cuts in _cuts(T):
        assert _err(_run([att], x, cuts, dtype, page)[0], ref) < limit, cuts[:3]
    off = dict(m, q_temp={"coef": temp[0], "every": temp[1] + 1})
    assert _err(plain.tempered_attention(off, P, x.double()), ref) > 1e-3


# ---------------------------------------------------------------- the recurrence ---

def _lightning(W, D, E, decay, eps, dtype, seed, weights=None):
    from tffinfer_amd.parts import LightningMixer
    part = LightningMixer(hidden_size=W, num_heads=len(decay), head_dim=D, value_dim=E, decay=decay, norm_eps=eps)
    w = _draw(part, seed, weights)
    part.load_weights(w, dtype, DEV)
    return part, {"heads": len(decay), "dim": D, "vdim": E, "decay": list(decay)}, {k: v.double() for k, v in w.items()}


@pytest.mark.parametrize("dtype,limit", [(torch.float32, 3e-5), (torch.bfloat16, 4e-2)])
@pytest.mark.parametrize("D,E,decay", [(8, 12, (0.6, 0.9, 0.99)), (24, 8, (0.97,)), (10, 14, (0.8, 0.3, 0.998)), (64, 64, (0.999, 0.5)),
                                       (128, 32, (0.98, 0.9999)), (32, 128, (0.95,)), (160, 48, (0.99,)), (256, 16, (1.0, 0.0))])
def test_recurrence_with_a_decay_per_head(D, E, decay, dtype, limit):
    W, T, eps = 48, 230, 1e-5
    part, m, P = _lightning(W, D, E, decay, eps, dtype, D + E)
    x = _rand(T, W, seed=6).to(BF).float()
    ref = plain.lightning(m, P, x.double(), eps)
    for cuts in _cuts(T) + [[64, 65, 63, 38], [128, 102]]:
        err = _err(_run([part], x, cuts, dtype, 16)[0], ref)
        assert err < limit, f"cut {cuts[:3]}: {err:.3e}"


def test_a_loud_token_far_back_in_the_recurrence():
    """What a token far back wrote into the state is read by the last token, in a prompt and decoded, and a state lost
    at a portion's border would show."""
    W, D, E, T, eps = 16, 8, 8, 400, 1e-5
    part, m, P = _lightning(W, D, E, (0.999, 0.99), eps, torch.float32, 3)
    x = _rand(T, W, seed=4, scale=0.1).to(BF).float()
    x[30] *= 60.0
    ref = plain.lightning(m, P, x.double(), eps)
    calm = x.clone()
    calm[30] *= 0
    assert _err(plain.lightning(m, P, calm.double(), eps)[-1], ref[-1]) > 0.1
    for cuts in ([T], [31] + [1] * (T - 31), [100, 2, 200, 98]):
        assert _err(_run([part], x, cuts, torch.float32, 16)[0], ref) < 5e-5, cuts[:3]


def test_two_mixers_side_by_side_and_batches_of_unequal_requests():
    """The pair of a tempered attention and a recurrence, each output normed, half their sum: three requests of unequal
    length in shared steps give what each gives alone; pages and slots are freed and used again."""
    from tffinfer_amd.cache import CacheManager
    from tffinfer_amd.config.base import PartSpec
    from tffinfer_amd.parts import NormedPair
    W, eps, page = 40, 1e-5, 8
    H, G, D, E, temp, decay, rd, re = 4, 2, 16, 24, (0.5, 5), (0.9, 0.99, 0.5), 12, 20
    mixer = NormedPair(W, PartSpec("grouped_attention", {"hidden_size": W, "num_heads": H, "num_kv_heads": G, "head_dim": D,
                                                         "value_dim": E, "scale": 0.2, "q_temp_coef": temp[0], "q_temp_every": temp[1]}),
                       PartSpec("lightning", {"hidden_size": W, "num_heads": 3, "head_dim": rd, "value_dim": re, "decay": decay,
                                              "norm_eps": eps}), norm_eps=eps)
    w = _draw(mixer, 17)
    mixer.load_weights(w, torch.float32, DEV)
    m = {"left": {"heads": H, "kv_heads": G, "dim": D, "vdim": E, "scale": 0.2, "q_temp": {"coef": temp[0], "every": temp[1]}},
         "right": {"heads": 3, "dim": rd, "vdim": re, "decay": list(decay)}}
    P = {k: v.double() for k, v in w.items()}
    lengths = {"a": 60, "b": 41, "c": 7}
    xs = {r: _rand(n, W, seed=n).to(BF).float() for r, n in lengths.items()}
    refs = {r: plain.parallel(m, P, x.double(), eps) for r, x in xs.items()}
    cache = CacheManager([(0, True, mixer.cache_spec(), mixer.state_spec())], page, 15, 3, dtype=torch.float32, device=DEV)
    for plan in ([[("a", 35), ("b", 40)], [("a", 25), ("b", 1), ("c", 7)]],
                 [[("b", 2), ("a", 30)], [("c", 1), ("b", 20)], [("c", 1), ("a", 1), ("b", 1)], [("a", 29), ("b", 18), ("c", 5)]]):
        at = dict.fromkeys("abc", 0)
        for parts, batch in zip(plan, _steps(cache, plan)):
            ctx = _ctx(batch, torch.float32)
            ctx.kv, ctx.state = _view(cache, batch, 0), cache.state_tensors[0]
            rows = torch.cat([xs[r][at[r]:at[r] + n] for r, n in parts]).to(DEV)
            out = mixer.forward(ctx, rows)
            assert _err(out, torch.cat([refs[r][at[r]:at[r] + n] for r, n in parts])) < 3e-5, parts
            for r, n in parts:
                at[r] += n
        for r in "abc":
            cache.release(r)
        cache.check()


def test_batches_of_unequal_requests_share_a_window_with_blocks():
    """Requests of unequal length in one step, single tokens beside portions, through an owner of a cache and a reader;
    the pool holds the window's pages and the blocks' and no more."""
    from tffinfer_amd.cache import CacheManager
    W, page = 40, 8
    masks, keeps = [(10, 4), (17, 3)], (17, (3, 4))
    own, reader = (_attention(W, 4, 2, 16, 24, 0.3, mk, (8, 100.0), torch.float32, 31 + i, shared=i > 0, keeps=keeps)
                   for i, mk in enumerate(masks))
    lengths = {"a": 90, "b": 61, "c": 9}
    xs = {r: _rand(n, W, seed=n).to(BF).float() for r, n in lengths.items()}
    refs = {}
    for r, x in xs.items():
        c = plain.attention_cache(own[1], own[2], x.double())
        refs[r] = [plain.window_attention(m, P, x.double(), c) for _, m, P in (own, reader)]
    spec = own[0].cache_spec()
    cache = CacheManager([(0, True, spec, None), (0, False, reader[0].cache_spec(), None)], page, {spec: 32}, 3,
                         dtype=torch.float32, device=DEV)
    for plan in ([[("a", 35), ("b", 40)], [("a", 1), ("b", 1), ("c", 7)], [("a", 54), ("c", 2)], [("b", 20)]],
                 [[("b", 2), ("a", 30)], [("c", 1), ("b", 20)], [("c", 1), ("a", 1), ("b", 1)], [("a", 40), ("b", 37), ("c", 7)]]):
        at = dict.fromkeys("abc", 0)
        for parts, batch in zip(plan, _steps(cache, plan)):
            ctx = _ctx(batch, torch.float32)
            rows = torch.cat([xs[r][at[r]:at[r] + n] for r, n in parts]).to(DEV)
            for i, (part, _, _) in enumerate((own, reader)):
                ctx.kv = _view(cache, batch, 0, writes=i == 0)
                out = _ops().as_tensor(part.forward(ctx, rows))
                assert _err(out, torch.cat([refs[r][i][at[r]:at[r] + n] for r, n in parts])) < 3e-5, (i, parts)
            for r, n in parts:
                at[r] += n
        cache.check()
        for r in "abc":
            cache.release(r)
    assert cache.groups[0].pool.num_used == 0


@pytest.mark.parametrize("dtype,limit", [(torch.float32, 3e-5), (torch.bfloat16, 3e-2)])
def test_long_contexts_decode_beside_a_portion(dtype, limit):
    """Requests of 300 to 900 tokens that decode beside another's portion get the kernel that splits keys among waves,
    those of the blocks before the window among them."""
    from tffinfer_amd.cache import CacheManager
    W, page = 40, 16
    att, m, P = _attention(W, 8, 2, 64, 64, 0.04, (70, 4), (64, 1000.0), dtype, 41)
    lengths = {"a": 901, "b": 302, "c": 90}
    xs = {r: _rand(n, W, seed=n).to(BF).float() for r, n in lengths.items()}
    refs = {r: plain.window_attention(m, P, x.double(), plain.attention_cache(m, P, x.double())) for r, x in xs.items()}
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
    # the blocks matter: without them the last rows are others
    bare = dict(m, mask={"size": 70, "pool": 0})
    lost = plain.window_attention(bare, P, xs["a"].double(), plain.attention_cache(bare, P, xs["a"].double()))
    assert _err(lost[-1], refs["a"][-1]) > 0.1


# ---------------------------------------------------------------------- whole models ---

def requests_for(name, model_dir):
    V = read_config(model_dir)["vocab"]
    # (sequences in which no choice of experts is a close call that rounding could turn)
    return {f"{name}{i}": list(clear_tokens(model_dir, n, V, 3000 + 13 * i + n)) for i, n in enumerate(GOPUZEN_LENGTHS[name])}


def make_runner(model_dir, dtype, page_size, num_pages, max_seqs=4, use_graphs=False):
    from tffinfer_amd.engine.runner import ModelRunner
    from tffinfer_amd.models import load_model
    model = load_model(model_dir, DTYPES[dtype], DEV)
    return ModelRunner(model, page_size=page_size, num_pages=num_pages, max_seqs=max_seqs, max_model_len=512,
                       use_graphs=use_graphs)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", NAMES)
def test_residual_stream_after_every_layer(gopuzen_dirs, name, dtype):
    """Layer by layer, so that a fault names its layer.  A block leaves its last sublayer's output to the norm
    after it; the stream after a layer is the stream plus what is pending."""
    from tffinfer_amd.engine.batch import StepEntry, build_step_batch
    from tffinfer_amd.engine.runner import StepContext
    d = gopuzen_dirs[name]
    toks = list(clear_tokens(d, 70, read_config(d)["vocab"], 77))
    want = []
    plain.forward(*plain.load(d), toks, want)
    runner = make_runner(d, dtype, GOPUZEN_PAGE[name], 16)
    model, ops = runner.model, runner.ops
    runner.add_request("a")
    e = [StepEntry("a", toks, [])]
    runner.reserve(e)
    batch = build_step_batch(e, runner.cache, runner.device, runner._pinned)
    ctx = StepContext(ops, runner.act_dtype, batch, runner.max_model_len, runner._calls, runner.cache)
    resid, pending = model.embedding.forward(ctx, batch.token_ids), None
    assert len(model.schedule) == len(want)
    for it, call in enumerate(model.schedule):
        pending = model.blocks[call.layer].forward(ctx.for_call(it), resid, pending)
        after = resid + ops.as_tensor(pending) if pending is not None else resid
        err = _err(after, want[it])
        assert err < (4e-5 if dtype == "float32" else 5e-2), f"layer {it}: {err:.3e}"


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", NAMES)
@pytest.mark.parametrize("mode", ["whole", "tail", "chunks", "mixed"])
def test_replay_modes(gopuzen_dirs, name, dtype, mode):
    model_dir = gopuzen_dirs[name]
    reqs = requests_for(name, model_dir)
    steps = {"whole": rl.trace_whole, "tail": rl.trace_tail, "chunks": rl.trace_chunks,
             "mixed": rl.trace_mixed}[mode](reqs)
    ps = GOPUZEN_PAGE[name]
    # the pool holds what is live at the worst moment and no more, so pages and slots are used again
    num_pages = rl.max_live_tokens(steps, unit=ps) // ps
    runner = make_runner(model_dir, dtype, ps, num_pages)
    results = rl.run_steps_in_process(runner, steps)
    worst = rl.check_against_oracle(model_dir, reqs, steps, results, tol(dtype, name), dtype)
    print(f"{name} {dtype} {mode}: worst rel. error {worst:.3e} over {len(steps)} steps, {num_pages} pages")
    assert all(g.pool.num_used == 0 for g in runner.cache.groups)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", ["gzA", "gzD"])
def test_long_decoding_through_captured_graphs(gopuzen_dirs, name, dtype):
    """Three requests decode some 150 tokens each as replays of captured HIP graphs beside eager prompt steps."""
    model_dir = gopuzen_dirs[name]
    V = read_config(model_dir)["vocab"]
    reqs = {f"g{i}": list(clear_tokens(model_dir, n, V, 300 + n)) for i, n in enumerate((160, 171, 190))}
    steps = rl.trace_mixed(reqs, max_live=3, prompt_frac=0.1, want_all=True)
    ps = GOPUZEN_PAGE[name]
    runner = make_runner(model_dir, dtype, ps, rl.max_live_tokens(steps, unit=ps) // ps, use_graphs=True)
    results = rl.run_steps_in_process(runner, steps)
    rl.check_against_oracle(model_dir, reqs, steps, results, tol(dtype, name), dtype)
    assert runner._graphs, "no decode step ran as a graph"


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_trace_run_program(gopuzen_dirs, tmp_path, dtype):
    """The program itself, as a user calls it, on a model of this architecture."""
    model_dir = gopuzen_dirs["gzA"]
    reqs = requests_for("gzA", model_dir)
    steps = rl.trace_mixed(reqs, want_all=False)
    out = rl.run_steps_subprocess(model_dir, dtype, steps, str(tmp_path / "out"), rl.max_live_tokens(steps, 64))
    rl.check_against_oracle(model_dir, reqs, steps, out, tol(dtype, "gzA"), dtype)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", ["gzA", "gzC"])
def test_greedy_generation_through_the_engine(gopuzen_dirs, name, dtype):
    """The engine's own entry point: scheduler, portions beside decoding requests, graphs, sampler, a cache too small
    for all requests at once.  Every kept row of logits matches the plain logits of the engine's own sequence (up to
    the first close call of a router), and every token is the first maximum of its row."""
    from tffinfer_amd import EngineOptions, LLMEngine
    from gopuzen_models import MIN_MARGIN
    d = gopuzen_dirs[name]
    V = read_config(d)["vocab"]
    prompts = [list(clear_tokens(d, n, V, 80 + n)) for n in (1, 9, 40, 70)]
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
    from gopuzen_models import GZ_B
    prog = os.path.join(os.path.dirname(os.path.dirname(os.path.abspath(__file__))), "bin", "tffinfer")
    cfg = tmp_path / "config.json"
    cfg.write_text(json.dumps(GZ_B))
    folder, dump = str(tmp_path / "gzB"), str(tmp_path / "logits.f32")
    cmd = [sys.executable, prog, "--config", str(cfg), "--random-weights", "--seed", "5", "--fp32", "--n-ctx", "256",
           "--n-predict", "12", "--ignore-eos", "--json", "--random-prompts", "3:30", "--page-size", "8",
           "--max-batches", "3", "--save-model", folder, "--dump-logits", dump, "--kv-tokens", "512"]
    p = subprocess.run(cmd, capture_output=True, text=True, timeout=300)
    assert p.returncode == 0, p.stderr[-3000:]
    recs = [json.loads(ln) for ln in p.stdout.strip().splitlines()]
    meta = json.load(open(dump + ".json"))
    V = GZ_B["vocab"]
    rows = np.fromfile(dump, dtype="<f4").reshape(meta["shape"])
    assert meta["shape"] == [36, V]
    for i, r in enumerate(recs):
        ref = oracle_logits(folder, r["prompt"] + r["output"])
        first = meta["requests"][i]["first_row"]
        for j, tok in enumerate(r["output"]):
            row = torch.from_numpy(rows[first + j].copy())
            assert rel_err(row, ref[len(r["prompt"]) - 1 + j]) <= tol("float32", "gzB")
            assert tok == int(torch.argmax(row))
