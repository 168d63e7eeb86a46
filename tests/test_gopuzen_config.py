"""The Gopuzen configuration: what its config.json turns into, what is refused, which layer calls share a cache and
a state, the books of a cache that keeps keys of blocks, and properties of the plain implementation (all on the CPU)."""
import copy
import json
import random

import pytest
import torch

import plain_gopuzen as plain
from gopuzen_models import GOPUZEN_CONFIGS, GZ_A, GZ_B, GZ_C, GZ_D, clear_tokens, make_gopuzen_dir
from helpers import rel_err
from tffinfer_amd.cache import CacheManager
from tffinfer_amd.cache.sizing import plan_pages, request_pages, state_bytes
from tffinfer_amd.config.base import ConfigError, LayerCall
from tffinfer_amd.models import build_model_skeleton, config_from_dict, load_config
from tffinfer_amd.parts import (GroupedAttention, KVCacheSpec, LayerNorm, LightningMixer, NoFeedForward, NormedPair, RoutedExperts,
                                SandwichBlock, StateSpec, SwiGLU)
from tffinfer_amd.weights.loader import WeightError, check_weights
from tffinfer_amd.weights.safetensors_io import load_model_dir


def _model(cfg):
    return build_model_skeleton(config_from_dict(copy.deepcopy(cfg)))


def test_every_size_and_constant_comes_from_the_file():
    model = _model(GZ_A)
    assert [type(b) for b in model.blocks] == [SandwichBlock] * 5
    assert [type(b.mixer) for b in model.blocks] == [GroupedAttention, NormedPair, GroupedAttention, NormedPair, GroupedAttention]
    assert [type(b.feed_forward) for b in model.blocks] == [SwiGLU, RoutedExperts, RoutedExperts, NoFeedForward, SwiGLU]
    a = model.blocks[0].mixer
    assert (a.num_heads, a.num_kv_heads, a.head_dim, a.value_dim, a.scale, a.window, a.pool) == (4, 2, 16, 24, 0.08, 20, 6)
    assert (a.has_gate, a.shared_cache, a.q_temp_coef) == (True, False, 0.0)
    assert (a.position.rotary_dim, a.position.theta, a.position.pairing) == (8, 500.0, "interleaved")
    # the cache keeps what any of its readers sees
    spec = KVCacheSpec(2, 32, 33, pools=(4, 6, 12))
    assert [model.blocks[i].mixer.cache_spec() for i in (0, 2, 4)] == [spec] * 3 and spec.reach == 33
    r = model.blocks[4].mixer
    assert r.shared_cache and (r.window, r.pool) == (5, 12)
    p = model.blocks[1].mixer
    assert (p.left.head_dim, p.left.value_dim, p.left.q_temp_coef, p.left.q_temp_every, p.left.position, p.left.has_gate) == \
        (16, 8, 0.5, 7, None, False)
    assert (p.left.window, p.left.pool, p.norm_eps, p.left.cache_spec()) == (0, 0, 1e-6, KVCacheSpec(2, 16))
    assert isinstance(p.right, LightningMixer) and (p.right.head_dim, p.right.value_dim, p.right.decay_list) == (8, 12, (0.6, 0.9, 0.99))
    e = model.blocks[1].feed_forward
    assert (e.num_experts, e.identity, e.top, e.intermediate_size, e.router_softmax, e.has_correction, e.weight_input) == \
        (5, 3, 2, 24, True, True, False)
    assert e.limit == float("inf") and (e.act_alpha, e.up_offset) == (1.0, 0.0)
    ff = model.blocks[0].feed_forward
    assert ff.has_bias and ff.intermediate_size == 72
    b = model.blocks[0]
    assert b.conv_taps == 4 and b.layer_scale and isinstance(model.final_norm, LayerNorm) and model.final_norm.eps == 1e-6
    assert model.embedding.scale == 8.0 and model.head.tied_to is None and model.graph_safe()
    d = _model(GZ_D)
    assert d.blocks[0].state_spec() is None and d.blocks[0].mixer.cache_spec() == KVCacheSpec(2, 128, 65, pools=(8, 16))
    m = copy.deepcopy(GZ_B)
    del m["layers"][2]["mixer"]["kv_heads"], m["layers"][2]["mixer"]["vdim"], m["layers"][0]["mlp"]["router"]["identity"]
    c = _model(m)
    assert (c.blocks[2].mixer.num_kv_heads, c.blocks[2].mixer.value_dim, c.blocks[0].feed_forward.identity) == (6, 8, 0)


def test_which_layer_calls_share_a_cache_and_which_a_state():
    """A layer with kv_from works on the cache of the layer it names and writes nothing there; the last inputs of its
    convolutions are its own."""
    assert config_from_dict(copy.deepcopy(GZ_A)).layer_schedule() == [
        LayerCall(0, 0), LayerCall(1, 1), LayerCall(2, 0, False, state=2), LayerCall(3, 3), LayerCall(4, 0, False, state=4)]
    model = _model(GZ_A)
    needs = model.call_requirements()
    conv = 3 * 64
    assert [n[3] for n in needs] == [StateSpec((2 * conv,)), StateSpec((3 * 8 * 12 + 2 * conv,)), StateSpec((2 * conv,)),
                                     StateSpec((2 * 16 * 16 + conv,)), StateSpec((2 * conv,))]
    assert [n[4:] for n in needs] == [(), (), (2,), (), (4,)]
    assert [b.state_offset for b in model.blocks] == [0, 288, 0, 512, 0]
    cache = CacheManager(needs, page_size=16, num_pages=8, max_seqs=2)
    assert sorted(cid for g in cache.groups for cid in g.cache_ids) == [0, 1, 3]
    assert sorted(cache._state_specs) == [0, 1, 2, 3, 4]
    assert state_bytes(needs, 2) == 3 * 4 * (3 * 2 * conv + 288 + 2 * conv + 512 + conv)


def test_books_of_a_cache_that_keeps_keys_of_blocks():
    """Pages of the window go back once it has passed and its block is whole; the blocks' pages stay to the end."""
    spec = KVCacheSpec(2, 16, 10, pools=(4, 24))
    ps = 8
    c = CacheManager([(0, True, spec, None)], ps, 40, 2)
    assert c.groups[0].pool.num_pages == 40 + (80 // 8 + 2) + (-(-13 // 8) + 2)
    c.add_request("r")
    n = 0
    for k in [1] * 30 + [50, 7, 2, 61] + [1] * 40:
        assert c.can_reserve("r", k)
        c.reserve("r", k)
        n += k
        c.commit("r", k)
        c.check()
        assert [len(t) for t in c.groups[0].pool_tables["r"]] == [-(-(n // 4) // ps), -(-(n // 24) // ps)]
        first = next((b for b, p in enumerate(c.groups[0].tables["r"]) if p >= 0), -(-n // ps))
        # every token that is still to be seen, or still to go into a block, is there
        assert first * ps <= max(0, min(n - 10 + 1, n // 4 * 4, n // 24 * 24))
        held = sum(p >= 0 for p in c.groups[0].tables["r"])
        assert held <= -(-24 // ps) + 2
    assert request_pages(spec, n, ps) >= c.groups[0].pool.num_used - 2
    c.reserve("r", 100)
    assert c.rollback("r", keep_new=3) > 0
    c.check()
    c.release("r")
    assert c.groups[0].pool.num_used == 0


@pytest.mark.parametrize("seed", range(4))
def test_random_orders_keep_the_books(seed):
    rng = random.Random(seed)
    spec, full = KVCacheSpec(1, 8, 9, pools=(2, 5, 16)), KVCacheSpec(1, 8)
    c = CacheManager([(0, True, spec, None), (1, True, full, None)], 8, {spec: 22, full: 26}, 4)
    live, nxt = {}, 0
    for _ in range(500):
        op = rng.random()
        free = [g.pool.num_free for g in c.groups]
        if op < 0.2 and len(live) < 4:
            n = c.fit(None, rng.randint(1, 40), free)
            if n:
                c.add_request(nxt)
                c.reserve(nxt, n)
                c.commit(nxt, n)
                live[nxt] = n
                nxt += 1
        elif op < 0.85 and live:
            r = rng.choice(list(live))
            want = rng.randint(1, 30)
            n = c.fit(r, want, free)
            assert c.can_reserve(r, n) and (n == want or not c.can_reserve(r, n + 1))
            c.reserve(r, n)
            if n and rng.random() < 0.3:
                n = rng.randint(0, n)
                c.rollback(r, keep_new=n)
            c.commit(r, n)
        elif live:
            r = rng.choice(list(live))
            c.release(r)
            del live[r]
        c.check()
    for r in live:
        c.release(r)
    assert all(g.pool.num_used == 0 for g in c.groups)


def test_pages_are_planned_for_windows_and_their_blocks():
    spec, full = KVCacheSpec(2, 16, 32, pools=(8,)), KVCacheSpec(4, 16)
    reqs = [(0, True, spec, None), (1, True, full, None)]
    ps, seqs, budget = 16, 4, 64
    pages = plan_pages(reqs, ps, 2, seqs, budget, tokens=40000)
    assert pages[full] == 2500 + seqs and 40000 // 8 // ps + seqs < pages[spec] < 400
    size = lambda p: sum(2 * s.num_kv_heads * s.head_dim * ps * 2 * n for s, n in p.items())      # noqa: E731
    half = plan_pages(reqs, ps, 2, seqs, budget, kv_bytes=size(pages) // 2)
    assert size(half) <= size(pages) // 2 and size(half) > size(pages) * 0.49
    with pytest.raises(ValueError, match="holds no page"):
        plan_pages(reqs, ps, 2, seqs, budget, kv_bytes=100)


def test_tensor_names_follow_the_files():
    names = _model(GZ_A).expected_tensors()
    for n in ("embed", "final.norm", "final.norm.b", "head", "l0.norm1", "l0.norm1.b", "l0.norm1b", "l0.norm1b.b", "l0.norm2", "l0.norm2.b",
              "l0.norm2b", "l0.norm2b.b", "l0.ls1", "l0.ls2", "l0.canon1", "l0.canon2", "l0.mix.q", "l0.mix.k", "l0.mix.v", "l0.mix.g",
              "l0.mix.o", "l0.mlp.gate", "l0.mlp.gate.b", "l0.mlp.up.b", "l0.mlp.down.b", "l1.mix.left.q", "l1.mix.left.o",
              "l1.mix.left.out", "l1.mix.right.q", "l1.mix.right.g", "l1.mix.right.norm", "l1.mix.right.o", "l1.mix.right.out",
              "l1.mlp.router", "l1.mlp.correction", "l1.mlp.e4.down", "l2.mix.q", "l2.mix.g", "l2.mix.o", "l3.ls1"):
        assert n in names, n
    assert not any(n in names for n in ("l2.mix.k", "l2.mix.v", "l1.mlp.e5.gate", "l1.mix.left.g", "l3.mlp.gate", "l1.mlp.gate.b"))
    assert all(names[n].optional for n in ("l3.norm2", "l3.norm2.b", "l3.norm2b", "l3.ls2", "l3.canon2")) and not names["l3.norm1b"].optional
    assert names["l0.mix.q"].shape == (64, 64) and names["l0.mix.v"].shape == (48, 64) and names["l0.mix.g"].shape == (4, 64)
    assert names["l1.mlp.router"].shape == (8, 64) and names["l1.mlp.correction"].shape == (8,) and names["l0.canon1"].shape == (64, 4)
    assert names["l1.mix.right.norm"].shape == (36,) and names["l1.mix.left.out"].shape == (64,)


def test_round_trip_and_refusals(tmp_path):
    d = make_gopuzen_dir(str(tmp_path / "m"), GZ_A, 1, sharp=False)
    cfg = load_config(d)
    back = cfg.to_dict()
    assert back["layers"] == GZ_A["layers"] and back["canon"] == {"taps": 4} and back["embedding"] == {"scale": 8.0}
    assert config_from_dict(json.loads(json.dumps(back))).layer_schedule() == cfg.layer_schedule()
    found, names = load_model_dir(d), build_model_skeleton(cfg).expected_tensors()
    check_weights(names, found, set(), d)
    assert "l3.norm2" not in found
    del found["l0.mlp.up.b"]
    with pytest.raises(WeightError) as e:
        check_weights(names, found, set(), d)
    assert e.value.missing == ["l0.mlp.up.b"]
    for breaker, text in (
            (lambda c: c["layers"][0].update(type="other"), "mixer"),
            (lambda c: c["layers"][1]["mlp"].update(kind="sparse"), "feed-forward"),
            (lambda c: c["layers"][0]["mixer"].update(kv_from=2), "kv_from"),
            (lambda c: c["layers"][2]["mixer"].update(kv_from=1), "kv_from"),
            (lambda c: c["layers"][2]["mixer"].update(kv_from=4), "kv_from"),
            (lambda c: c["layers"][1]["mixer"].update(kv_from=0), "only an attention"),
            (lambda c: c["layers"][2]["mixer"].update(dim=32), "must be equal"),
            (lambda c: c["layers"][2]["mixer"]["rot"].update(base=3.0), "must be equal"),
            (lambda c: c["layers"][0]["mixer"]["mask"].update(size=0), "mask"),
            (lambda c: c["layers"][0]["mixer"]["rot"].update(dims=7), "even"),
            (lambda c: c["layers"][1]["mixer"]["right"].update(decay=[0.5]), "decay"),
            (lambda c: c["layers"][1]["mixer"]["left"]["q_temp"].update(every=0), "every"),
            (lambda c: c["layers"][1]["mixer"].pop("left"), "left"),
            (lambda c: c["layers"][1]["mlp"]["router"].update(top=9), "top"),
            (lambda c: c["canon"].update(taps=0), "conv_taps"),
            (lambda c: c.pop("norm"), "norm"),
            (lambda c: c["norm"].update(eps=0), "eps")):
        bad = copy.deepcopy(GZ_A)
        breaker(bad)
        with pytest.raises(ConfigError, match=text):
            _model(bad)


def test_the_plain_functions_on_cases_done_by_hand():
    t, b = plain.visible(8, 3, 2)
    assert t[7].nonzero().flatten().tolist() == [5, 6, 7] and b[7].nonzero().flatten().tolist() == [0, 1]
    assert b[4].nonzero().flatten().tolist() == [0] and not b[3].any()      # block 1 (tokens 2, 3) is seen from token 6 on
    assert b[6].nonzero().flatten().tolist() == [0, 1] and b[5].nonzero().flatten().tolist() == [0]
    h = torch.tensor([[1.0], [10.0], [100.0]], dtype=torch.float64)
    w = torch.tensor([[0.25, 0.5, 2.0]], dtype=torch.float64)
    assert plain.with_input_conv(h, w).flatten().tolist() == [1 + 2, 10 + 20 + 0.5, 100 + 200 + 5 + 0.25]
    S = plain.lightning_states(*(torch.tensor(v, dtype=torch.float64).reshape(3, 1, 1) for v in ([1, 1, 2], [1, 2, 3], [1, 1, 1])), [0.5])
    assert S.flatten().tolist() == [1.0, 2.5, 8.5]
    assert plain.query_temperature(5, 1.0, 2).tolist() == pytest.approx([1, 1 + 0.6931471805599453, 1.6931471805599453,
                                                                        1 + 1.0986122886681098, 2.09861228866811])


@pytest.mark.parametrize("name", ["gzA", "gzC"])
def test_the_sharpened_weights_show_a_fault(tmp_path, name):
    """A window one token off, blocks of another size, a wrong source, decay or temperature, a lost tap or a lost expert
    move the plain logits by far more than the tolerance of the engine's comparison (in bfloat16 too for most of them)."""
    cfg, seed = GOPUZEN_CONFIGS[name]
    d = make_gopuzen_dir(str(tmp_path / name), cfg, seed)
    base, P = plain.load(d)
    toks = list(clear_tokens(d, 75, cfg["vocab"], 99))
    ref = plain.forward(base, P, toks)

    def moved(change, tensors=None):
        c, Q = copy.deepcopy(base), dict(P)
        if change:
            change(c["layers"])
        Q.update(tensors or {})
        return rel_err(plain.forward(c, Q, toks)[-20:], ref[-20:])

    for i in (0, 2):
        assert moved(lambda L: L[i]["mixer"]["mask"].update(size=L[i]["mixer"]["mask"]["size"] + 1)) > 0.05
        assert moved(lambda L: L[i]["mixer"]["mask"].update(pool=L[i]["mixer"]["mask"]["pool"] + 1)) > 0.01
    assert moved(lambda L: L[1]["mixer"]["left"]["q_temp"].update(every=L[1]["mixer"]["left"]["q_temp"]["every"] + 1)) > 1e-3
    assert moved(lambda L: L[1]["mixer"]["right"].update(decay=[x * 0.9 for x in L[1]["mixer"]["right"]["decay"]])) > 0.1
    w = P["l1.canon1"].clone()
    w[:, 0] = 0
    assert moved(None, {"l1.canon1": w}) > 0.1
    assert moved(None, {"l0.ls1": P["l0.ls1"] * 0 + 1}) > 0.02
    assert moved(lambda L: [m["mlp"]["router"].update(experts=m["mlp"]["router"]["experts"] + 1) for m in L
                            if m["mlp"] and m["mlp"]["kind"] == "moe"],
                 {k.replace(".e0.", f".e{L['mlp']['router']['experts']}."): v for i, L in enumerate(base["layers"])
                  if L["mlp"] and L["mlp"]["kind"] == "moe" for k, v in P.items() if k.startswith(f"l{i}.mlp.e0.")}) > 0.1
