"""The Pupinex configuration: what its config.json turns into, what is refused, the run order and who keeps which
cache and state, and properties of the plain implementation (all on the CPU)."""
import copy
import json
import math

import pytest
import torch

import plain_pupinex as plain
from helpers import rel_err
from pupinex_models import PUPINEX_CONFIGS, PX_A, PX_B, PX_C, clear_tokens, make_pupinex_dir
from tffinfer_amd.cache import CacheManager
from tffinfer_amd.cache.sizing import state_bytes
from tffinfer_amd.config.base import ConfigError, LayerCall, PartSpec
from tffinfer_amd.models import build_model_skeleton, config_from_dict, load_config
from tffinfer_amd.parts import (GatedLinearAttention, GroupedAttention, KVCacheSpec, LayerNorm, LinearRotaryEmbedding, MatrixMemory,
                                MixerPair, NoFeedForward, POSITION_ENCODINGS, PreNormBlock, RoutedExperts, StateSpec, SwiGLU)
from tffinfer_amd.weights.loader import WeightError, check_weights
from tffinfer_amd.weights.safetensors_io import load_model_dir


def _model(cfg):
    return build_model_skeleton(config_from_dict(copy.deepcopy(cfg)))


def test_every_size_and_constant_comes_from_the_file():
    model = _model(PX_A)
    assert [type(b) for b in model.blocks] == [PreNormBlock] * 5
    assert [type(b.mixer) for b in model.blocks] == [GroupedAttention, GatedLinearAttention, MixerPair, GroupedAttention,
                                                     GatedLinearAttention]
    assert [type(b.feed_forward) for b in model.blocks] == [SwiGLU, RoutedExperts, RoutedExperts, NoFeedForward, SwiGLU]
    a = model.blocks[0].mixer
    assert (a.num_heads, a.num_kv_heads, a.head_dim, a.value_dim, a.scale, a.window) == (4, 2, 16, 24, 0.2, 20)
    assert (a.has_bias, a.has_output_bias, a.has_sinks, a.qk_norm_eps, a.has_gate) == (True, True, True, None, False)
    assert (a.position.rotary_dim, a.position.theta, a.position.pairing) == (8, 500.0, "interleaved")
    assert type(a.position).__name__ == "RotaryEmbedding" and a.cache_spec() == KVCacheSpec(2, 32, 20)
    g = model.blocks[1].mixer
    assert (g.num_heads, g.head_dim, g.value_dim, g.tau, g.decay_rank, g.norm_eps) == (3, 8, 12, 4.0, 6, 1e-2)
    assert g.state_spec() == StateSpec((3 * 8 * 12,)) and g.cache_spec() is None
    p = model.blocks[2].mixer
    assert p.joint and (p.left_scale, p.right_scale) == (0.7, 0.4)
    assert (p.left.window, p.left.scale, p.left.qk_norm_eps, p.left.has_bias, p.left.has_output_bias, p.left.has_sinks) == \
        (13, 0.5, 1e-2, True, False, False)
    assert isinstance(p.left.position, LinearRotaryEmbedding) and (p.left.position.factor, p.left.position.pairing) == (3.0, "half")
    assert isinstance(p.right, MatrixMemory) and (p.right.num_heads, p.right.head_dim, p.right.value_dim, p.right.gate_cap) == (3, 8, 12, 10.0)
    assert p.state_spec().shape[0] >= 3 * 8 * 13 + 3 and p.state_spec().shape[0] % 4 == 0
    e = model.blocks[2].feed_forward
    assert (e.num_experts, e.top, e.groups, e.keep_groups, e.intermediate_size, e.shared, e.shared_expert.intermediate_size,
            e.weight_scale) == (6, 2, 3, 2, 16, 40, 40, 1.0)
    assert not e.has_correction and not e.router_softmax and e.normalize and (e.limit, e.act_alpha, e.up_offset) == (math.inf, 1.0, 0.0)
    assert model.blocks[0].feed_forward.act == (1.5, 1.702, 1.0)
    assert isinstance(model.final_norm, LayerNorm) and not model.final_norm.has_bias and model.final_norm.eps == 1e-2
    b = model.embedding.bigram
    assert (b.buckets, b.mul_prev, b.mul_cur) == (211, 31, 7) and model.head.tied_to is model.embedding and model.graph_safe()
    m = copy.deepcopy(PX_B)
    del m["layers"][1]["mixer"]["kv_heads"], m["layers"][1]["mixer"]["vdim"], m["layers"][1]["mlp"]["router"]["groups"]
    del m["layers"][1]["mlp"]["router"]["scale"], m["layers"][1]["mlp"]["shared"], m["embedding"], m["loop"]
    c = _model(m)
    r = c.blocks[1].feed_forward
    assert (c.blocks[1].mixer.num_kv_heads, c.blocks[1].mixer.value_dim, r.groups, r.weight_scale, r.shared) == (2, 32, 1, 1.0, 0)
    assert c.embedding.bigram is None and not c.keeps_embedding


def test_run_order_caches_and_states():
    """The loop's passes follow each other, each call with a cache and state of its own; the embedding's output is added
    before every pass but the first; the embedding's last token is one more state."""
    calls = config_from_dict(copy.deepcopy(PX_A)).layer_schedule()
    assert [(c.layer, c.add_embedding) for c in calls] == [(0, False), (1, False), (2, False), (1, True), (2, False), (1, True), (2, False),
                                                           (3, False), (4, False)]
    assert [c.cache for c in calls] == list(range(9))
    assert [(c.layer, c.add_embedding) for c in config_from_dict(copy.deepcopy(PX_B)).layer_schedule()] == \
        [(0, False), (1, False), (2, False), (0, True), (1, False), (2, False)]
    assert config_from_dict(copy.deepcopy(PX_C)).layer_schedule() == [LayerCall(i, i) for i in range(4)]
    model = _model(PX_A)
    needs = model.call_requirements()
    assert len(needs) == 10 and needs[9] == (9, True, None, StateSpec((1,), torch.int32)) and model.keeps_embedding
    cache = CacheManager(needs, page_size=16, num_pages=8, max_seqs=2, dtype=torch.float32, device="cpu")
    assert sorted(cid for g in cache.groups for cid in g.cache_ids) == [0, 2, 4, 6, 7]
    assert sorted(cache.state_tensors) == [1, 2, 3, 4, 5, 6, 8, 9] and cache.state_tensors[9].dtype == torch.int32
    right = model.blocks[2].mixer.state_spec().shape[0]
    assert state_bytes(needs, 2) == 3 * 4 * (3 * 288 + 3 * right + 512 + 1)
    # a slot that is taken again starts from zeros
    cache.add_request("a")
    cache.state_tensors[9][cache.slot("a")] = 7
    slot = cache.slot("a")
    cache.release("a")
    cache.add_request("b")
    assert cache.slot("b") == slot and int(cache.state_tensors[9][slot]) == 0


def test_tensor_names_follow_the_files():
    names = _model(PX_A).expected_tensors()
    for n in ("embed", "bigram", "final.norm", "l0.norm1", "l0.norm2", "l0.mix.q", "l0.mix.q.b", "l0.mix.k.b", "l0.mix.v.b", "l0.mix.o",
              "l0.mix.o.b", "l0.mix.sink", "l0.mlp.gate", "l0.mlp.up", "l0.mlp.down", "l1.mix.q", "l1.mix.k", "l1.mix.v", "l1.mix.g",
              "l1.mix.a1", "l1.mix.a2", "l1.mix.a2.b", "l1.mix.norm", "l1.mix.o", "l1.mlp.router", "l1.mlp.e7.down", "l1.mlp.shared.gate",
              "l1.mlp.shared.up", "l1.mlp.shared.down", "l1.mlp.shared.sg", "l2.mix.left.q", "l2.mix.left.q.b", "l2.mix.left.q.norm",
              "l2.mix.left.k.norm", "l2.mix.left.v.b", "l2.mix.left.o", "l2.mix.right.q", "l2.mix.right.g", "l2.mix.right.i",
              "l2.mix.right.i.b", "l2.mix.right.f.b", "l2.mix.right.norm", "l2.mix.right.o"):
        assert n in names, n
    assert not any(n in names for n in ("head", "l0.norm1.b", "final.norm.b", "l0.mix.q.norm", "l2.mix.left.o.b", "l2.mix.left.sink",
                                        "l1.mlp.correction", "l1.mlp.e8.gate", "l3.mlp.gate", "l0.mix.g"))
    assert names["l3.norm2"].optional and not names["l3.norm1"].optional
    assert names["bigram"].shape == (212, 64) and names["l2.mix.left.q.norm"].shape == (64,) and names["l2.mix.left.k.norm"].shape == (32,)
    assert names["l1.mix.a1"].shape == (6, 64) and names["l1.mix.a2"].shape == (24, 6) and names["l1.mix.norm"].shape == (12,)
    assert names["l2.mix.right.norm"].shape == (36,) and names["l2.mlp.shared.down"].shape == (64, 40)
    assert names["l0.mix.sink"].shape == (4,) and names["l1.mlp.router"].shape == (8, 64)


def test_round_trip_and_refusals(tmp_path):
    d = make_pupinex_dir(str(tmp_path / "m"), PX_A, 1, sharp=False)
    cfg = load_config(d)
    back = cfg.to_dict()
    assert all(back[k] == PX_A[k] for k in PX_A)
    assert config_from_dict(json.loads(json.dumps(back))).layer_schedule() == cfg.layer_schedule()
    found, names = load_model_dir(d), build_model_skeleton(cfg).expected_tensors()
    check_weights(names, found, set(), d)
    # a file without the decay's inner size in its configuration: the tensors give it
    open_rank = copy.deepcopy(PX_A)
    for L in open_rank["layers"]:
        L["mixer"].pop("decay_rank", None)
    check_weights(_model(open_rank).expected_tensors(), found, set(), d)
    del found["l0.mix.o.b"]
    with pytest.raises(WeightError) as e:
        check_weights(names, found, set(), d)
    assert e.value.missing == ["l0.mix.o.b"]
    for breaker, text in (
            (lambda c: c["layers"][0].update(type="other"), "mixer"),
            (lambda c: c["layers"][1]["mlp"].update(kind="sparse"), "feed-forward"),
            (lambda c: c["layers"][0]["mlp"].pop("limit"), "limit"),
            (lambda c: c["layers"][0]["mixer"]["mask"].update(size=0), "mask"),
            (lambda c: c["layers"][0]["mixer"]["rot"].update(dims=7), "even"),
            (lambda c: c["layers"][0]["mixer"].update(kv_heads=3), "multiple"),
            (lambda c: c["layers"][0]["mixer"].pop("scale"), "scale"),
            (lambda c: c["layers"][1]["mixer"].update(tau=0), "tau"),
            (lambda c: c["layers"][1]["mixer"].update(dim=300), "key channels"),
            (lambda c: c["layers"][2]["mixer"]["right"].update(gate_cap=0), "cap"),
            (lambda c: c["layers"][2]["mixer"]["left"]["rot"]["scaling"].update(factor=0), "factor"),
            (lambda c: c["layers"][2]["mixer"].pop("right"), "right"),
            (lambda c: c["layers"][1]["mlp"]["router"]["groups"].update(count=3), "groups"),
            (lambda c: c["layers"][1]["mlp"]["router"]["groups"].update(keep=5), "groups"),
            (lambda c: c["layers"][1]["mlp"]["router"].update(top=5), "groups"),
            (lambda c: c["layers"][1]["mlp"]["router"].update(top=9), "top"),
            (lambda c: c["embedding"]["bigram"].update(buckets=0), "buckets"),
            (lambda c: c["embedding"]["bigram"].pop("mul_cur"), "mul_cur"),
            (lambda c: c["loop"].update(stop=9), "loop"),
            (lambda c: c["loop"].update(times=0), "loop"),
            (lambda c: c.pop("norm"), "norm"),
            (lambda c: c["norm"].update(eps=0), "eps")):
        bad = copy.deepcopy(PX_A)
        breaker(bad)
        with pytest.raises(ConfigError, match=text):
            _model(bad)


def test_the_linear_rotation_divides_every_angle():
    args = {"head_dim": 16, "theta": 500.0, "rotary_dim": 8}
    one = POSITION_ENCODINGS.build(PartSpec("rope", args)).angles(50)
    assert torch.allclose(POSITION_ENCODINGS.build(PartSpec("rope_linear", dict(args, factor=4.0))).angles(50), one / 4.0)
    keys = {POSITION_ENCODINGS.build(PartSpec("rope_linear", dict(args, factor=f))).table_key() for f in (2.0, 4.0)}
    assert len(keys) == 2


def test_the_plain_functions_on_cases_done_by_hand():
    assert plain.bigram_rows([3, 5, 2], 10, 7, 3) == [10, (21 + 15) % 10, (35 + 6) % 10]
    one = lambda *v: torch.tensor(v, dtype=torch.float64).reshape(-1, 1, 1)      # noqa: E731
    assert plain.gla_states(one(1, 1, 2), one(1, 2, 3), one(1, 1, 1), one(0.9, 0.5, 0.25)).flatten().tolist() == [1.0, 2.5, 7.25]
    i, f = torch.log(torch.tensor([[0.5], [4.0]], dtype=torch.float64)), torch.log(torch.tensor([[0.5], [0.25]], dtype=torch.float64))
    # m: max(ln .5, ln .5) = ln .5, max(ln .125, ln 4) = ln 4
    o = plain.mlstm_states(one(1, 1), one(1, 1), one(3, 5), i, f).flatten()
    assert o[0] == pytest.approx(3 / (2 + 1e-6)) and o[1] == pytest.approx((0.125 / 4 * 3 + 5) / (1 + 0.125 / 4 + 1e-6))
    r = {"top": 2, "groups": {"count": 3, "keep": 1}}
    chosen, gap = plain.router_choice(r, torch.tensor([0.9, 0.1, 0.6, 0.5, 0.2, 0.3]))
    assert sorted(chosen) == [2, 3] and gap == pytest.approx(0.1)
    ones = torch.ones(1, 1, dtype=torch.float64)
    y = plain.dense_ff({"gate": ones * 5, "up": ones * -9, "down": ones}, ones, 2.0)
    assert float(y) == pytest.approx(2 / (1 + math.exp(-1.702 * 2)) * (-2 + 1))
    q = torch.ones(4, 1, 1, dtype=torch.float64)
    o = plain.windowed_attention(q, q, torch.tensor([1.0, 2, 4, 8], dtype=torch.float64).reshape(4, 1, 1), 0.0, 2, torch.tensor([0.0]))
    assert o.flatten().tolist() == pytest.approx([0.5, 1.0, 2.0, 4.0])
    assert plain.run_order({"layers": [0] * 4, "loop": {"start": 1, "stop": 3, "times": 2}}) == [(0, False), (1, False), (2, False), (1, True),
                                                                                                (2, False), (3, False)]


@pytest.mark.parametrize("name", ["pxA", "pxC"])
def test_the_sharpened_weights_show_a_fault(tmp_path, name):
    """A window one token off, a lost sink or bias, another decay, cap or scale, a router without its groups, another pair
    of tokens: each moves the plain logits by far more than the tolerance of the engine's comparison in float32, most of
    them by more than that in bfloat16."""
    cfg, seed = PUPINEX_CONFIGS[name]
    d = make_pupinex_dir(str(tmp_path / name), cfg, seed)
    base, P = plain.load(d)
    toks = list(clear_tokens(d, 40, cfg["vocab"], 99))
    ref = plain.forward(base, P, toks)

    def moved(change, tensors=None):
        c, Q = copy.deepcopy(base), dict(P)
        if change:
            change(c)
        Q.update(tensors or {})
        return rel_err(plain.forward(c, Q, toks)[-20:], ref[-20:])

    for i, L in enumerate(base["layers"]):
        m, at = L["mixer"], lambda c, i=i: c["layers"][i]["mixer"]
        if L["type"] == "attention":
            if m["mask"]["size"] < 38:
                assert moved(lambda c: at(c)["mask"].update(size=m["mask"]["size"] + 1)) > 0.02
            assert moved(None, {f"l{i}.mix.sink": P[f"l{i}.mix.sink"] - 50}) > 0.004
            assert moved(None, {f"l{i}.mix.o.b": P[f"l{i}.mix.o.b"] * 0}) > 0.04
        elif L["type"] == "gla":
            assert moved(lambda c: at(c).update(tau=m["tau"] * 1.5)) > 0.02
        else:
            if m["left"]["mask"]["size"] < 38:
                assert moved(lambda c: at(c)["left"]["mask"].update(size=m["left"]["mask"]["size"] + 1)) > 0.02
            assert moved(lambda c: at(c)["right"].update(gate_cap=m["right"]["gate_cap"] * 0.8)) > 4e-4
            assert moved(lambda c: at(c).update(right_scale=0.0)) > 0.05 and moved(lambda c: at(c).update(left_scale=0.0)) > 0.05
    if base.get("loop"):
        assert moved(lambda c: c["loop"].update(times=base["loop"]["times"] - 1)) > 0.1
    assert moved(lambda c: c["embedding"]["bigram"].update(mul_prev=base["embedding"]["bigram"]["mul_prev"] + 1)) > 0.2
    i = next(i for i, L in enumerate(base["layers"]) if L["mlp"] and L["mlp"]["kind"] == "moe")
    sub = f"l{i}.mlp.shared.sg"
    assert moved(None, {sub: P[sub] * 0}) > 0.1
