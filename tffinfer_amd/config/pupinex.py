"""Typed configuration of the Pupinex decoder, read from its config.json.

The file lists its layers one by one (``layers``): each entry names its mixer (``type``: ``attention``, a windowed
grouped attention with biases and a sink per head; ``gla``, a linear recurrence with a decay per key channel; or
``parallel``, a windowed attention whose queries and keys are normed as a whole beside a matrix memory with
exponential gates) with the mixer's sizes (``mixer``) and its feed-forward (``mlp``: a dense gated one with clamps, a
mixture of experts chosen from the best groups with a shared expert, or null for none).  Layers norm before each
sublayer (layer norms without bias).  ``loop`` runs a span of the layers several times in a row with the same weights
and a cache and state per pass, adding the embedding's output to the stream before each pass but the first.  The
embedding has a second table for pairs of tokens; its first table is the output head too.  Sizes and constants all
come from the file; nothing is assumed equal between layers.
"""
from __future__ import annotations

import copy
from dataclasses import dataclass, field

from .base import ConfigError, LayerCall, LayerSpec, ModelConfig, PartSpec, optional, require

ARCHITECTURE = "Pupinex"

#: a length limit for callers that give none (the file names none)
DEFAULT_MAX_POSITIONS = 1 << 20

#: the slope inside the dense feed-forward's sigmoid, and what is added to its second projection
ACT_ALPHA, UP_OFFSET = 1.702, 1.0


def _obj(m: dict, key: str, where: str, needed: bool = True):
    v = m.get(key)
    if v is None and not needed:
        return None
    if not isinstance(v, dict):
        raise ConfigError(f"{where}.{key} must be an object")
    return v


def _rotation(m: dict, dim: int, pairing: str, where: str) -> PartSpec | None:
    rot = _obj(m, "rot", where, needed=False)
    if rot is None:
        return None
    where += ".rot"
    dims = optional(rot, "dims", int, dim, where)
    if dims == 0:
        return None
    if dims < 0 or dims % 2 or dims > dim:
        raise ConfigError(f"{where}.dims={dims} must be even and at most {dim}")
    args = {"head_dim": dim, "theta": require(rot, "base", float, where), "pairing": pairing, "rotary_dim": dims}
    scaling = _obj(rot, "scaling", where, needed=False)
    if scaling is None:
        return PartSpec("rope", args)
    return PartSpec("rope_linear", dict(args, factor=require(scaling, "factor", float, where + ".scaling")))


def _window(m: dict, where: str) -> int:
    mask = _obj(m, "mask", where, needed=False)
    if mask is None:
        return 0
    size = require(mask, "size", int, where + ".mask")
    if size <= 0:
        raise ConfigError(f"{where}.mask.size={size} must be positive")
    return size


def _attention(width: int, m: dict, pairing: str, where: str, **options) -> PartSpec:
    heads = require(m, "heads", int, where)
    dim = require(m, "dim", int, where)
    return PartSpec("grouped_attention", {
        "hidden_size": width, "num_heads": heads, "num_kv_heads": optional(m, "kv_heads", int, heads, where),
        "head_dim": dim, "value_dim": optional(m, "vdim", int, dim, where), "scale": require(m, "scale", float, where),
        "position": _rotation(m, dim, pairing, where), "window": _window(m, where), "bias": True, **options})


def _recurrence_sizes(width: int, eps: float, m: dict, where: str) -> dict:
    dim = require(m, "dim", int, where)
    return {"hidden_size": width, "num_heads": require(m, "heads", int, where), "head_dim": dim,
            "value_dim": optional(m, "vdim", int, dim, where), "norm_eps": eps}


def _mixer_spec(i: int, width: int, eps: float, kind: str, m) -> PartSpec:
    where = f"config.json: layers[{i}].mixer"
    if not isinstance(m, dict):
        raise ConfigError(f"{where} must be an object")
    if kind == "attention":
        return _attention(width, m, "interleaved", where, output_bias=True, sinks=True)
    if kind == "gla":
        # (the decay's inner size comes from its tensors; a caller that draws random weights names it)
        return PartSpec("gated_linear_attention", dict(_recurrence_sizes(width, eps, m, where), tau=require(m, "tau", float, where),
                                                       decay_rank=optional(m, "decay_rank", int, None, where)))
    if kind == "parallel":
        left, right = _obj(m, "left", where), _obj(m, "right", where)
        rw = where + ".right"
        return PartSpec("mixer_pair", {
            "hidden_size": width,
            "left": _attention(width, left, "half", where + ".left", qk_norm_eps=eps),
            "right": PartSpec("matrix_memory", dict(_recurrence_sizes(width, eps, right, rw),
                                                    gate_cap=require(right, "gate_cap", float, rw))),
            "left_scale": optional(m, "left_scale", float, 1.0, where),
            "right_scale": optional(m, "right_scale", float, 1.0, where),
        })
    raise ConfigError(f"config.json: layers[{i}].type '{kind}' is not a mixer of this architecture (attention, gla, parallel)")


def _mlp_spec(i: int, width: int, m) -> PartSpec:
    where = f"config.json: layers[{i}].mlp"
    if m is None:
        return PartSpec("none", {"hidden_size": width})
    if not isinstance(m, dict):
        raise ConfigError(f"{where} must be an object or null")
    kind = require(m, "kind", str, where)
    if kind == "dense":
        return PartSpec("swiglu", {"hidden_size": width, "intermediate_size": require(m, "ff", int, where),
                                   "names": ("gate", "up", "down"), "limit": require(m, "limit", float, where),
                                   "act_alpha": ACT_ALPHA, "up_offset": UP_OFFSET})
    if kind == "moe":
        ex, ro = _obj(m, "expert", where), _obj(m, "router", where)
        rw = where + ".router"
        groups, shared = _obj(ro, "groups", rw, needed=False), _obj(m, "shared", where, needed=False)
        return PartSpec("routed_experts", {
            "hidden_size": width,
            "intermediate_size": require(ex, "ff", int, where + ".expert"),
            "num_experts": require(ro, "experts", int, rw),
            "top": require(ro, "top", int, rw),
            "limit": None, "act_alpha": 1.0, "up_offset": 0.0,          # silu(gate) * up, no clamp
            "correction": False,
            "groups": require(groups, "count", int, rw + ".groups") if groups is not None else 1,
            "keep_groups": require(groups, "keep", int, rw + ".groups") if groups is not None else 1,
            "weight_scale": optional(ro, "scale", float, 1.0, rw),
            "shared": require(shared, "ff", int, where + ".shared") if shared is not None else 0,
        })
    raise ConfigError(f"{where}.kind '{kind}' is not a feed-forward of this architecture (dense, moe)")


@dataclass
class PupinexConfig(ModelConfig):
    hidden_size: int
    vocab_size: int
    layers: list
    norm_eps: float
    bigram: dict | None = None
    loop_start: int = 0
    loop_stop: int = 0
    loop_times: int = 1
    max_position_embeddings: int = DEFAULT_MAX_POSITIONS
    eos_token_id: int | None = None
    extra: dict = field(default_factory=dict, repr=False)

    architecture = ARCHITECTURE
    tie_word_embeddings = True
    caller_options = {}

    @classmethod
    def from_dict(cls, d: dict) -> "PupinexConfig":
        if d.get("architecture") != ARCHITECTURE:
            raise ConfigError(f"config.json: 'architecture' must be '{ARCHITECTURE}', found {d.get('architecture')!r}")
        layers = d.get("layers")
        if not isinstance(layers, list) or not layers:
            raise ConfigError("config.json: 'layers' must list at least one layer")
        norm = _obj(d, "norm", "config.json")
        emb = _obj(d, "embedding", "config.json", needed=False) or {}
        pairs, where = _obj(emb, "bigram", "config.json: embedding", needed=False), "config.json: embedding.bigram"
        loop = _obj(d, "loop", "config.json", needed=False)
        start = stop = 0
        times = 1
        if loop is not None:
            start, stop, times = (require(loop, k, int, "config.json: loop") for k in ("start", "stop", "times"))
        eos = d.get("eos_token_id")
        known = {"architecture", "architectures", "layers", "norm", "embedding", "loop", "vocab", "width",
                 "max_position_embeddings", "eos_token_id"}
        cfg = cls(
            hidden_size=require(d, "width", int),
            vocab_size=require(d, "vocab", int),
            layers=copy.deepcopy(layers),
            norm_eps=require(norm, "eps", float, "config.json: norm"),
            bigram=None if pairs is None else {k: require(pairs, k, int, where) for k in ("buckets", "mul_prev", "mul_cur")},
            loop_start=start, loop_stop=stop, loop_times=times,
            max_position_embeddings=optional(d, "max_position_embeddings", int, DEFAULT_MAX_POSITIONS),
            eos_token_id=eos if isinstance(eos, int) and not isinstance(eos, bool) else None,
            extra={k: v for k, v in d.items() if k not in known},
        )
        cfg.validate()
        return cfg

    @property
    def has_loop(self) -> bool:
        return self.loop_stop > self.loop_start

    def validate(self) -> None:
        for k in ("hidden_size", "vocab_size", "max_position_embeddings"):
            if getattr(self, k) <= 0:
                raise ConfigError(f"config.json: '{k}' must be positive, found {getattr(self, k)}")
        if not (self.norm_eps > 0):
            raise ConfigError(f"config.json: norm.eps={self.norm_eps} must be positive")
        if self.bigram is not None and self.bigram["buckets"] <= 0:
            raise ConfigError(f"config.json: embedding.bigram.buckets={self.bigram['buckets']} must be positive")
        n = len(self.layers)
        if not (0 <= self.loop_start <= self.loop_stop <= n) or self.loop_times < 1:
            raise ConfigError(f"config.json: loop {self.loop_start} .. {self.loop_stop} x {self.loop_times} "
                              f"does not fit {n} layers")
        for i, L in enumerate(self.layers):
            if not isinstance(L, dict):
                raise ConfigError(f"config.json: layers[{i}] must be an object")
        self.layer_specs()      # every entry is read once, so that a bad one is reported at load

    def to_dict(self) -> dict:
        d = {"architecture": ARCHITECTURE, "layers": copy.deepcopy(self.layers), "norm": {"eps": self.norm_eps},
             "vocab": self.vocab_size, "width": self.hidden_size}
        if self.bigram is not None:
            d["embedding"] = {"bigram": dict(self.bigram)}
        if self.has_loop:
            d["loop"] = {"start": self.loop_start, "stop": self.loop_stop, "times": self.loop_times}
        if self.max_position_embeddings != DEFAULT_MAX_POSITIONS:
            d["max_position_embeddings"] = self.max_position_embeddings
        if self.eos_token_id is not None:
            d["eos_token_id"] = self.eos_token_id
        for k, v in self.extra.items():
            d.setdefault(k, v)
        return d

    def layer_specs(self) -> list[LayerSpec]:
        norm = self.final_norm_spec()
        return [LayerSpec(PartSpec("prenorm"),
                          _mixer_spec(i, self.hidden_size, self.norm_eps, require(L, "type", str, f"config.json: layers[{i}]"),
                                      L.get("mixer")),
                          _mlp_spec(i, self.hidden_size, L.get("mlp")), norm)
                for i, L in enumerate(self.layers)]

    def layer_schedule(self) -> list[LayerCall]:
        """The layers before the looped span, the span ``times`` times in a row (the embedding's output added before
        every pass but the first), the layers after it.  Every call has a cache and state of its own."""
        n = len(self.layers)
        if not self.has_loop:
            return [LayerCall(i, i) for i in range(n)]
        order = [(i, False) for i in range(self.loop_start)]
        for t in range(self.loop_times):
            order += [(i, t > 0 and i == self.loop_start) for i in range(self.loop_start, self.loop_stop)]
        order += [(i, False) for i in range(self.loop_stop, n)]
        return [LayerCall(layer, call, add_embedding=again) for call, (layer, again) in enumerate(order)]

    def final_norm_spec(self) -> PartSpec:
        return PartSpec("layernorm", {"size": self.hidden_size, "eps": self.norm_eps, "has_bias": False})

    def bigram_spec(self) -> dict | None:
        return None if self.bigram is None else dict(self.bigram)
