"""Typed configuration of the Gopuzen decoder, read from its config.json.

The file lists its layers one by one (``layers``): each entry names its mixer (``type``: ``attention``,
a rotated grouped attention that sees a window of tokens and, before it, the mean keys of whole
blocks of tokens; or ``parallel``, a full attention without rotation whose queries grow with the
position beside a linear recurrence with a fixed decay per head) with the mixer's sizes (``mixer``)
and its feed-forward (``mlp``: a dense gated one with biases, a mixture of experts some of which
hand their input on, or null for none).  An attention with ``kv_from: j`` has no keys and values of
its own: it reads what layer j's call left in its cache.  Layers norm before and after each
sublayer, scale what they add, and convolve what the sublayers read over time.  Sizes and constants
all come from the file; nothing is assumed equal between layers.
"""
from __future__ import annotations

import copy
from dataclasses import dataclass, field

from .base import ConfigError, LayerCall, LayerSpec, ModelConfig, PartSpec, coerce, optional, require

ARCHITECTURE = "Gopuzen"

#: a length limit for callers that give none (the file names none)
DEFAULT_MAX_POSITIONS = 1 << 20


def _obj(m: dict, key: str, where: str, needed: bool = True):
    v = m.get(key)
    if v is None and not needed:
        return None
    if not isinstance(v, dict):
        raise ConfigError(f"{where}.{key} must be an object")
    return v


def _rotation(m: dict, dim: int, where: str) -> PartSpec | None:
    rot = _obj(m, "rot", where, needed=False)
    if rot is None:
        return None
    dims = optional(rot, "dims", int, dim, where + ".rot")
    if dims == 0:
        return None
    if dims < 0 or dims % 2 or dims > dim:
        raise ConfigError(f"{where}.rot.dims={dims} must be even and at most {dim}")
    return PartSpec("rope", {"head_dim": dim, "theta": require(rot, "base", float, where + ".rot"),
                             "pairing": "interleaved", "rotary_dim": dims})


def _mask(m: dict, where: str) -> tuple[int, int]:
    """(window, block size of the mean keys before it), 0 for none."""
    mask = _obj(m, "mask", where, needed=False)
    if mask is None:
        return 0, 0
    size = require(mask, "size", int, where + ".mask")
    pool = optional(mask, "pool", int, 0, where + ".mask")
    if size <= 0 or pool < 0:
        raise ConfigError(f"{where}.mask: size {size} must be positive and pool {pool} not negative")
    return size, pool


def _heads(m: dict, where: str) -> dict:
    heads = require(m, "heads", int, where)
    dim = require(m, "dim", int, where)
    return {"num_heads": heads, "num_kv_heads": optional(m, "kv_heads", int, heads, where), "head_dim": dim,
            "value_dim": optional(m, "vdim", int, dim, where), "scale": require(m, "scale", float, where),
            "position": _rotation(m, dim, where)}


def _q_temp(m: dict, where: str) -> dict:
    t = _obj(m, "q_temp", where, needed=False)
    if t is None:
        return {}
    every = require(t, "every", int, where + ".q_temp")
    if every <= 0:
        raise ConfigError(f"{where}.q_temp.every must be positive, found {every}")
    return {"q_temp_coef": require(t, "coef", float, where + ".q_temp"), "q_temp_every": every}


def _mlp_spec(i: int, width: int, m) -> PartSpec:
    where = f"config.json: layers[{i}].mlp"
    if m is None:
        return PartSpec("none", {"hidden_size": width})
    if not isinstance(m, dict):
        raise ConfigError(f"{where} must be an object or null")
    kind = require(m, "kind", str, where)
    if kind == "dense":
        return PartSpec("swiglu", {"hidden_size": width, "intermediate_size": require(m, "ff", int, where),
                                   "names": ("gate", "up", "down"), "bias": True})
    if kind == "moe":
        ex, ro = _obj(m, "expert", where), _obj(m, "router", where)
        return PartSpec("routed_experts", {
            "hidden_size": width,
            "intermediate_size": require(ex, "ff", int, where + ".expert"),
            "num_experts": require(ro, "experts", int, where + ".router"),
            "top": require(ro, "top", int, where + ".router"),
            "identity": optional(ro, "identity", int, 0, where + ".router"),
            "limit": None, "act_alpha": 1.0, "up_offset": 0.0,          # silu(gate) * up, no clamp
            "correction": True, "router_softmax": True,
        })
    raise ConfigError(f"{where}.kind '{kind}' is not a feed-forward of this architecture (dense, moe)")


@dataclass
class GopuzenConfig(ModelConfig):
    hidden_size: int
    vocab_size: int
    layers: list
    norm_eps: float
    conv_taps: int
    embedding_scale: float = 1.0
    max_position_embeddings: int = DEFAULT_MAX_POSITIONS
    eos_token_id: int | None = None
    extra: dict = field(default_factory=dict, repr=False)

    architecture = ARCHITECTURE
    tie_word_embeddings = False
    caller_options = {}

    @classmethod
    def from_dict(cls, d: dict) -> "GopuzenConfig":
        if d.get("architecture") != ARCHITECTURE:
            raise ConfigError(f"config.json: 'architecture' must be '{ARCHITECTURE}', found {d.get('architecture')!r}")
        layers = d.get("layers")
        if not isinstance(layers, list) or not layers:
            raise ConfigError("config.json: 'layers' must list at least one layer")
        norm = _obj(d, "norm", "config.json")
        conv = _obj(d, "canon", "config.json")
        emb = _obj(d, "embedding", "config.json", needed=False) or {}
        eos = d.get("eos_token_id")
        known = {"architecture", "architectures", "layers", "norm", "canon", "embedding", "vocab", "width",
                 "max_position_embeddings", "eos_token_id"}
        cfg = cls(
            hidden_size=require(d, "width", int),
            vocab_size=require(d, "vocab", int),
            layers=copy.deepcopy(layers),
            norm_eps=require(norm, "eps", float, "config.json: norm"),
            conv_taps=require(conv, "taps", int, "config.json: canon"),
            embedding_scale=optional(emb, "scale", float, 1.0, "config.json: embedding"),
            max_position_embeddings=optional(d, "max_position_embeddings", int, DEFAULT_MAX_POSITIONS),
            eos_token_id=eos if isinstance(eos, int) and not isinstance(eos, bool) else None,
            extra={k: v for k, v in d.items() if k not in known},
        )
        cfg.validate()
        return cfg

    # ---- which layers share a cache ---------------------------------------
    def _mixer(self, i: int) -> dict:
        m = self.layers[i].get("mixer")
        if not isinstance(m, dict):
            raise ConfigError(f"config.json: layers[{i}].mixer must be an object")
        return m

    def kv_source(self, i: int) -> int | None:
        """The layer whose cache layer i reads, or None if it fills its own."""
        j = self._mixer(i).get("kv_from")
        return None if j is None else coerce(j, "kv_from", int, f"config.json: layers[{i}].mixer")

    def _cache_needs(self, i: int) -> tuple[int, tuple]:
        """(window, block sizes) that the cache layer i works on must keep for all layers that read it."""
        src = self.kv_source(i)
        src = i if src is None else src
        masks = [_mask(self._mixer(k), f"config.json: layers[{k}].mixer") for k in range(len(self.layers))
                 if self.layers[k].get("type") == "attention" and (k == src or self.kv_source(k) == src)]
        window = 0 if any(w == 0 for w, _ in masks) else max(w for w, _ in masks)
        return window, tuple(sorted({p for _, p in masks if p}))

    def validate(self) -> None:
        for k in ("hidden_size", "vocab_size", "max_position_embeddings", "conv_taps"):
            if getattr(self, k) <= 0:
                raise ConfigError(f"config.json: '{k}' must be positive, found {getattr(self, k)}")
        if not (self.norm_eps > 0):
            raise ConfigError(f"config.json: norm.eps={self.norm_eps} must be positive")
        for i, L in enumerate(self.layers):
            if not isinstance(L, dict):
                raise ConfigError(f"config.json: layers[{i}] must be an object")
        for i, L in enumerate(self.layers):
            j = self.kv_source(i)
            if j is None:
                continue
            where = f"config.json: layers[{i}].mixer.kv_from={j}"
            if L.get("type") != "attention":
                raise ConfigError(f"{where}: only an attention layer reads another layer's cache")
            if not 0 <= j < len(self.layers) or j == i or self.layers[j].get("type") != "attention" \
                    or self.kv_source(j) is not None:
                raise ConfigError(f"{where} must name another attention layer that fills a cache of its own")
            if j > i:
                raise ConfigError(f"{where}: the layer whose cache is read must run before the reader")
        specs = self.layer_specs()      # every entry is read once, so that a bad one is reported at load
        for i in range(len(self.layers)):
            j = self.kv_source(i)
            if j is None:
                continue
            a, b = specs[i].mixer.args, specs[j].mixer.args
            if any(a[k] != b[k] for k in ("num_kv_heads", "head_dim", "value_dim", "position")):
                raise ConfigError(f"config.json: layers[{i}].mixer.kv_from={j}: key/value heads, their sizes and the "
                                  "rotation of the two layers must be equal")

    def to_dict(self) -> dict:
        d = {"architecture": ARCHITECTURE, "layers": copy.deepcopy(self.layers), "norm": {"eps": self.norm_eps},
             "canon": {"taps": self.conv_taps}, "embedding": {"scale": self.embedding_scale}, "vocab": self.vocab_size,
             "width": self.hidden_size}
        if self.max_position_embeddings != DEFAULT_MAX_POSITIONS:
            d["max_position_embeddings"] = self.max_position_embeddings
        if self.eos_token_id is not None:
            d["eos_token_id"] = self.eos_token_id
        for k, v in self.extra.items():
            d.setdefault(k, v)
        return d

    # ---- what a layer is made of -------------------------------------------
    def _attention_spec(self, i: int, m: dict, where: str) -> PartSpec:
        window, pool = _mask(m, where)
        kept, pools = self._cache_needs(i)
        return PartSpec("grouped_attention", dict(
            _heads(m, where), hidden_size=self.hidden_size, window=window, pool=pool, cache_window=kept,
            cache_pools=pools, head_gate=True, shared_cache=self.kv_source(i) is not None, **_q_temp(m, where)))

    def _parallel_spec(self, m: dict, where: str) -> PartSpec:
        left, right = _obj(m, "left", where), _obj(m, "right", where)
        lw, rw = where + ".left", where + ".right"
        window, pool = _mask(left, lw)
        heads = require(right, "heads", int, rw)
        decay = right.get("decay")
        if not isinstance(decay, list) or len(decay) != heads:
            raise ConfigError(f"{rw}.decay must list a number for each of the {heads} heads")
        dim = require(right, "dim", int, rw)
        return PartSpec("normed_pair", {
            "hidden_size": self.hidden_size, "norm_eps": self.norm_eps,
            "left": PartSpec("grouped_attention", dict(
                _heads(left, lw), hidden_size=self.hidden_size, window=window, pool=pool, cache_window=window,
                cache_pools=(pool,) if pool else (), head_gate=False, **_q_temp(left, lw))),
            "right": PartSpec("lightning", {
                "hidden_size": self.hidden_size, "num_heads": heads, "head_dim": dim,
                "value_dim": optional(right, "vdim", int, dim, rw),
                "decay": tuple(coerce(x, "decay", float, rw) for x in decay), "norm_eps": self.norm_eps}),
        })

    def layer_specs(self) -> list[LayerSpec]:
        block = PartSpec("sandwich", {"hidden_size": self.hidden_size, "conv_taps": self.conv_taps, "layer_scale": True})
        norm = self.final_norm_spec()
        specs = []
        for i, L in enumerate(self.layers):
            kind, m, where = require(L, "type", str, f"config.json: layers[{i}]"), self._mixer(i), f"config.json: layers[{i}].mixer"
            if kind == "attention":
                mixer = self._attention_spec(i, m, where)
            elif kind == "parallel":
                mixer = self._parallel_spec(m, where)
            else:
                raise ConfigError(f"config.json: layers[{i}].type '{kind}' is not a mixer of this architecture "
                                  "(attention, parallel)")
            specs.append(LayerSpec(block, mixer, _mlp_spec(i, self.hidden_size, L.get("mlp")), norm))
        return specs

    def layer_schedule(self) -> list[LayerCall]:
        """Every layer once, in order; a layer with ``kv_from`` works on the cache of the layer it names, writes
        nothing there, and has a state of its own (the last inputs of its convolutions)."""
        out = []
        for i in range(len(self.layers)):
            j = self.kv_source(i)
            out.append(LayerCall(i, i) if j is None else LayerCall(i, j, False, state=i))
        return out

    def final_norm_spec(self) -> PartSpec:
        return PartSpec("layernorm", {"size": self.hidden_size, "eps": self.norm_eps})
