"""A linear recurrence with a fixed decay per head, and two mixers side by side whose outputs are
normed before they are added."""
from __future__ import annotations

import torch

from ..config.base import ConfigError, PartSpec
from .base import MIXERS, Mixer, StateSpec, WeightSpec, register_mixer, to_device


@register_mixer("lightning")
class LightningMixer(Mixer):
    """With x the token's row, heads of queries and keys of ``head_dim`` and of values of ``value_dim``:

        q = silu(Wq x), k = silu(Wk x), v = silu(Wv x)
        S_h <- decay_h S_h + k_h v_h^T,   o_h = S_h^T q_h          (S [head_dim, value_dim], zero at the start)
        out = Wo [ [o_h]_h / rms([o_h]_h) * norm * sigmoid(Wg x) ]  (one root mean square over all heads)

    S is the request's state, float32, kept transposed, [head][value channel][key channel].  The four
    projections are one product whose results stay float32; everything up to the output matrix is
    float32.  ``external``: see ``GroupedAttention``."""

    graph_safe = True
    input_goes_to_linear = True

    def __init__(self, hidden_size: int, num_heads: int, head_dim: int, value_dim: int, decay, norm_eps: float = 1e-6,
                 external: bool = False):
        self.hidden_size = int(hidden_size)
        self.num_heads = int(num_heads)
        self.head_dim = int(head_dim)
        self.value_dim = int(value_dim)
        self.decay_list = tuple(float(d) for d in decay)
        self.norm_eps = float(norm_eps)
        self.external = bool(external)
        if min(self.hidden_size, self.num_heads, self.head_dim, self.value_dim) <= 0:
            raise ConfigError("lightning: sizes must be positive")
        if len(self.decay_list) != self.num_heads:
            raise ConfigError(f"lightning: {len(self.decay_list)} decays for {self.num_heads} heads")
        if self.head_dim > 256:
            raise ConfigError(f"lightning: heads of {head_dim} key channels (up to 256)")
        self.w_in = self.w_o = self.norm = self.decay = None

    @property
    def columns(self) -> int:
        return 2 * self.num_heads * (self.head_dim + self.value_dim)

    def state_spec(self):
        return StateSpec((self.num_heads * self.value_dim * self.head_dim,), torch.float32)

    def weight_specs(self):
        W, H, D, E = self.hidden_size, self.num_heads, self.head_dim, self.value_dim
        return {"q": WeightSpec((H * D, W)), "k": WeightSpec((H * D, W)), "v": WeightSpec((H * E, W)),
                "g": WeightSpec((H * E, W)), "norm": WeightSpec((H * E,), "norm"), "o": WeightSpec((W, H * E))}

    def stacked(self, weights) -> list:
        return [weights[n] for n in ("q", "k", "v", "g")]

    def load_weights(self, weights, dtype, device):
        if not self.external:
            w = self.stacked(weights)
            self.w_in = to_device(torch.cat([t.to(w[0].dtype) for t in w], 0), dtype, device)
        self.w_o = to_device(weights["o"], dtype, device)
        self.norm = weights["norm"].to(torch.float32).contiguous().to(device)
        self.decay = torch.tensor(self.decay_list, dtype=torch.float64).to(torch.float32).to(device)

    def forward_projected(self, ctx, proj):
        ops = ctx.ops
        H, D, E = self.num_heads, self.head_dim, self.value_dim
        o = ops.lightning(proj, self.decay, ctx.state, ctx.batch, H, D, E, chunked=False if min(self.decay_list) < 0 else None)
        gate = proj[:, H * (2 * D + E):self.columns]
        y = ops.row_norm_gate(o, gate, self.norm, self.norm_eps, ctx.act_dtype)
        return ops.linear(y, self.w_o, out_dtype=torch.float32, partials=True)

    def forward(self, ctx, x):
        if self.external:
            raise RuntimeError("lightning: its projections were left to a combining mixer")
        return self.forward_projected(ctx, ctx.ops.linear(x, self.w_in, out_dtype=torch.float32))


@register_mixer("normed_pair")
class NormedPair(Mixer):
    """Two mixers side by side that read the same rows: out = (norm_l(left(x)) + norm_r(right(x))) / 2, each norm an
    RMS norm over the row with a weight of its own (``left.out``, ``right.out``).

    Both must be able to start from a projection that was formed for them (``external`` / ``stacked`` /
    ``forward_projected``): the input matrices of both are one product.  One of them may keep keys and
    values (``cache_spec``) and one a state (``state_spec``).  The two outputs leave as they are, with
    their norms' weights, for the kernel that adds the mixer's result to the stream
    (``ops.OutputTerm``).  Their tensors are named ``left.*`` and ``right.*``."""

    graph_safe = True
    input_goes_to_linear = True

    def __init__(self, hidden_size: int, left, right, norm_eps: float = 1e-6):
        self.hidden_size = int(hidden_size)
        self.norm_eps = float(norm_eps)
        self.left, self.right = self._build(left), self._build(right)
        if sum(m.cache_spec() is not None for m in (self.left, self.right)) > 1 or \
                sum(m.state_spec() is not None for m in (self.left, self.right)) > 1:
            raise ConfigError("normed pair: both mixers ask for a cache, or both for a state; a layer call has one of each")
        self.w_in = self.out_left = self.out_right = None

    @staticmethod
    def _build(spec):
        if not isinstance(spec, PartSpec):
            raise ConfigError("normed pair: 'left' and 'right' are the specs of two mixers")
        m = MIXERS.build(PartSpec(spec.kind, dict(spec.args, external=True)))
        if not hasattr(m, "forward_projected"):
            raise ConfigError(f"normed pair: a '{spec.kind}' cannot start from a given projection")
        return m

    def cache_spec(self):
        return self.left.cache_spec() or self.right.cache_spec()

    def state_spec(self):
        return self.left.state_spec() or self.right.state_spec()

    def flops_per_query_key_pair(self):
        return self.left.flops_per_query_key_pair() + self.right.flops_per_query_key_pair()

    def weight_specs(self):
        specs = {f"left.{k}": v for k, v in self.left.weight_specs().items()}
        specs.update({f"right.{k}": v for k, v in self.right.weight_specs().items()})
        return specs | {"left.out": WeightSpec((self.hidden_size,), "norm"), "right.out": WeightSpec((self.hidden_size,), "norm")}

    def load_weights(self, weights, dtype, device):
        stacked = []
        for name, m in (("left.", self.left), ("right.", self.right)):
            own = {k[len(name):]: v for k, v in weights.items() if k.startswith(name) and k != name + "out"}
            m.load_weights(own, dtype, device)
            stacked += m.stacked(own)
        self.w_in = to_device(torch.cat([t.to(stacked[0].dtype) for t in stacked], 0), dtype, device)
        self.out_left = weights["left.out"].to(torch.float32).contiguous().to(device)
        self.out_right = weights["right.out"].to(torch.float32).contiguous().to(device)

    def forward(self, ctx, x):
        proj = ctx.ops.linear(x, self.w_in, out_dtype=torch.float32)
        n = self.left.columns
        a = self.left.forward_projected(ctx, proj)
        b = self.right.forward_projected(ctx, proj[:, n:])
        return ctx.ops.OutputTerm(a, pair=(b, self.out_left, self.out_right, self.norm_eps))
