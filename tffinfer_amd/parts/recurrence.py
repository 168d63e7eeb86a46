"""Linear recurrences whose decay or gates depend on the token: a decay per key channel, and exponential gates per
head with a running maximum.  Both run on one family of kernels."""
from __future__ import annotations

import torch

from ..config.base import ConfigError
from .base import Mixer, StateSpec, WeightSpec, register_mixer, to_device


class _Recurrence(Mixer):
    """What the two have in common: q, k, v and an output gate from one product whose results stay float32, a
    norm over each head, the gate, the output matrix.  Everything up to the output matrix is float32.

    ``external``: whoever combines several mixers that read the same rows forms all their projections in one product
    (``stacked``, ``columns``) and calls ``forward_projected`` or ``inner_projected``; ``external_output``: the output matrix is
    left to that combiner as well (``w_o_host``)."""

    graph_safe = True
    input_goes_to_linear = True
    #: a combiner may form this mixer's projections and apply its output matrix
    joint_input = True

    def __init__(self, hidden_size: int, num_heads: int, head_dim: int, value_dim: int, norm_eps: float = 1e-6,
                 external: bool = False, external_output: bool = False):
        self.hidden_size = int(hidden_size)
        self.num_heads = int(num_heads)
        self.head_dim = int(head_dim)
        self.value_dim = int(value_dim)
        self.norm_eps = float(norm_eps)
        self.external = bool(external)
        self.external_output = bool(external_output)
        if min(self.hidden_size, self.num_heads, self.head_dim, self.value_dim) <= 0:
            raise ConfigError(f"{type(self).__name__}: sizes must be positive")
        if self.head_dim > 256:
            raise ConfigError(f"{type(self).__name__}: heads of {head_dim} key channels (up to 256)")
        self.w_in = self.w_o = self.w_o_host = self.norm = None

    #: the projections' names in the order of the joint product's columns
    ORDER: tuple = ()

    def _widths(self) -> dict:
        """Columns of every projection."""
        H, D, E = self.num_heads, self.head_dim, self.value_dim
        return {"q": H * D, "k": H * D, "v": H * E, "g": H * E}

    @property
    def columns(self) -> int:
        """Columns of the joint projection (a multiple of 4, so that what follows it starts at 16 bytes)."""
        return -(-sum(self._widths()[n] for n in self.ORDER) // 4) * 4

    @property
    def inner_size(self) -> int:
        return self.num_heads * self.value_dim

    def _first_columns(self, names: dict) -> dict:
        """Where each projection's columns start, by the kernels' names for them."""
        at, out = 0, {}
        for n in self.ORDER:
            out[names.get(n, n)] = at
            at += self._widths()[n]
        return out

    def stacked(self, weights) -> list:
        """The projections' matrices in the order of the joint product's columns, and zero rows up to ``columns``."""
        out = [weights[n] for n in self.ORDER]
        pad = self.columns - sum(w.shape[0] for w in out)
        return out + ([torch.zeros(pad, self.hidden_size, dtype=out[0].dtype)] if pad else [])

    def load_weights(self, weights, dtype, device):
        self._load_vectors(weights, lambda n: weights[n].to(torch.float32).contiguous().to(device))
        if not self.external:
            w = self.stacked(weights)
            self.w_in = to_device(torch.cat([t.to(w[0].dtype) for t in w], 0), dtype, device)
        if self.external_output:
            self.w_o_host = weights["o"]
        else:
            self.w_o = to_device(weights["o"], dtype, device)

    def inner_projected(self, ctx, proj, out=None, out_scale: float = 1.0):
        """From the joint projection (float32 [T, >= columns], rows may be strided) to the input of the output matrix,
        [T, heads * value_dim] in the activation type, into ``out`` if given (rows may be strided), times ``out_scale``."""
        if out is None:
            out = torch.empty(proj.shape[0], self.inner_size, dtype=ctx.act_dtype, device=proj.device)
        return self._run(ctx, proj, out, out_scale)

    def forward_projected(self, ctx, proj):
        return ctx.ops.linear(self.inner_projected(ctx, proj), self.w_o, out_dtype=torch.float32, partials=True)

    def forward(self, ctx, x):
        if self.external or self.external_output:
            raise RuntimeError(f"{type(self).__name__}: its projections or its output matrix were left to a combining mixer")
        return self.forward_projected(ctx, ctx.ops.linear(x, self.w_in, out_dtype=torch.float32))


@register_mixer("gated_linear_attention")
class GatedLinearAttention(_Recurrence):
    """With x the token's row, heads of queries and keys of ``head_dim`` and of values of ``value_dim``:

        q = Wq x * head_dim^(-1/2),  k = Wk x,  v = Wv x
        alpha = sigmoid(Wa2 (Wa1 x) + ba2)^(1/tau)                       (a decay per head and key channel)
        S_h <- diag(alpha_h) S_h + k_h v_h^T,   o_h = S_h^T q_h          (S [head_dim, value_dim], zero at the start)
        out = Wo [ o_h / rms(o_h) * norm * silu(Wg x)_h ]_h              (norm [value_dim], shared by the heads)

    S is the request's state, float32, kept transposed, [head][value channel][key channel].  ``decay_rank`` (the inner
    size of the decay's two matrices) may be left open: the tensors then give it."""

    ORDER = ("q", "k", "v", "g", "a1")

    def __init__(self, hidden_size: int, num_heads: int, head_dim: int, value_dim: int, tau: float, decay_rank: int | None = None,
                 norm_eps: float = 1e-6, external: bool = False, external_output: bool = False):
        super().__init__(hidden_size, num_heads, head_dim, value_dim, norm_eps, external, external_output)
        self.tau = float(tau)
        self.decay_rank = None if decay_rank is None else int(decay_rank)
        if not self.tau > 0:
            raise ConfigError(f"gated linear attention: tau={tau} must be positive")
        self.a2_t = self.a_bias = None

    def _widths(self):
        return super()._widths() | {"a1": self.decay_rank or 0}

    def state_spec(self):
        return StateSpec((self.num_heads * self.value_dim * self.head_dim,), torch.float32)

    def weight_specs(self):
        W, N, V = self.hidden_size, self.num_heads * self.head_dim, self.num_heads * self.value_dim
        return {"q": WeightSpec((N, W)), "k": WeightSpec((N, W)), "v": WeightSpec((V, W)), "g": WeightSpec((V, W)),
                "a1": WeightSpec((self.decay_rank, W)), "a2": WeightSpec((N, self.decay_rank)), "a2.b": WeightSpec((N,), "vector"),
                "norm": WeightSpec((self.value_dim,), "norm"), "o": WeightSpec((W, V))}

    def _load_vectors(self, weights, f32):
        if weights["a1"].shape[0] != weights["a2"].shape[1]:
            raise ConfigError(f"gated linear attention: the decay's matrices {tuple(weights['a1'].shape)} and "
                              f"{tuple(weights['a2'].shape)} do not fit each other")
        self.decay_rank = int(weights["a1"].shape[0])
        # the decay's second product is float32 and runs inside the recurrence's kernels
        self.a2_t = f32("a2").t().contiguous()
        self.a_bias, self.norm = f32("a2.b"), f32("norm")

    def _run(self, ctx, proj, out, out_scale):
        return ctx.ops.decay_recurrence(proj, self._first_columns({"g": "gate"}), self.a2_t, self.a_bias, self.tau, self.norm,
                                        self.norm_eps, ctx.state, ctx.batch, self.num_heads, self.head_dim, self.value_dim, out,
                                        out_scale, q_scale=self.head_dim ** -0.5)


@register_mixer("matrix_memory")
class MatrixMemory(_Recurrence):
    """With x the token's row, heads of queries and keys of ``head_dim`` and of values of ``value_dim``:

        q = Wq x * head_dim^(-1/2),  k = Wk x,  v = Wv x
        i = cap tanh((Wi x + bi) / cap),   f = logsigmoid(cap tanh((Wf x + bf) / cap))         (log gates, one a head)
        m' = max(f + m, i);   S <- exp(f + m - m') S + exp(i - m') k v^T;   n <- exp(f + m - m') n + exp(i - m') k
        o = S^T q / (max(|n . q|, exp(-m')) + den_eps)
        out = Wo [ o_h / rms(o_h) * norm_h * sigmoid(Wg x)_h ]_h                               (norm [heads * value_dim])

    S, n and m (all zero at the start) are the request's state, float32: [head][value channel][key channel] with n
    as one more value channel, then the heads' m."""

    ORDER = ("q", "k", "v", "g", "i", "f")

    def __init__(self, hidden_size: int, num_heads: int, head_dim: int, value_dim: int, gate_cap: float, norm_eps: float = 1e-6,
                 den_eps: float = 1e-6, external: bool = False, external_output: bool = False):
        super().__init__(hidden_size, num_heads, head_dim, value_dim, norm_eps, external, external_output)
        self.gate_cap = float(gate_cap)
        self.den_eps = float(den_eps)
        if not self.gate_cap > 0:
            raise ConfigError(f"matrix memory: the gates' cap {gate_cap} must be positive")
        self.i_bias = self.f_bias = None

    def _widths(self):
        return super()._widths() | {"i": self.num_heads, "f": self.num_heads}

    def state_spec(self):
        # (rows of whole 16 bytes)
        n = self.num_heads * (self.value_dim + 1) * self.head_dim + self.num_heads
        return StateSpec((-(-n // 4) * 4,), torch.float32)

    def weight_specs(self):
        W, H, N, V = self.hidden_size, self.num_heads, self.num_heads * self.head_dim, self.num_heads * self.value_dim
        return {"q": WeightSpec((N, W)), "k": WeightSpec((N, W)), "v": WeightSpec((V, W)), "g": WeightSpec((V, W)),
                "i": WeightSpec((H, W)), "i.b": WeightSpec((H,), "vector"), "f": WeightSpec((H, W)), "f.b": WeightSpec((H,), "vector"),
                "norm": WeightSpec((V,), "norm"), "o": WeightSpec((W, V))}

    def _load_vectors(self, weights, f32):
        self.i_bias, self.f_bias, self.norm = f32("i.b"), f32("f.b"), f32("norm")

    def _run(self, ctx, proj, out, out_scale):
        return ctx.ops.exp_gate_recurrence(proj, self._first_columns({"g": "gate", "i": "ig", "f": "fg"}), self.i_bias, self.f_bias,
                                           self.gate_cap, self.norm, self.norm_eps, ctx.state, ctx.batch, self.num_heads, self.head_dim,
                                           self.value_dim, out, out_scale, q_scale=self.head_dim ** -0.5, den_eps=self.den_eps)
