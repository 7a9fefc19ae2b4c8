"""A recurrent mixer with a matrix memory per head whose decay and write strength are one number a token (Mamba-2).

One projection gives, side by side, a gate ``z`` (``heads * vdim``), values ``x`` (as many), write keys ``B`` and read keys
``C`` (``groups`` heads of ``state`` elements each; memory head ``h`` uses group ``h // (heads / groups)``) and a step size
``dt`` per head.  ``x``, ``B`` and ``C`` pass a short causal convolution over time on every channel, with a bias (``y[t] =
b + sum_j w[:, j] u[t - taps + 1 + j]``, zeros before the sequence's start), and silu.  Then per head::

    d = softplus(dt + dt_bias);   S <- exp(-exp(A_log) d) S + d B x^T;   y = S^T C + D x       (S: state x vdim)

``y * silu(z)``, the heads side by side, is divided by the root mean square of each of ``norm_groups`` equal parts and
multiplied by a weight; ``W_o`` follows.  The memory is the request's state, float32, zero at the start, in two halves
(a step reads the half that the request's last committed step wrote and writes the other); the convolution's last
``taps - 1`` projected rows are state too, in the run dtype.  Step sizes, decays, the memory and its products, the
gated norm are float32 whatever the run dtype; the projections, the convolution and its activation are in the run
dtype.
"""
from __future__ import annotations

import torch

from .base import CacheNeed, Mixer, ParamSpec, register_mixer


@register_mixer("mamba2")
class Mamba2(Mixer):
    graph_safe = True

    def __init__(self, spec) -> None:
        super().__init__()
        self.hidden = int(spec.hidden_size)
        self.num_heads, self.value_dim = int(spec.num_heads), int(spec.value_dim)
        self.state_dim, self.num_groups = int(spec.state_dim), int(spec.get("num_groups") or 1)
        self.conv_taps = int(spec.conv_taps)
        self.norm_groups = int(spec.get("norm_groups") or 1)
        self.norm_eps = float(spec.norm_eps)
        if (min(self.num_heads, self.value_dim, self.state_dim, self.num_groups, self.conv_taps, self.norm_groups) < 1
                or self.num_heads % self.num_groups or self.inner % self.norm_groups):
            raise ValueError("mamba2 needs positive sizes, heads a multiple of groups, and heads * vdim of norm_groups")
        self.state_dtype = None
        self.conv_by_tap = None

    @property
    def inner(self) -> int:
        return self.num_heads * self.value_dim

    @property
    def channels(self) -> int:
        """The rows that pass the convolution: x, B, C."""
        return self.inner + 2 * self.num_groups * self.state_dim

    def param_specs(self):
        h, c, d = self.num_heads, self.channels, self.hidden
        return {
            "w_in": ParamSpec((self.inner + c + h, d), init=("normal", d ** -0.5)),  # rows: z, x, B, C, dt
            "conv": ParamSpec((c, self.conv_taps), policy="float32", init=("normal", 0.5)),
            "conv_bias": ParamSpec((c,), policy="float32", init=("normal", 0.3)),
            "dt_bias": ParamSpec((h,), policy="float32", init=("uniform", -4.0, 0.0)),
            "a_log": ParamSpec((h,), policy="float32", init=("uniform", -4.0, 1.0)),
            "skip": ParamSpec((h,), policy="float32", init=("uniform", 0.5, 1.5)),
            "norm": ParamSpec((self.inner,), policy="float32", init=("uniform", 0.5, 1.5)),
            "wo": ParamSpec((d, self.inner), init=("normal", self.inner ** -0.5)),
        }

    def allocate(self, dtype, device) -> None:
        super().allocate(dtype, device)
        self.state_dtype = dtype

    def finalize(self) -> None:
        self.conv_by_tap = self.params["conv"].t().contiguous()

    def cache_need(self) -> CacheNeed:
        states = [("memory", (2, self.num_heads, self.value_dim, self.state_dim), torch.float32)]  # (S transposed)
        if self.conv_taps > 1:
            states.append(("conv", (2, self.conv_taps - 1, self.channels), self.state_dtype))
        return CacheNeed(states=tuple(states))

    def mixing_flops(self, start: int, count: int) -> float:
        """Per token and head: the memory's update and its product with the read key."""
        return 4.0 * self.num_heads * self.state_dim * self.value_dim * count

    def forward(self, h: torch.Tensor, ctx, cache) -> torch.Tensor:
        ops, P = ctx.ops, self.params
        proj = ops.linear(h, P["w_in"])
        rows = ops.conv_rows(proj[:, self.inner: self.inner + self.channels], None, self.conv_by_tap, self.conv_taps,
                             cache.states.get("conv"), ctx, activation="silu", conv_bias=P["conv_bias"])
        o = ops.mamba2(proj, rows, P["dt_bias"], P["a_log"], P["skip"], P["norm"], self.num_heads, self.value_dim,
                       self.state_dim, self.num_groups, self.norm_groups, self.norm_eps, cache.states["memory"], ctx)
        return ops.linear(o, P["wo"])
