"""A recurrent mixer with one number of memory per channel (the real-gated linear recurrent unit of Griffin's recurrent
block).

Two branches of ``width`` channels: ``y = gelu_tanh(W_y h + b_y)`` and ``u = conv(W_x h + b_x) + b_c``, a short causal
convolution over time on every channel (``sum_j w[:, j] v[t - taps + 1 + j]``, zeros before the sequence's start).
``u`` is cut into ``blocks`` equal parts; a part's gates are products with its own square matrices::

    r = sigmoid(A_b u_b + a_b);   i = sigmoid(B_b u_b + b_b);   log a = -rate * r * softplus(lam)
    S <- a S + sqrt(1 - a^2) i u;      output  W_o (S y)

``S`` is the request's state, float32, zero at the start, in two halves (a step reads the half that the request's last
committed step wrote and writes the other); the convolution's last ``taps - 1`` input rows are state too, in the run
dtype.  The gates (products with float32 sums, kept in float32), the decays, ``S`` and its product with ``y`` are
float32 whatever the run dtype; the projections and the convolution are in the run dtype.
"""
from __future__ import annotations

import torch

from .base import CacheNeed, Mixer, ParamSpec, register_mixer


@register_mixer("gated_unit")
class GatedUnit(Mixer):
    graph_safe = True

    def __init__(self, spec) -> None:
        super().__init__()
        self.hidden, self.width = int(spec.hidden_size), int(spec.width)
        self.blocks, self.conv_taps = int(spec.blocks), int(spec.conv_taps)
        self.decay_rate = float(spec.decay_rate)
        if min(self.width, self.blocks, self.conv_taps) < 1 or self.width % self.blocks or self.decay_rate <= 0:
            raise ValueError("the gated unit needs a width of equal blocks, a convolution and a positive decay rate")
        self.state_dtype = None
        self.conv_by_tap = None

    def param_specs(self):
        w, n, d = self.width, self.blocks, self.hidden
        s = w // n
        vec = lambda std: ParamSpec((w,), policy="float32", init=("normal", std))
        return {
            "w_in": ParamSpec((2 * w, d), init=("normal", d ** -0.5)),  # rows: x (the recurrence's branch), y
            "b_x": vec(0.2), "b_y": vec(0.2),
            "conv": ParamSpec((w, self.conv_taps), policy="float32", init=("normal", 0.5)),
            "conv_bias": vec(0.2),
            "w_ra": ParamSpec((n, s, s), init=("normal", s ** -0.5)),  # per block [out, in]
            "w_ri": ParamSpec((n, s, s), init=("normal", s ** -0.5)),
            "b_ra": ParamSpec((n, s), policy="float32", init=("normal", 0.3)),
            "b_ri": ParamSpec((n, s), policy="float32", init=("normal", 0.3)),
            "lam": ParamSpec((w,), policy="float32", init=("uniform", -7.0, 0.0)),
            "wo": ParamSpec((d, w), init=("normal", w ** -0.5)),
        }

    def allocate(self, dtype, device) -> None:
        super().allocate(dtype, device)
        self.state_dtype = dtype

    def finalize(self) -> None:
        self.conv_by_tap = self.params["conv"].t().contiguous()

    def cache_need(self) -> CacheNeed:
        states = [("memory", (2, self.width), torch.float32)]
        if self.conv_taps > 1:
            states.append(("conv", (2, self.conv_taps - 1, self.width), self.state_dtype))
        return CacheNeed(states=tuple(states))

    def mixing_flops(self, start: int, count: int) -> float:
        """Per token and channel: the memory's update and its product with the other branch."""
        return 4.0 * self.width * count

    def forward(self, h: torch.Tensor, ctx, cache) -> torch.Tensor:
        ops, P = ctx.ops, self.params
        proj = ops.linear(h, P["w_in"])
        u = ops.conv_rows(proj[:, : self.width], P["b_x"], self.conv_by_tap, self.conv_taps, cache.states.get("conv"), ctx,
                          conv_bias=P["conv_bias"])
        o = ops.gated_unit(u, proj[:, self.width:], P["b_y"], P["w_ra"], P["b_ra"], P["w_ri"], P["b_ri"], P["lam"],
                           self.decay_rate, cache.states["memory"], ctx)
        return ops.linear(o, P["wo"])
