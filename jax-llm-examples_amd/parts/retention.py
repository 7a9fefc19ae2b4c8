"""Retention: linear attention with a fixed decay per head, no softmax and no denominator.

``q = W_q h``, ``k = W_k h`` (``heads`` of ``dk`` elements), ``v = W_v h`` (``heads`` of ``dv``), q and k turned by the
position encoding, k then divided by ``sqrt(dk)``.  Per head::

    S <- decay S + k v^T;   o = S^T q             (S: dk x dv, zero at the start)

so the read-out sees the token's own write.  Every head's ``o`` is divided by its root mean square (no weight), the
heads side by side are multiplied by ``silu(W_g h)``, and ``W_o`` follows.  The memory is the request's state, float32,
in two halves (a step reads the half that the request's last committed step wrote and writes the other).  The turned
queries and keys, the memory and its products and the norm are float32 whatever the run dtype; the projections are in
the run dtype.
"""
from __future__ import annotations

import torch

from .base import CacheNeed, Mixer, ParamSpec, build_position, register_mixer


@register_mixer("retention")
class Retention(Mixer):
    graph_safe = True

    def __init__(self, spec) -> None:
        super().__init__()
        self.hidden = int(spec.hidden_size)
        self.num_heads, self.head_dim = int(spec.num_heads), int(spec.head_dim)
        self.value_dim = int(spec.get("value_dim") or self.head_dim)
        self.norm_eps = float(spec.norm_eps)
        self.decay = tuple(float(g) for g in spec.decay)
        self.position = build_position(spec.position, self.head_dim)
        if min(self.num_heads, self.head_dim, self.value_dim) < 1 or len(self.decay) != self.num_heads:
            raise ValueError("retention needs positive sizes and a decay for every head")
        if not all(0.0 <= g <= 1.0 for g in self.decay):
            raise ValueError("retention's decays lie between 0 and 1")
        self.decays = None  # [2, heads] float32: the decays and their base-2 logarithms
        self.rotation = None

    def param_specs(self):
        h, dk, dv, d = self.num_heads, self.head_dim, self.value_dim, self.hidden
        return {
            # rows: q heads, k heads, v heads, output gate; each [out, in]
            "w_in": ParamSpec((2 * h * dk + 2 * h * dv, d), init=("normal", d ** -0.5)),
            "wo": ParamSpec((d, h * dv), init=("normal", (h * dv) ** -0.5)),
        }

    def finalize(self) -> None:
        dev = self.params["w_in"].device
        g = torch.tensor(self.decay, dtype=torch.float32)
        # (a decay of zero: a power so negative that every product with it but the zeroth vanishes)
        self.decays = torch.stack([g, torch.log2(g.double()).clamp_min(-1e6).float()]).contiguous().to(dev)
        self.rotation = self.position.rotation()
        if self.rotation is not None:
            self.rotation.inv_freq = self.rotation.inv_freq.to(dev)

    def cache_need(self) -> CacheNeed:
        return CacheNeed(states=(("memory", (2, self.num_heads, self.value_dim, self.head_dim), torch.float32),))  # (S transposed)

    def mixing_flops(self, start: int, count: int) -> float:
        """Per token and head: the memory's update and its product with the query."""
        return 4.0 * self.num_heads * self.head_dim * self.value_dim * count

    def forward(self, h: torch.Tensor, ctx, cache) -> torch.Tensor:
        ops = ctx.ops
        rows = ops.linear(h, self.params["w_in"])
        o = ops.retention(rows, self.num_heads, self.head_dim, self.value_dim, self.rotation, self.decays, self.norm_eps,
                          cache.states["memory"], ctx)
        return ops.linear(o, self.params["wo"])
