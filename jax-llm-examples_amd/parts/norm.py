"""RMS norm (``llama4/llama4_jax/model.py:885-888``): ``x / sqrt(mean(x^2) + eps) * weight``,
statistics in float32, eps inside the root, the weight used as it is (not ``1 + weight``).  With the option
``unit_offset`` the checkpoint stores the weight as its distance from one: the part adds the one when the weights
are in place (in float32, as a kernel that formed ``1 + weight`` would), and the kernels see a plain weight.  With
the option ``one_number`` the weight is a single number for all elements of a row: the checkpoint's tensor has no
axis, and the kernels see it told for every element.

Layer norm (``layernorm``): ``(x - mean) / sqrt(variance + eps) * weight + bias``, the variance the mean of the squared
deviations, float32."""
from __future__ import annotations

from .base import Norm, ParamSpec, register_norm


@register_norm("rmsnorm")
class RMSNorm(Norm):
    def __init__(self, spec) -> None:
        super().__init__()
        self.eps = float(spec.eps)
        self.weighted = bool(spec.get("weighted", True))
        self.size = spec.get("size")
        self.unit_offset = bool(spec.get("unit_offset", False))
        self._offset_added = False
        self.one_number = bool(spec.get("one_number", False))
        self._told = None
        if self.one_number and (self.unit_offset or not self.weighted):
            raise ValueError("a norm's one number is its plain weight")

    graph_safe = True

    def param_specs(self):
        if not self.weighted:
            return {}
        if self.one_number:
            return {"weight": ParamSpec((), policy="float32", init=("ones",))}
        init = ("normal", 0.1) if self.unit_offset else ("ones",)
        return {"weight": ParamSpec((int(self.size),), policy="float32", init=init)}

    def finalize(self) -> None:
        if self.unit_offset and self.weighted and not self._offset_added:
            self.params["weight"].add_(1.0)
            self._offset_added = True
        if self.one_number:
            self._told = self.params["weight"].expand(int(self.size)).contiguous()

    def forward(self, residual, ctx, want32: bool = False, defer: bool = False):
        return residual.normed(ctx, self._told if self.one_number else self.params.get("weight"), self.eps, want32, defer)


@register_norm("layernorm")
class LayerNorm(Norm):
    graph_safe = True

    def __init__(self, spec) -> None:
        super().__init__()
        self.eps, self.size = float(spec.eps), int(spec.size)

    def param_specs(self):
        return {"weight": ParamSpec((self.size,), policy="float32", init=("ones",)),
                "bias": ParamSpec((self.size,), policy="float32", init=("normal", 0.1))}

    def flops_per_token(self) -> float:
        return 0.0

    def forward(self, residual, ctx, want32: bool = False, defer: bool = False):
        return residual.layer_normed(ctx, self.params["weight"], self.params["bias"], self.eps, want32)
