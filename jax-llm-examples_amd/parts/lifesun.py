"""The Lifesun decoder as an architecture: its configuration, its plan and the names of its checkpoint tensors.

The model's ends: ``embed``, ``final.norm`` (and ``.b``), ``head``; ``loop.in`` (``[width, 2 width]``) in front of
every pass of the looped layers.  A layer ``i`` stores, under ``l<i>.``: its norm ``norm1`` (and ``.b``), the mixers'
tensors under ``mix.left.`` and ``mix.right.`` and the feed-forward's under ``mlp.`` (``gate``, ``up``, ``down``).
Attentions: ``q``, ``k``, ``v``, ``o``; in a ``parallel`` layer the head gates ``g``; in a ``parallel_2`` layer the
weights ``q.norm``, ``k.norm`` over the projections.  Gated recurrent unit: ``y``, ``x`` with biases (``.b``),
``conv`` (``[channels, taps]``) and ``conv.b``, the gates' block matrices ``ra``, ``ri`` (``[blocks, out, in]``) and
biases, ``lam``, ``o``.  Retention: ``q``, ``k``, ``v``, the output gate ``g``, ``o``.  Linear weights are
``[out, in]``.
"""
from __future__ import annotations

import math
from typing import Any, Mapping

from ..config.lifesun import LifesunConfig
from ..config.registry import register_architecture
from ..config.specs import ModelPlan
from ..weights.bindings import TensorBinding


class LifesunArchitecture:
    names = ("Lifesun", "lifesun")
    # what of csrc/ a model of this design calls (a first run on a machine without a built library compiles these)
    kernel_sources = ("elementwise.hip", "parallel.hip", "terms.hip", "retention.hip", "gated_unit.hip",
                      "attention_heads.hip", "attention_conv.hip", "attention_span.hip", "attention_generic.hip",
                      "attention_mfma.hip", "attention_f32.hip", "gemm_skinny.hip", "gemm_stream.hip",
                      "gemm_grouped.hip", "gemm_generic.hip", "sampling.hip")

    def parse_config(self, top: Mapping[str, Any]) -> LifesunConfig:
        return LifesunConfig.from_dict(top)

    def plan(self, cfg: LifesunConfig) -> ModelPlan:
        return cfg.plan()

    def config_to_dict(self, cfg: LifesunConfig, architecture: str | None = None) -> dict:
        return cfg.to_dict(architecture or "Lifesun")

    def bindings(self, cfg: LifesunConfig, plan: ModelPlan) -> list[TensorBinding]:
        D, V = cfg.width, cfg.vocab
        mat = lambda fan_in: ("normal", 1.0 / math.sqrt(fan_in))
        weight, bias = ("uniform", 0.5, 1.5), ("normal", 0.2)
        norm = lambda name, target: [TensorBinding(name, (D,), target + ".weight", init=weight),
                                     TensorBinding(name + ".b", (D,), target + ".bias", init=bias)]

        def stacked(p, pieces, target):
            """Matrices stored apart that land one behind the other in ``target``."""
            out, o = [], 0
            for name, rows in pieces:
                out.append(TensorBinding(p + name, (rows, D), target, rows=(o, o + rows), init=mat(D)))
                o += rows
            return out

        out = [TensorBinding("embed", (V, D), "embed.weight", init=("normal", 1.0))]
        if cfg.loop is not None:
            out.append(TensorBinding("loop.in", (D, 2 * D), "loop.weight", init=mat(2 * D)))
        for i, lc in enumerate(cfg.layers):
            p, t = f"l{i}.", f"layers.{i}."
            out += norm(p + "norm1", t + "mixer_norm")
            a, b = lc.mixer.left, lc.mixer.right
            x, tm = p + "mix.left.", t + "mixer.left."
            heads = [("q", a.heads * a.dim), ("k", a.kv_heads * a.dim), ("v", a.kv_heads * a.vdim)]
            out += stacked(x, heads + ([("g", a.heads)] if lc.type == "parallel" else []), tm + "wqkv")
            if lc.type == "parallel_2":
                out += [TensorBinding(x + "q.norm", (a.heads * a.dim,), tm + "q_norm", init=weight),
                        TensorBinding(x + "k.norm", (a.kv_heads * a.dim,), tm + "k_norm", init=weight)]
            out.append(TensorBinding(x + "o", (D, a.heads * a.vdim), tm + "wo", init=mat(a.heads * a.vdim)))
            x, tm = p + "mix.right.", t + "mixer.right."
            out += getattr(self, "_" + lc.type + "_right")(b, D, x, tm, mat, stacked)
            if lc.mlp is not None:
                F = lc.mlp.ff
                out += stacked(p, (("mlp.gate", F), ("mlp.up", F)), t + "feed_forward.w_gate_up")
                out.append(TensorBinding(p + "mlp.down", (D, F), t + "feed_forward.w_down", init=mat(F)))
        return out + norm("final.norm", "final_norm") + [TensorBinding("head", (V, D), "lm_head.weight", init=mat(D))]

    @staticmethod
    def _parallel_right(m, D, x, t, mat, stacked) -> list[TensorBinding]:
        W, n = m.width, m.blocks
        s = W // n
        out = stacked(x, (("x", W), ("y", W)), t + "w_in")
        out += [TensorBinding(x + "x.b", (W,), t + "b_x", init=("normal", 0.2)),
                TensorBinding(x + "y.b", (W,), t + "b_y", init=("normal", 0.2)),
                TensorBinding(x + "conv", (W, m.conv), t + "conv", init=("normal", 0.5)),
                TensorBinding(x + "conv.b", (W,), t + "conv_bias", init=("normal", 0.2))]
        for name in ("ra", "ri"):
            out += [TensorBinding(x + name, (n, s, s), t + "w_" + name, init=mat(s)),
                    TensorBinding(x + name + ".b", (n, s), t + "b_" + name, init=("normal", 0.3))]
        return out + [TensorBinding(x + "lam", (W,), t + "lam", init=("uniform", -7.0, 0.0)),
                      TensorBinding(x + "o", (D, W), t + "wo", init=mat(W))]

    @staticmethod
    def _parallel_2_right(m, D, x, t, mat, stacked) -> list[TensorBinding]:
        H = m.heads
        return stacked(x, (("q", H * m.dim), ("k", H * m.dim), ("v", H * m.vdim), ("g", H * m.vdim)), t + "w_in") + [
            TensorBinding(x + "o", (D, H * m.vdim), t + "wo", init=mat(H * m.vdim))]


LIFESUN = register_architecture(LifesunArchitecture())
