"""The Folivik decoder as an architecture: its configuration, its plan and the names of its checkpoint tensors.

The model's ends: ``embed``, ``final.norm``, ``head``.  A layer ``i`` stores, under ``l<i>.``: its two norms (``norm1``
for the mixer, ``norm2`` for the feed-forward; one number each), the mixer's tensors under ``mix.`` and the
feed-forward's under ``mlp.``.  Mixer ``latent_attention``: the queries' way down and up ``dq``, ``dq.norm``, ``uq``
(rows head by head, a head's unrotated elements before its rotated ones), the shared latent ``dkv`` (latent rows,
then the rotated key's), ``dkv.norm``, ``uk``, ``uv``, the head gates ``g`` and ``o``.  Mixer ``attention``: ``q``,
``k``, ``v``, the q/k norms' weights ``q.norm``, ``k.norm`` (over a head's elements, shared by heads), one number per
head ``temp``, ``r1``, ``r2``, and ``o``.  Mixer ``mamba2``: ``in`` (gate, values, write keys, read keys, step sizes,
in this order), ``conv`` (``[channels, taps]``) and ``conv.b``, one number per head ``dt_bias``, ``A_log``, ``D``, the
output norm's weight ``norm`` and ``o``.  Feed-forward: ``router``, ``correction``, the experts
``e<j>.gate|up|down`` and the shared expert ``shared.gate|up|down``.  Linear weights are ``[out, in]``.
"""
from __future__ import annotations

import math
from typing import Any, Mapping

from ..config.folivik import FolivikConfig
from ..config.registry import register_architecture
from ..config.specs import ModelPlan
from ..weights.bindings import TensorBinding


class FolivikArchitecture:
    names = ("Folivik", "folivik")
    # what of csrc/ a model of this design calls (a first run on a machine without a built library compiles these)
    kernel_sources = ("elementwise.hip", "mamba2.hip", "attention_latent.hip", "attention_heads.hip", "attention_conv.hip",
                      "attention_generic.hip", "attention_mfma.hip", "attention_f32.hip", "attention_prep.hip",
                      "moe_route.hip", "moe_choose.hip", "gemm_skinny.hip", "gemm_stream.hip", "gemm_grouped.hip",
                      "gemm_generic.hip", "gemm_f32.hip", "parallel.hip", "sampling.hip")

    def parse_config(self, top: Mapping[str, Any]) -> FolivikConfig:
        return FolivikConfig.from_dict(top)

    def plan(self, cfg: FolivikConfig) -> ModelPlan:
        return cfg.plan()

    def config_to_dict(self, cfg: FolivikConfig, architecture: str | None = None) -> dict:
        return cfg.to_dict(architecture or "Folivik")

    def unused_prefixes(self, cfg: FolivikConfig) -> tuple:
        """Tensors that a checkpoint may hold and this model does not read: the feed-forward's norm of a layer that
        has no feed-forward."""
        return tuple(f"l{i}.norm2" for i, lc in enumerate(cfg.layers) if lc.mlp is None)

    def bindings(self, cfg: FolivikConfig, plan: ModelPlan) -> list[TensorBinding]:
        D, V = cfg.width, cfg.vocab
        mat = lambda fan_in: ("normal", 1.0 / math.sqrt(fan_in))
        norm = ("uniform", 0.5, 1.5)
        out = [TensorBinding("embed", (V, D), "embed.weight", init=("normal", 1.0))]
        for i, lc in enumerate(cfg.layers):
            p, t = f"l{i}.", f"layers.{i}."
            out.append(TensorBinding(p + "norm1", (), t + "mixer_norm.weight", init=norm))
            out += getattr(self, "_" + lc.type)(lc.mixer, D, p + "mix.", t + "mixer.", mat, norm)
            if lc.mlp is not None:
                out.append(TensorBinding(p + "norm2", (), t + "feed_forward_norm.weight", init=norm))
                out += self._experts(lc.mlp, D, p + "mlp.", t + "feed_forward.", mat)
        return out + [TensorBinding("final.norm", (), "final_norm.weight", init=norm),
                      TensorBinding("head", (V, D), "lm_head.weight", init=mat(D))]

    @staticmethod
    def _stacked(pieces, D: int, target: str, mat) -> list[TensorBinding]:
        """Matrices stored apart that land one behind the other in ``target``."""
        out, o = [], 0
        for name, rows in pieces:
            out.append(TensorBinding(name, (rows, D), target, rows=(o, o + rows), init=mat(D)))
            o += rows
        return out

    def _latent_attention(self, m, D, x, t, mat, norm) -> list[TensorBinding]:
        return self._stacked(((x + "dq", m.q_rank), (x + "dkv", m.kv_rank + m.rot_dim), (x + "g", m.heads)), D,
                             t + "w_in", mat) + [
            TensorBinding(x + "dq.norm", (m.q_rank,), t + "query_norm", init=norm),
            TensorBinding(x + "uq", (m.heads * (m.dim + m.rot_dim), m.q_rank), t + "w_uq", init=mat(m.q_rank)),
            TensorBinding(x + "dkv.norm", (m.kv_rank,), t + "latent_norm", init=norm),
            TensorBinding(x + "uk", (m.heads * m.dim, m.kv_rank), t + "w_uk", init=mat(m.kv_rank)),
            TensorBinding(x + "uv", (m.heads * m.vdim, m.kv_rank), t + "w_uv", init=mat(m.kv_rank)),
            TensorBinding(x + "o", (D, m.heads * m.vdim), t + "wo", init=mat(m.heads * m.vdim))]

    def _attention(self, m, D, x, t, mat, norm) -> list[TensorBinding]:
        return self._stacked(((x + "q", m.heads * m.dim), (x + "k", m.kv_heads * m.dim), (x + "v", m.kv_heads * m.vdim)),
                             D, t + "wqkv", mat) + [
            TensorBinding(x + "q.norm", (m.dim,), t + "q_norm", init=norm),
            TensorBinding(x + "k.norm", (m.dim,), t + "k_norm", init=norm),
            TensorBinding(x + "temp", (m.heads,), t + "head_temp", init=norm),
            TensorBinding(x + "r1", (m.heads,), t + "dist_mul", init=("uniform", 0.0, 2.0)),
            TensorBinding(x + "r2", (m.heads,), t + "dist_rate", init=("uniform", 0.05, 0.5)),
            TensorBinding(x + "o", (D, m.heads * m.vdim), t + "wo", init=mat(m.heads * m.vdim))]

    def _mamba2(self, m, D, x, t, mat, norm) -> list[TensorBinding]:
        return [TensorBinding(x + "in", (m.inner + m.channels + m.heads, D), t + "w_in", init=mat(D)),
                TensorBinding(x + "conv", (m.channels, m.conv), t + "conv", init=("normal", 0.5)),
                TensorBinding(x + "conv.b", (m.channels,), t + "conv_bias", init=("normal", 0.3)),
                TensorBinding(x + "dt_bias", (m.heads,), t + "dt_bias", init=("uniform", -4.0, 0.0)),
                TensorBinding(x + "A_log", (m.heads,), t + "a_log", init=("uniform", -4.0, 1.0)),
                TensorBinding(x + "D", (m.heads,), t + "skip", init=norm),
                TensorBinding(x + "norm", (m.inner,), t + "norm", init=norm),
                TensorBinding(x + "o", (D, m.inner), t + "wo", init=mat(m.inner))]

    def _experts(self, m, D, x, t, mat) -> list[TensorBinding]:
        F = m.ff
        out = [TensorBinding(x + "router", (m.outputs, D), t + "router", init=mat(D)),
               TensorBinding(x + "correction", (m.outputs,), t + "correction", init=("normal", 0.1))]
        for e in range(m.experts):
            out += [TensorBinding(x + f"e{e}.gate", (F, D), t + "w_gate_up", index=e, rows=(0, F), init=mat(D)),
                    TensorBinding(x + f"e{e}.up", (F, D), t + "w_gate_up", index=e, rows=(F, 2 * F), init=mat(D)),
                    TensorBinding(x + f"e{e}.down", (D, F), t + "w_down", index=e, init=mat(F))]
        if m.shared_ff is not None:
            S = m.shared_ff
            out += [TensorBinding(x + "shared.gate", (S, D), t + "shared_gate_up", rows=(0, S), init=mat(D)),
                    TensorBinding(x + "shared.up", (S, D), t + "shared_gate_up", rows=(S, 2 * S), init=mat(D)),
                    TensorBinding(x + "shared.down", (D, S), t + "shared_down", init=mat(S))]
        return out


FOLIVIK = register_architecture(FolivikArchitecture())
