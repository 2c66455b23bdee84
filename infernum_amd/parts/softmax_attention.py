"""Softmax attention between two plain products, with what designs vary about it as parameters.

q = Wq x, k = Wk x, v = Wv x without biases, query head h over key/value head h // (nh / nkv), key heads of ``head_dim``
and value heads of ``value_dim`` values.  In the order in which they act:

* ``values="keys"``: there is no Wv; a value head is its key head as the projection leaves it.
* ``value_mix``: v <- (1 - lambda) v + lambda v1 with v1 the same token's values in the first layer that takes part
  ("first": this layer is the one, its values stay as they are and later layers of the step read them; "mixed": a later
  one, with a learned number lambda).  What is kept in the pages is the mixed v.
* ``qk_norm``: every query and key head divided by its root mean square, times a weight that the heads share.
* rotation by the position encoding (either pairing), score times ``scale``, then ``softcap`` c: s <- c tanh(s / c).
* mask: every earlier key, or a ``window`` of them and with ``keep_first`` also the request's first positions (whose
  pages never go back to the pool while the request lives).
* ``sink``: the softmax's denominator also holds exp(sink_h): "learned" (a number per head), "zero" (one is added).

The projection's rows become queries, pages' keys and pages' values in one kernel (``kernels.api.qk_prepare``), then the
attention kernels of every mixer here do the rest.
"""
from __future__ import annotations

from typing import Any, Dict, Mapping, Optional, Sequence

import torch

from ..kernels import api as K
from .attention import Attention
from .base import CacheView, Runtime, StepContext, WeightSpec, register_part
from .projected import ProjectedMixer

FIRST_VALUES = "value_mix.first"         # in ctx.extras: the first mixing layer's values [N, nkv dv]


class SoftmaxAttention(ProjectedMixer, Attention):
    graph_safe = True

    def __init__(self, rt: Runtime, hidden_size: int, num_heads: int, num_kv_heads: int, head_dim: int, value_dim: int,
                 scale: float, position: Optional[Mapping[str, Any]] = None, window: Optional[int] = None,
                 keep_first: int = 0, softcap: Optional[float] = None, sink: Optional[str] = None, qk_norm: bool = False,
                 norm_eps: float = 1e-6, values: str = "projected", value_mix: Optional[str] = None, init_std: float = 0.02,
                 names: Sequence[str] = ("q", "k", "v", "o"), kernels: str = "auto"):
        Attention.__init__(self, rt, hidden_size, num_heads, num_kv_heads, head_dim, position=position, window=window,
                           scale=scale, kernels=kernels, init_std=init_std, value_dim=value_dim, keep_first=keep_first,
                           softcap=softcap)
        if sink not in (None, "learned", "zero") or values not in ("projected", "keys") \
                or value_mix not in (None, "first", "mixed"):
            raise ValueError(f"softmax_attention: sink {sink!r}, values {values!r}, value_mix {value_mix!r}")
        if values == "keys" and self.vd != self.d:
            raise ValueError(f"values that are the keys have their size, {self.d}, not {self.vd}")
        if not self.scale > 0:
            raise ValueError("the scale of the scores must be positive")
        self.sink, self.qk_norm, self.norm_eps = sink, bool(qk_norm), float(norm_eps)
        self.values_are_keys, self.value_mix, self.names = values == "keys", value_mix, tuple(names)
        self.v_col = self.nh * self.d if self.values_are_keys else (self.nh + self.nkv) * self.d
        self.out_cols = self.nh * self.vd
        self.q_norm = self.k_norm = None
        self.mix_lambda = 0.0
        self.graph_safe = getattr(self.position, "graph_safe", False)

    # ---- tensors -----------------------------------------------------------------------------
    def weights(self) -> Dict[str, WeightSpec]:
        nh, nkv, d, dv, H, small = self.nh, self.nkv, self.d, self.vd, self.hidden_size, dict(follows_compute_dtype=False)
        q, k, v, o = self.names
        init = ("normal", self.init_std)
        out = {q: WeightSpec((nh * d, H), init), k: WeightSpec((nkv * d, H), init)}
        if not self.values_are_keys:
            out[v] = WeightSpec((nkv * dv, H), init)
        out[o] = WeightSpec((H, nh * dv), init)
        if self.qk_norm:
            out[q + ".norm"] = WeightSpec((d,), ("uniform", 0.8, 1.2), **small)
            out[k + ".norm"] = WeightSpec((d,), ("uniform", 0.8, 1.2), **small)
        if self.sink == "learned":
            out["sink"] = WeightSpec((nh,), ("normal", 1.0), **small)
        if self.value_mix == "mixed":
            out["vmix"] = WeightSpec((), ("uniform", 0.2, 0.8), **small)
        return out

    def stack_rows(self, tensors) -> Sequence[torch.Tensor]:
        q, k, v, _ = self.names
        return [tensors[q], tensors[k]] + ([] if self.values_are_keys else [tensors[v]])

    def output_matrix(self, tensors) -> torch.Tensor:
        return tensors[self.names[3]]

    def load_small(self, tensors) -> None:
        q, k, _, _ = self.names
        f32 = lambda name: tensors[name].to(torch.float32).contiguous()            # noqa: E731
        if self.qk_norm:
            self.q_norm, self.k_norm = f32(q + ".norm"), f32(k + ".norm")
        if self.sink == "learned":
            self.sinks = f32("sink")
        elif self.sink == "zero":
            self.sinks = torch.zeros(self.nh, dtype=torch.float32, device=self.rt.device)
        if self.value_mix == "mixed":
            self.mix_lambda = float(tensors["vmix"].to(torch.float32))

    def load(self, tensors) -> None:
        ProjectedMixer.load(self, tensors)

    def forward(self, x, ctx, cache):
        return ProjectedMixer.forward(self, x, ctx, cache)

    def _forward_is_own(self) -> bool:
        return type(self).forward is SoftmaxAttention.forward and type(self).attend is Attention.attend

    def native(self, program, view) -> None:
        ProjectedMixer.native(self, program, view)

    def rows_key(self) -> str:
        return "value_mix.rows" if self.value_mix == "first" else "projected.rows"

    # ---- one step ----------------------------------------------------------------------------
    def _pages(self, cache: CacheView):
        if cache is None or cache.k_pages is None or cache.v_pages is None or not cache.writable:
            raise K.KernelError("softmax_attention needs pages of its own")
        return cache.k_pages, cache.v_pages

    def mix(self, proj: torch.Tensor, ctx: StepContext, cache: CacheView, out: torch.Tensor) -> None:
        nh, nkv, d, dv, pos = self.nh, self.nkv, self.d, self.vd, self.position
        kp, vp = self._pages(cache)
        n = proj.shape[0]
        first = None
        if self.value_mix == "first":
            ctx.extras[FIRST_VALUES] = proj[:, self.v_col:self.v_col + nkv * dv]
        elif self.value_mix == "mixed":
            first = ctx.extras.get(FIRST_VALUES)
            if first is None or first.shape[1] != nkv * dv:
                raise K.KernelError("softmax_attention: no earlier layer left values of this size to mix with")
        q = torch.empty((n, nh * d), dtype=proj.dtype, device=proj.device)
        K.qk_prepare(proj, q, nh, nkv, d, ctx.positions, self.q_norm, self.k_norm, self.norm_eps, pos.inv_freq,
                     pos.rotary_dim if pos.inv_freq is not None else 0, pos.pairing, pos.magnitude, ctx.slots[cache.group],
                     kp, vp, values_are_keys=self.values_are_keys, v_scale=self.result_scale, v_first=first,
                     v_lambda=self.mix_lambda)
        self.attend(q, out, ctx, cache)

    def emit_mix(self, program, view: CacheView, proj, proj_row: int, out, out_row: int) -> None:
        from ..engine.program import ALWAYS, STREAM
        nh, nkv, d, dv, pos = self.nh, self.nkv, self.d, self.vd, self.position
        kp, vp = self._pages(view)
        act, ab = program.act_code, program.act_bytes
        program.keep(self.q_norm, self.k_norm, pos.inv_freq, kp, vp)
        first, first_row = None, 0
        if self.value_mix == "first":
            program.value_mix_first = (_at(proj, self.v_col * ab), proj_row, nkv * dv)
        elif self.value_mix == "mixed":
            kept = getattr(program, "value_mix_first", None)
            if kept is None or kept[2] != nkv * dv:
                raise K.KernelError("softmax_attention: no earlier layer left values of this size to mix with")
            first, first_row = kept[0], kept[1]
        q = program.buffer("attention.q", program.T * nh * d * ab)
        rot = pos.rotary_dim if pos.inv_freq is not None else 0
        program.op("core", "ia_qk_prepare",
                   [proj, act, proj_row, q, nh * d, self.q_norm, self.k_norm, float(self.norm_eps), program.positions,
                    program.slots(view.group), pos.inv_freq if rot else None,
                    int(bool(rot) and pos.inv_freq.dtype == torch.float64), rot, K.PAIRINGS[pos.pairing],
                    float(pos.magnitude), kp, vp, program.N, nh, nkv, d, dv, int(kp.shape[2]), int(kp.shape[0]),
                    int(self.values_are_keys), float(self.result_scale), first, first_row, float(self.mix_lambda), STREAM])
        self.emit_attend(program, view, q, nh * d, ALWAYS, out, out_row)


def _at(where, nbytes: int):
    """The place ``nbytes`` behind an address of the program (a Buffer, or a place inside one)."""
    from ..engine.program import Buffer
    return where.at(nbytes) if isinstance(where, Buffer) else where.buffer.at(where.nbytes + nbytes)


register_part("mixer", "softmax_attention", SoftmaxAttention)
