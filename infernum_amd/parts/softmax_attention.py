"""Softmax attention between two plain products, with what designs vary about it as parameters.

q = Wq x, k = Wk x, v = Wv x without biases, query head h over key/value head h // (nh / nkv), key heads of ``head_dim``
and value heads of ``value_dim`` values.  In the order in which they act:

* ``values="keys"``: there is no Wv; a value head is its key head as the projection leaves it.
* ``value_mix``: v <- (1 - lambda) v + lambda v1 with v1 the same token's values in the first layer that takes part
  ("first": this layer is the one, its values stay as they are and later layers of the step read them; "mixed": a later
  one, with a learned number lambda).  What is kept in the pages is the mixed v.
* ``qk_norm``: every query and key head divided by its root mean square, times a weight that the heads share; ``"rows"``:
  all of a token's queries (and all of its keys) at once, times a weight for every value of every head.
* rotation by the position encoding (either pairing), score times ``scale``, then ``softcap`` c: s <- c tanh(s / c).
* ``distance_bias`` {far, rows}: a learned number by head and distance n = i - j, added to the score: row bucket(n) of a
  table [B, heads].  With h = B / 2 the first h distances have a row each; from there on the rows' distances grow
  geometrically, bucket(n) = min(B - 1, h + floor((B - h) ln(n / h) / ln(far / h))).
* mask: every earlier key, or a ``window`` of them and with ``keep_first`` also the request's first positions (whose
  pages never go back to the pool while the request lives).
* ``sink``: the softmax's denominator also holds exp(sink_h): "learned" (a number per head), "zero" (one is added).

* ``output_gate``: the heads' results, value by value, times sigmoid(Wg x).

The projection's rows become queries, pages' keys and pages' values in one kernel (``kernels.api.qk_prepare`` or ``qk_rows_prepare``), then the
attention kernels of every mixer here do the rest.
"""
from __future__ import annotations

from fractions import Fraction
from typing import Any, Dict, List, Mapping, Optional, Sequence, Union

import torch

from ..kernels import api as K
from .attention import Attention
from .base import CacheView, Runtime, StepContext, WeightSpec, register_part
from .projected import ProjectedMixer

FIRST_VALUES = "value_mix.first"         # in ctx.extras: the first mixing layer's values [N, nkv dv]


def bucket_starts(rows: int, far: float) -> List[int]:
    """The first distance of every row of a bias table (see ``distance_bias``), in whole numbers and fractions: row h + k
    begins at the smallest n with (n / h)^(B - h) >= (far / h)^k."""
    h = rows // 2
    if rows < 2 or not far > h:
        raise ValueError(f"a bias table of {rows} rows needs at least two, and a furthest distance above half of them, got {far}")
    ratio, starts = Fraction(far) / h, list(range(h))
    for k in range(rows - h):
        n = max(h, int(h * float(ratio) ** (k / (rows - h))) - 1)       # close below, then exactly
        while Fraction(n, h) ** (rows - h) < ratio ** k:
            n += 1
        starts.append(n)
    return starts


def bias_by_distance(table: torch.Tensor, far: float) -> torch.Tensor:
    """table [B, heads] -> fp32 [heads, span]: the number for every distance up to the first of the last row."""
    starts = bucket_starts(int(table.shape[0]), far)
    span = starts[-1] + 1
    row, rows = 0, []
    for n in range(span):
        while row + 1 < len(starts) and starts[row + 1] <= n:
            row += 1
        rows.append(row)
    return table.to(torch.float32)[torch.tensor(rows, device=table.device)].t().contiguous()


class SoftmaxAttention(ProjectedMixer, Attention):
    graph_safe = True

    def __init__(self, rt: Runtime, hidden_size: int, num_heads: int, num_kv_heads: int, head_dim: int, value_dim: int,
                 scale: float, position: Optional[Mapping[str, Any]] = None, window: Optional[int] = None,
                 keep_first: int = 0, softcap: Optional[float] = None, sink: Optional[str] = None, qk_norm: Union[bool, str] = False,
                 norm_eps: float = 1e-6, values: str = "projected", value_mix: Optional[str] = None, init_std: float = 0.02,
                 names: Sequence[str] = ("q", "k", "v", "o"), kernels: str = "auto",
                 distance_bias: Optional[Mapping[str, Any]] = None, output_gate: bool = False):
        """``distance_bias`` {far, rows (None: read off a file's table), name ("rel")}."""
        Attention.__init__(self, rt, hidden_size, num_heads, num_kv_heads, head_dim, position=position, window=window,
                           scale=scale, kernels=kernels, init_std=init_std, value_dim=value_dim, keep_first=keep_first,
                           softcap=softcap, distance_bias=distance_bias is not None, output_gate=output_gate)
        self.far = float(distance_bias["far"]) if distance_bias is not None else 0.0
        self.bias_rows = int(distance_bias.get("rows") or -1) if distance_bias is not None else 0
        self.bias_name = str(distance_bias.get("name", "rel")) if distance_bias is not None else ""
        self.norm_rows = qk_norm == "rows"
        if qk_norm not in (False, True, "rows"):
            raise ValueError(f"softmax_attention: qk_norm {qk_norm!r}")
        if self.norm_rows and (values != "projected" or value_mix or getattr(self.position, "inv_freq", None) is not None):
            raise ValueError("a norm over all heads at once goes with projected values of the layer's own, without rotation")
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
        self.g_col = self.v_col + (0 if self.values_are_keys else self.nkv * self.vd)
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
            wide = (nh, nkv) if self.norm_rows else (1, 1)
            out[q + ".norm"] = WeightSpec((wide[0] * d,), ("uniform", 0.8, 1.2), **small)
            out[k + ".norm"] = WeightSpec((wide[1] * d,), ("uniform", 0.8, 1.2), **small)
        if self.distance_bias:
            out[self.bias_name] = WeightSpec((self.bias_rows, nh), ("normal", 1.0), **small)
        if self.output_gate:
            out["g"] = WeightSpec((nh * dv, H), init)
        if self.sink == "learned":
            out["sink"] = WeightSpec((nh,), ("normal", 1.0), **small)
        if self.value_mix == "mixed":
            out["vmix"] = WeightSpec((), ("uniform", 0.2, 0.8), **small)
        return out

    def stack_rows(self, tensors) -> Sequence[torch.Tensor]:
        q, k, v, _ = self.names
        return [tensors[q], tensors[k]] + ([] if self.values_are_keys else [tensors[v]]) + \
            ([tensors["g"]] if self.output_gate else [])

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
        if self.distance_bias:
            self.bias = K.distance_table(bias_by_distance(tensors[self.bias_name], self.far))
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
        gate = proj[:, self.g_col:self.g_col + nh * dv] if self.output_gate else None
        if self.norm_rows:
            K.qk_rows_prepare(proj, q, nh, nkv, d, self.q_norm, self.k_norm, self.norm_eps, ctx.slots[cache.group], kp, vp,
                              self.result_scale)
            self.attend(q, out, ctx, cache, gate)
            return
        K.qk_prepare(proj, q, nh, nkv, d, ctx.positions, self.q_norm, self.k_norm, self.norm_eps, pos.inv_freq,
                     pos.rotary_dim if pos.inv_freq is not None else 0, pos.pairing, pos.magnitude, ctx.slots[cache.group],
                     kp, vp, values_are_keys=self.values_are_keys, v_scale=self.result_scale, v_first=first,
                     v_lambda=self.mix_lambda)
        self.attend(q, out, ctx, cache, gate)

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
        gate = _at(proj, self.g_col * ab) if self.output_gate else None
        if self.norm_rows:
            program.op("core", "ia_qk_rows_prepare",
                       [proj, act, proj_row, q, nh * d, self.q_norm, self.k_norm, float(self.norm_eps),
                        program.slots(view.group), kp, vp, program.N, nh, nkv, d, dv, int(kp.shape[2]), int(kp.shape[0]),
                        float(self.result_scale), STREAM])
            self.emit_attend(program, view, q, nh * d, ALWAYS, out, out_row, gate, proj_row)
            return
        rot = pos.rotary_dim if pos.inv_freq is not None else 0
        program.op("core", "ia_qk_prepare",
                   [proj, act, proj_row, q, nh * d, self.q_norm, self.k_norm, float(self.norm_eps), program.positions,
                    program.slots(view.group), pos.inv_freq if rot else None,
                    int(bool(rot) and pos.inv_freq.dtype == torch.float64), rot, K.PAIRINGS[pos.pairing],
                    float(pos.magnitude), kp, vp, program.N, nh, nkv, d, dv, int(kp.shape[2]), int(kp.shape[0]),
                    int(self.values_are_keys), float(self.result_scale), first, first_row, float(self.mix_lambda), STREAM])
        self.emit_attend(program, view, q, nh * d, ALWAYS, out, out_row, gate, proj_row if gate is not None else 0)


def _at(where, nbytes: int):
    """The place ``nbytes`` behind an address of the program (a Buffer, or a place inside one)."""
    from ..engine.program import Buffer
    return where.at(nbytes) if isinstance(where, Buffer) else where.buffer.at(where.nbytes + nbytes)


register_part("mixer", "softmax_attention", SoftmaxAttention)
