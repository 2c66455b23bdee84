"""Hyper-connections: what one sublayer of the ``hyper`` arrangement owns (category ``hyper``).

With S streams X_s, all equal to the residual stream where the first sublayer begins, a sublayer f with the vectors in,
out [S] and the matrix mix [from, to]:

    u = sum_s in[s] X_s,      y = f(norm(u)),      X_t <- sum_s mix[s, t] X_s + mult out[t] y     (all from the old X),

and behind the last sublayer the residual stream is the sum of the streams.  ``last`` marks that sublayer; which one is
first follows from the step (no sublayer before it has run).  What a sublayer returned is kept, with its own weights,
until the next one enters (or the stream is closed): one kernel then writes it back and forms the next u, normed.
Streams, sums and weights are fp32.
"""
from __future__ import annotations

from typing import Any, Dict, Sequence

import torch

from ..kernels import api as K
from .base import Part, Runtime, StepContext, WeightSpec, register_part

STREAMS = "hyper.streams"        # in ctx.extras: (streams [N, S, H] or None, the sublayer whose result is pending)


class HyperConnection(Part):
    category = "hyper"
    graph_safe = True

    def __init__(self, rt: Runtime, hidden_size: int, streams: int, mult: float = 1.0, last: bool = False,
                 names: Sequence[str] = ("in", "out", "mix"), init_std: float = 0.02):
        super().__init__(rt)
        self.hidden_size, self.streams, self.mult, self.last = int(hidden_size), int(streams), float(mult), bool(last)
        if not 1 <= self.streams <= K.HYPER_MAX_STREAMS:
            raise ValueError(f"hyper-connections: 1 .. {K.HYPER_MAX_STREAMS} streams, got {streams}")
        self.names = tuple(names)

    def weights(self) -> Dict[str, WeightSpec]:
        S, small = self.streams, dict(follows_compute_dtype=False)
        a, b, m = self.names
        return {a: WeightSpec((S,), ("uniform", 0.5 / S, 1.5 / S), **small), b: WeightSpec((S,), ("uniform", 0.5, 1.5), **small),
                m: WeightSpec((S, S), ("uniform", 0.0, 2.0 / S), **small)}

    def load(self, tensors: Dict[str, torch.Tensor]) -> None:
        a, b, m = (tensors[n].to(torch.float32).contiguous() for n in self.names)
        self.w_in, self.w_mix = a, m
        self.w_out = (b * self.mult).contiguous()

    # ---- the parts' own way --------------------------------------------------------------------
    def enter(self, h: torch.Tensor, pending: Any, ctx: StepContext, norm) -> torch.Tensor:
        """What the sublayer reads: norm(u), in the compute dtype, after the sublayer before (if any) is written back."""
        x = torch.empty(h.shape, dtype=self.rt.dtype, device=h.device)
        streams, before = ctx.extras.get(STREAMS, (None, None))
        if pending is not None and before is None:
            raise K.KernelError("hyper: a layer of another arrangement left its delta unadded")
        new = streams
        if before is not None and streams is None:
            new = torch.empty((h.shape[0], self.streams, h.shape[1]), dtype=torch.float32, device=h.device)
        K.hyper_step(h if streams is None else streams, self.streams, new, pending, before.w_mix if before else None,
                     before.w_out if before else None, self.w_in, norm.weight, norm.eps, x)
        ctx.extras[STREAMS] = (new, None)
        return x

    def leave(self, h: torch.Tensor, y: Any, ctx: StepContext) -> Any:
        """The sublayer's result, pending; after the last sublayer h becomes the sum of the streams and nothing is."""
        streams, _ = ctx.extras.get(STREAMS, (None, None))
        if not self.last:
            ctx.extras[STREAMS] = (streams, self)
            return y
        out = torch.empty_like(h) if streams is None else h
        K.hyper_step(h if streams is None else streams, self.streams, None, y, self.w_mix, self.w_out, None, None, 0.0, out)
        if streams is None:
            h.copy_(out)
        ctx.extras.pop(STREAMS, None)
        return None

    # ---- the step's program --------------------------------------------------------------------
    def _emit(self, program, writes_back, norm, inw) -> None:
        from ..engine.program import STREAM
        S, H, T = self.streams, self.hidden_size, program.T
        state = getattr(program, "hyper_state", None) or {"live": False}
        streams = program.buffer("hyper.streams", T * S * H * 4)
        src, src_streams = (streams, S) if state["live"] else (program.h, 0)
        program.keep(self.w_in, writes_back.w_mix if writes_back else None, writes_back.w_out if writes_back else None,
                     norm.weight if norm is not None else None)
        for alt in (program.pending.alts if writes_back is not None else [None]):
            where, code, splits = None, 0, 1
            if alt is not None:
                where, splits = alt.where, alt.splits or 1
                code = K.DTYPE_CODE[torch.float32] if alt.splits else K.DTYPE_CODE[alt.dtype]
            args = [src, src_streams, streams, where, code, splits, program.N, writes_back.w_mix if writes_back else None,
                    writes_back.w_out if writes_back else None, inw, norm.weight if norm is not None else None,
                    K.DTYPE_CODE[norm.weight.dtype] if norm is not None else 0, None if norm is not None else program.h,
                    program.x if norm is not None else None, program.act_code, program.N, S, H,
                    float(norm.eps) if norm is not None else 0.0, STREAM]
            program.op("core", "ia_hyper_step", args, *([alt.when] if alt is not None else []))
        program.pending = None

    def emit_enter(self, program, norm) -> None:
        state = getattr(program, "hyper_state", None) or {"live": False, "before": None}
        if program.pending is not None and state["before"] is None:
            raise K.KernelError("hyper: a layer of another arrangement left its delta unadded")
        before = state["before"]
        self._emit(program, before, norm, self.w_in)
        program.hyper_state = {"live": state["live"] or before is not None, "before": None}

    def emit_leave(self, program) -> None:
        state = program.hyper_state
        if not self.last:
            program.hyper_state = {"live": state["live"], "before": self}
            return
        self._emit(program, self, None, None)
        program.hyper_state = None


register_part("hyper", "hyper_connection", HyperConnection)
