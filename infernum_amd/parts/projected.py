"""Mixers whose work lies between two plain products, and several of them side by side.

A :class:`ProjectedMixer` multiplies a token's input with ONE matrix (all its projections stacked), works on the rows of
that product, and multiplies what it leaves with its output matrix:

    p = A x,      m = mix(p, cache, state),      y = c O m,

``result_scale`` c being part of m.  A mixer that keeps to this (``stack_rows``, ``load_small``, ``mix``, ``emit_mix``)
can stand alone (:meth:`forward` and :meth:`native` here) or beside others on the same input:

``side_by_side``: y = sum_i c_i mixer_i(x).  The mixers' stacked matrices are stacked once more and their output
matrices laid side by side, so that all of them cost the two products that one costs; every mixer keeps its own pages
and its own state slot (``Block.cached_parts``).
"""
from __future__ import annotations

from typing import Any, Dict, Mapping, Optional, Sequence, Tuple

import torch

from ..kernels import api as K
from .base import CacheView, Mixer, PartSpec, Runtime, StepContext, WeightSpec, make_part, register_part
from .linear import emit_linear, linear, prepare_weights

ROW_MULTIPLE = 8        # a mixer's columns of the common row begin and end on a multiple of 16 bytes


def _padded(n: int) -> int:
    return -(-n // ROW_MULTIPLE) * ROW_MULTIPLE


class ProjectedMixer(Mixer):
    graph_safe = True
    hidden_size: int
    result_scale: float = 1.0        # multiplies the mixer's result; folded into what ``mix`` leaves
    out_cols: int                    # values that ``mix`` leaves per token

    # ---- what a mixer of this kind gives ---------------------------------------------------------
    def stack_rows(self, tensors: Mapping[str, torch.Tensor]) -> Sequence[torch.Tensor]:
        """The projections, in the order of their columns in the product's rows."""
        raise NotImplementedError

    def output_matrix(self, tensors: Mapping[str, torch.Tensor]) -> torch.Tensor:
        """[hidden, out_cols]."""
        raise NotImplementedError

    def load_small(self, tensors: Mapping[str, torch.Tensor]) -> None:
        """Everything else."""

    def mix(self, proj: torch.Tensor, ctx: StepContext, cache: CacheView, out: torch.Tensor) -> None:
        """proj [N, >= the stacked rows] (this mixer's columns, first), out [N, out_cols]: both may be columns of wider rows."""
        raise NotImplementedError

    def emit_mix(self, program, view: CacheView, proj: Any, proj_row: int, out: Any, out_row: int) -> None:
        """The launches of :meth:`mix`: ``proj`` and ``out`` are addresses, ``*_row`` values from a row to the next."""
        raise NotImplementedError

    def rows_key(self) -> str:
        """The name of the program's buffer for the product's rows (a mixer whose rows are read later in the step has
        a name of its own for them)."""
        return "projected.rows"

    # ---- alone -----------------------------------------------------------------------------------
    def load(self, tensors: Dict[str, torch.Tensor]) -> None:
        self.w_in = _stack(list(self.stack_rows(tensors)))
        self.w_o = self.output_matrix(tensors).contiguous()
        self.load_small(tensors)
        prepare_weights(self.rt, [(self.w_in, None, False), (self.w_o, None, True)])

    def forward(self, x: torch.Tensor, ctx: StepContext, cache: CacheView):
        proj = linear(x, self.w_in, kernels=self.rt.kernels)
        out = torch.empty((x.shape[0], self.out_cols), dtype=self.rt.dtype, device=x.device)
        self.mix(proj, ctx, cache, out)
        return linear(out, self.w_o, keep_split=True, kernels=self.rt.kernels)

    def _forward_is_own(self) -> bool:
        return type(self).forward is ProjectedMixer.forward

    def native(self, program, view: CacheView) -> None:
        if not self._forward_is_own():
            return super().native(program, view)
        rt, N = self.rt, program.N
        proj = emit_linear(program, program.x, N, self.w_in, rt.dtype, None, False, self.rows_key(), "projected.in").tensor()
        out = program.buffer("projected.mixed", program.T * self.out_cols * program.act_bytes)
        self.emit_mix(program, view, proj, int(self.w_in.shape[0]), out, self.out_cols)
        program.pending = emit_linear(program, out, N, self.w_o, rt.dtype, None, True, "projected.out", "projected.o")


def _stack(mats: Sequence[torch.Tensor]) -> torch.Tensor:
    rows = sum(int(m.shape[0]) for m in mats)
    pad = _padded(rows) - rows
    if pad:
        mats = list(mats) + [mats[0].new_zeros((pad, mats[0].shape[1]))]
    return torch.cat(list(mats), dim=0).contiguous()


class SideBySide(Mixer):
    graph_safe = True

    def __init__(self, rt: Runtime, hidden_size: int, mixers: Mapping[str, Mapping[str, Any]]):
        """``mixers``: name -> {kind, params, scale (default 1)}; a mixer's tensors stand under its name and a dot."""
        super().__init__(rt)
        self.hidden_size = int(hidden_size)
        self.parts: Dict[str, ProjectedMixer] = {}
        for name, m in mixers.items():
            part = make_part("mixer", PartSpec(m["kind"], m["params"]), rt)
            if not isinstance(part, ProjectedMixer):
                raise ValueError(f"side_by_side: a mixer of kind {m['kind']!r} does not work between two plain products")
            part.result_scale = float(m.get("scale", 1.0))
            self.parts[name] = part
        self.graph_safe = all(getattr(p, "graph_safe", False) for p in self.parts.values())

    def cached_companions(self) -> Dict[str, Any]:
        return dict(self.parts)

    def step_needs(self) -> Dict[str, Any]:
        out: Dict[str, Any] = {}
        for p in self.parts.values():
            out.update(p.step_needs())
        return out

    def weights(self) -> Dict[str, WeightSpec]:
        return {f"{name}.{local}": ws for name, p in self.parts.items() for local, ws in p.weights().items()}

    def load(self, tensors: Dict[str, torch.Tensor]) -> None:
        mats, outs, self.columns = [], [], {}          # name -> (first column of the rows, of what the mixers leave)
        at = out_at = 0
        for name, p in self.parts.items():
            own = {local: tensors[f"{name}.{local}"] for local in p.weights()}
            w = _stack(list(p.stack_rows(own)))
            mats.append(w)
            outs.append(p.output_matrix(own))
            self.columns[name] = (at, out_at)
            at, out_at = at + int(w.shape[0]), out_at + int(outs[-1].shape[1])
            p.load_small(own)
        self.w_in, self.w_o = torch.cat(mats, dim=0).contiguous(), torch.cat(outs, dim=1).contiguous()
        prepare_weights(self.rt, [(self.w_in, None, False), (self.w_o, None, True)])

    def _view(self, cache: Optional[CacheView], name: str) -> CacheView:
        view = (cache.others if cache is not None else {}).get(name)
        if view is None:
            raise K.KernelError(f"side_by_side: there is no cache view for {name!r}")
        return view

    def forward(self, x: torch.Tensor, ctx: StepContext, cache: CacheView):
        proj = linear(x, self.w_in, kernels=self.rt.kernels)
        out = torch.empty((x.shape[0], int(self.w_o.shape[1])), dtype=self.rt.dtype, device=x.device)
        for name, p in self.parts.items():
            c, o = self.columns[name]
            p.mix(proj[:, c:], ctx, self._view(cache, name), out[:, o:o + p.out_cols])
        return linear(out, self.w_o, keep_split=True, kernels=self.rt.kernels)

    def native(self, program, view: CacheView) -> None:
        if type(self).forward is not SideBySide.forward:
            return super().native(program, view)
        rt, N, ab = self.rt, program.N, program.act_bytes
        keys = [p.rows_key() for p in self.parts.values() if p.rows_key() != "projected.rows"]
        row, out_row = int(self.w_in.shape[0]), int(self.w_o.shape[1])
        proj = emit_linear(program, program.x, N, self.w_in, rt.dtype, None, False, keys[0] if keys else "projected.rows",
                           "projected.in").tensor()
        out = program.buffer("projected.mixed", program.T * out_row * ab)
        for name, p in self.parts.items():
            c, o = self.columns[name]
            p.emit_mix(program, self._view(view, name), proj.at(c * ab), row, out.at(o * ab), out_row)
        program.pending = emit_linear(program, out, N, self.w_o, rt.dtype, None, True, "projected.out", "projected.o")


register_part("mixer", "side_by_side", SideBySide)
