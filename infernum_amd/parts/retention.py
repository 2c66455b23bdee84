"""Retention: a recurrent mixer with one fixed decay per head and no softmax or denominator.

q, k (heads x dim), v and the gate g (heads x vdim) = projections of x, no biases; q and k rotated by the position encoding
(halves), k times dim^(-1/2) behind the rotation.  Per head, with a state S of [dim, vdim] that starts at zero,

    S_t = decay S_(t-1) + k_t v_t^T,        o_t = S_t^T q_t;

each head's o is divided by its root mean square, and the heads, concatenated, are multiplied by silu(g) and projected
back.  Between steps a request keeps every head's S in one state slot of fp32 values.  Rotated queries and keys, decays,
the state and the norm are fp32 whatever the activations' type.  Single tokens (and sizes that the chunks do not take) run
the recurrence itself, portions of prompts tiles of rows as matrix products; both end with the norm and the gate
(csrc/retention.hip).  The angles' cosines and sines are made once a step for all layers that rotate alike.
"""
from __future__ import annotations

import math
from typing import Any, Dict, Mapping, Optional, Sequence

import torch

from ..kernels import api as K
from .base import CacheView, PartSpec, Runtime, StateSpec, StepContext, WeightSpec, make_part, register_part
from .projected import ProjectedMixer


class Retention(ProjectedMixer):
    graph_safe = True

    def __init__(self, rt: Runtime, hidden_size: int, num_heads: int, head_dim: int, value_dim: int, decay: Sequence[float],
                 norm_eps: float, position: Optional[Mapping[str, Any]] = None, k_scale: Optional[float] = None,
                 init_std: float = 0.02, names: Sequence[str] = ("q", "k", "v", "g", "o")):
        """``decay``: a number in [0, 1] per head.  ``k_scale``: the factor on the keys (default head_dim^(-1/2))."""
        super().__init__(rt)
        self.hidden_size, self.nh, self.dim, self.vdim = int(hidden_size), int(num_heads), int(head_dim), int(value_dim)
        if max(self.dim, self.vdim) > K.RETENTION_MAX_DIM:
            raise ValueError(f"retention: heads of {self.dim} and {self.vdim}, at most {K.RETENTION_MAX_DIM}")
        decay = [float(d) for d in decay]
        if len(decay) != self.nh or not all(0.0 <= d <= 1.0 for d in decay):
            raise ValueError(f"retention: a decay between 0 and 1 for each of {self.nh} heads, got {decay}")
        logs = [math.log2(d) if d > 0.0 else -math.inf for d in decay]
        self.decay = torch.tensor([decay, logs], dtype=torch.float32).to(rt.device)
        self.norm_eps, self.init_std, self.names = float(norm_eps), init_std, tuple(names)
        self.k_scale = float(k_scale) if k_scale is not None else self.dim ** -0.5
        pos_spec = PartSpec(**position) if isinstance(position, Mapping) else (position or PartSpec("none"))
        self.position = make_part("position", pos_spec, rt)
        self.rot = int(self.position.rotary_dim) if self.position.inv_freq is not None else 0
        if self.rot and (getattr(self.position, "pairing", "half") != "half" or getattr(self.position, "magnitude", 1.0) != 1.0):
            raise ValueError("retention rotates halves, without a factor on sine and cosine")
        # layers with equal frequencies share a step's cosines and sines
        self._angles = ("rotation_table", self.rot, self.position.inv_freq.cpu().numpy().tobytes()) if self.rot else None
        self.graph_safe = getattr(self.position, "graph_safe", False)
        nq, nv = self.nh * self.dim, self.nh * self.vdim
        self.cols = (0, nq, 2 * nq, 2 * nq + nv)                 # columns of the projected row: q | k | v | g
        self.out_cols = nv

    # ---- what it needs ---------------------------------------------------
    def state_spec(self) -> StateSpec:
        return StateSpec((K.retention_state_floats(self.nh, self.dim, self.vdim),))

    def step_needs(self) -> Dict[str, Any]:
        return {"row_tiles": K.PREFILL_TILE_ROWS} if self.rt.dtype == torch.bfloat16 else {}

    def weights(self) -> Dict[str, WeightSpec]:
        H, nq, nv = self.hidden_size, self.nh * self.dim, self.nh * self.vdim
        q, k, v, g, o = self.names
        init = ("normal", self.init_std)
        return {q: WeightSpec((nq, H), init), k: WeightSpec((nq, H), init), v: WeightSpec((nv, H), init),
                g: WeightSpec((nv, H), init), o: WeightSpec((H, nv), init)}

    def stack_rows(self, tensors) -> Sequence[torch.Tensor]:
        return [tensors[name] for name in self.names[:4]]

    def output_matrix(self, tensors) -> torch.Tensor:
        return tensors[self.names[4]]

    def _state(self, cache: CacheView) -> torch.Tensor:
        if cache is None or cache.state is None:
            raise K.KernelError("retention needs a state slot")
        return cache.state

    def _chunks(self, proj_row: int) -> bool:
        return self.rt.kernels == "auto" and K.retention_chunked_takes(self.rt.dtype, self.nh, self.dim, self.vdim, proj_row,
                                                                       self.cols)

    # ---- one step --------------------------------------------------------
    def mix(self, proj: torch.Tensor, ctx: StepContext, cache: CacheView, out: torch.Tensor) -> None:
        state, table = self._state(cache), None
        if self.rot:
            table = ctx.extras.get(self._angles)
            if table is None:
                table = ctx.extras[self._angles] = K.rotation_table(ctx.positions, self.position.inv_freq)
        same = (self.cols, table, self.rot, self.k_scale, self.decay, self.norm_eps, self.result_scale, state, out)
        nd, sizes = ctx.num_decode, (self.nh, self.dim, self.vdim)
        stepped = nd if self._chunks(int(proj.stride(0))) else ctx.num_seqs
        if stepped > 0:
            K.retention_step(proj, *same, ctx.seq_starts[:stepped + 1], ctx.state_slots[:stepped], *sizes)
        if ctx.num_seqs > stepped:
            tiles, num_tiles = ctx.row_tiles(K.PREFILL_TILE_ROWS)
            K.retention_chunked(proj, *same, ctx.seq_starts, ctx.state_slots, tiles, num_tiles, nd, *sizes)

    def emit_mix(self, program, view: CacheView, proj, proj_row: int, out, out_row: int) -> None:
        from ..engine.program import STREAM, Guard
        N, T, act = program.N, program.T, program.act_code
        state, table = self._state(view), None
        program.keep(state, self.decay, self.position.inv_freq)
        if self.rot:
            made = getattr(program, "rotation_tables", None)
            if made is None:
                made = program.rotation_tables = {}
            table = made.get(self._angles)
            if table is None:               # the first layer of the step that rotates so makes it for all of them
                table = made[self._angles] = program.buffer(f"retention.angles.{len(made)}", T * (self.rot // 2) * 8)
                freq = self.position.inv_freq
                program.op("core", "ia_rotation_table", [program.positions, freq, int(freq.dtype == torch.float64), table, N,
                                                         self.rot // 2, STREAM])
        same = [proj, act, proj_row, *self.cols, table, self.rot, float(self.k_scale), self.decay, float(self.norm_eps),
                float(self.result_scale), state, int(state.stride(0)), out, out_row, program.seq_starts, program.state_slots]
        sizes = [self.nh, self.dim, self.vdim, STREAM]
        if not self._chunks(proj_row):
            program.op("core", "ia_retention_step", [*same, program.B, *sizes])
            return
        program.op("core", "ia_retention_step", [*same, program.ND, *sizes], Guard.between(program.ND, 1))
        # a request holds a state slot, and a tile at least one row: so many tiles a step has at most
        floats = K.retention_state_floats(self.nh, self.dim, self.vdim)
        most = -(-T // K.PREFILL_TILE_ROWS) + int(state.shape[0])
        records = program.buffer("retention.records", most * floats * 4)
        tiles, num_tiles = program.row_tiles(K.PREFILL_TILE_ROWS)
        program.op("core", "ia_retention_chunked", [*same, tiles, num_tiles, program.ND, records, floats, *sizes],
                   Guard.between(program.NP, 1))


register_part("mixer", "retention", Retention)
