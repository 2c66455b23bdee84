"""The generalized delta rule: a recurrent mixer that decays its state channel by channel, takes out part of what lies
along a token's key, and writes the token's own key and value.

r, k, v, g = projections of x, heads x dim each; the decay's logits come through a narrow middle.  Per head and key channel

    w = exp(-e^(-1/2) sigmoid(W2 tanh(W1 x) + w0)),        a = sigmoid(Wa x + ab),        u = k / sqrt(sum k^2 + 1e-6),

and with a state S of [dim, dim] that starts at zero

    S_t = diag(w_t) S_(t-1) - (a_t * u_t) (u_t^T S_(t-1)) + k_t v_t^T   (both terms read the old state),   o_t = S_t^T r_t.

Each head's o is divided by its root mean square, multiplied by a weight per value of every head and by sigmoid(g), and
the heads, concatenated, are projected back.  Between steps a request keeps every head's S in one state slot of fp32
values.  Decays, removal rates, unit norms, the state and the norm are fp32 whatever the activations' type.
Single tokens run the recurrence itself, portions of prompts chunks of rows as matrix products (csrc/delta_rule.hip).
"""
from __future__ import annotations

import math
from typing import Any, Dict, Optional, Sequence

import torch

from ..kernels import api as K
from .base import CacheView, Runtime, StateSpec, StepContext, WeightSpec, register_part
from .linear import emit_linear, linear, prepare_weights
from .projected import ProjectedMixer

DECAY_SCALE = math.exp(-0.5)
KEY_EPS = 1e-6


class DeltaRule(ProjectedMixer):
    graph_safe = True

    def __init__(self, rt: Runtime, hidden_size: int, num_heads: int, head_dim: int, norm_eps: float,
                 decay_rank: Optional[int] = None, init_std: float = 0.02,
                 names: Sequence[str] = ("r", "k", "v", "g", "a", "a.b", "w1", "w2", "w0", "norm", "o")):
        """``decay_rank``: the width of the decay logits' middle (None: read off the tensors of a file)."""
        super().__init__(rt)
        self.hidden_size, self.nh, self.dim = int(hidden_size), int(num_heads), int(head_dim)
        if self.dim > K.DELTA_MAX_DIM:
            raise ValueError(f"delta_rule: heads of {self.dim}, at most {K.DELTA_MAX_DIM}")
        self.norm_eps, self.init_std, self.names = float(norm_eps), init_std, tuple(names)
        if len(self.names) != 11:
            raise ValueError("delta_rule: eleven tensor names (r, k, v, g, a, a's bias, w1, w2, w0, norm, o)")
        self.rank = int(decay_rank) if decay_rank else -1
        n = self.n = self.nh * self.dim
        # columns of the projected row: r | k | v | g | a | w1's
        self.r_col, self.k_col, self.v_col, self.g_col, self.a_col, self.m_col = (i * n for i in range(6))
        self.out_cols = n

    def state_spec(self) -> StateSpec:
        return StateSpec((K.delta_state_floats(self.nh, self.dim),))

    def step_needs(self) -> Dict[str, Any]:
        return {"row_tiles": K.PREFILL_TILE_ROWS}

    def weights(self) -> Dict[str, WeightSpec]:
        H, n, rank, small = self.hidden_size, self.n, self.rank, dict(follows_compute_dtype=False)
        r, k, v, g, a, ab, w1, w2, w0, norm, o = self.names
        init = ("normal", self.init_std)
        out = {name: WeightSpec((n, H), init) for name in (r, k, v, g, a)}
        out.update({ab: WeightSpec((n,), ("normal", 1.0), **small), w1: WeightSpec((rank, H), init),
                    w2: WeightSpec((n, rank), ("normal", max(rank, 1) ** -0.5)),
                    w0: WeightSpec((n,), ("uniform", -6.0, 0.0), **small),
                    norm: WeightSpec((n,), ("uniform", 0.8, 1.2), **small), o: WeightSpec((H, n), init)})
        return out

    def stack_rows(self, tensors) -> Sequence[torch.Tensor]:
        r, k, v, g, a, _, w1, _, _, _, _ = self.names
        return [tensors[name] for name in (r, k, v, g, a, w1)]

    def output_matrix(self, tensors) -> torch.Tensor:
        return tensors[self.names[10]]

    def load_small(self, tensors) -> None:
        _, _, _, _, _, ab, w1, w2, w0, norm, _ = self.names
        f32 = lambda name: tensors[name].to(torch.float32).contiguous()            # noqa: E731
        self.w_2 = tensors[w2].contiguous()
        self.mid = int(tensors[w1].shape[0])
        if self.mid != int(self.w_2.shape[1]):
            raise ValueError(f"delta_rule: the decay's two matrices do not meet: {tuple(tensors[w1].shape)} and {tuple(self.w_2.shape)}")
        self.a_bias, self.w_0 = f32(ab), f32(w0)
        self.w_norm = (f32(norm) * self.result_scale).contiguous()          # the result's factor rides on the norm's weight
        prepare_weights(self.rt, [(self.w_2, None, False)])

    def _state(self, cache: CacheView) -> torch.Tensor:
        if cache is None or cache.state is None:
            raise K.KernelError("delta_rule needs a state slot")
        return cache.state

    def mix(self, proj: torch.Tensor, ctx: StepContext, cache: CacheView, out: torch.Tensor) -> None:
        n, dev = proj.shape[0], proj.device
        state = self._state(cache)
        mid = K.tanh_rows(proj[:, self.m_col:self.m_col + self.mid])
        z = linear(mid, self.w_2, out_dtype=torch.float32, kernels=self.rt.kernels)
        a, inv = K.delta_prepare(proj, self.k_col, self.a_col, z, self.w_0, self.a_bias, self.nh, self.dim, DECAY_SCALE, KEY_EPS)
        o = torch.empty((n, self.n), dtype=torch.float32, device=dev)
        nd = ctx.num_decode
        if nd > 0:              # single tokens: the recurrence itself
            K.delta_scan(proj, self.r_col, self.k_col, self.v_col, z, a, inv, state, o, ctx.seq_starts[:nd + 1],
                         ctx.state_slots[:nd], self.nh, self.dim)
        if ctx.num_seqs > nd:   # portions of prompts: chunks of rows as matrix products
            tiles, num_tiles = ctx.row_tiles(K.PREFILL_TILE_ROWS)
            K.delta_chunked(proj, self.r_col, self.k_col, self.v_col, z, a, inv, state, o, ctx.seq_starts, ctx.state_slots,
                            tiles, num_tiles, nd, ctx.num_seqs - nd, self.nh, self.dim)
        K.head_norm_gate(o, proj, self.g_col, self.w_norm, self.norm_eps, self.nh, self.dim, out, per_head=True,
                         plain_sigmoid=True)

    def emit_mix(self, program, view: CacheView, proj, proj_row: int, out, out_row: int) -> None:
        from ..engine.program import STREAM, Guard
        from .softmax_attention import _at
        rt, N, T, act, ab, nh, dim = self.rt, program.N, program.T, program.act_code, program.act_bytes, self.nh, self.dim
        state = self._state(view)
        program.keep(state, self.a_bias, self.w_0, self.w_norm)
        mid = program.buffer("delta.mid", T * self.mid * ab)
        program.op("core", "ia_delta_tanh_rows", [_at(proj, self.m_col * ab), proj_row, mid, act, N, self.mid, STREAM])
        z = emit_linear(program, mid, N, self.w_2, torch.float32, None, False, "delta.z", "delta.w2").tensor()
        a = program.buffer("delta.a", T * self.n * 4)
        inv = program.buffer("delta.inv", T * nh * 4)
        program.op("core", "ia_delta_prepare", [proj, act, proj_row, self.k_col, self.a_col, z, self.w_0, self.a_bias, a, inv,
                                                N, nh, dim, DECAY_SCALE, KEY_EPS, STREAM])
        o = program.buffer("delta.o", T * self.n * 4)
        program.op("core", "ia_delta_scan", [proj, act, proj_row, self.r_col, self.k_col, self.v_col, z, a, inv, state,
                                             int(state.stride(0)), o, program.seq_starts, program.state_slots, program.ND, nh,
                                             dim, STREAM], Guard.between(program.ND, 1))
        # a request holds a state slot, and a tile at least one row: so many tiles a step has at most
        most = -(-T // K.PREFILL_TILE_ROWS) + int(state.shape[0])
        records = program.buffer("delta.records", most * 4 * K.delta_chunk_floats(nh, dim) * 4)
        tiles, num_tiles = program.row_tiles(K.PREFILL_TILE_ROWS)
        program.op("core", "ia_delta_chunked", [proj, act, proj_row, self.r_col, self.k_col, self.v_col, z, a, inv, state,
                                                int(state.stride(0)), o, program.seq_starts, program.state_slots, tiles,
                                                num_tiles, program.ND, program.NP, records, nh, dim, STREAM],
                   Guard.between(program.NP, 1))
        program.op("core", "ia_head_norm_gate", [o, proj, act, proj_row, self.g_col, self.w_norm, out, out_row, N, nh, dim,
                                                 float(self.norm_eps), 1, 1, STREAM])


register_part("mixer", "delta_rule", DeltaRule)
