"""A selective state-space mixer of the Mamba-1 form: a decay per channel and state value.

One input projection makes, side by side in a row, x and the gate z (``inner`` values each).  x passes a short causal
convolution per channel (with a bias) and silu.  A second projection of that x makes a narrow row [dt: dt_rank | B: states |
C: states]; a third one brings dt back to the channels.  Per channel c and state value n, with a state that starts at zero,

    dt_c = softplus((Wdt dt)_c + bias_c),      S[c, n] <- exp(-exp(A_log[c, n]) dt_c) S[c, n] + dt_c x_c B_n,
    y_c = sum_n S[c, n] C_n + D_c x_c;

y times silu(z) is projected back to the model's width.  Between steps a request keeps, in one state slot of fp32 values:
the last ``conv_taps - 1`` inputs of the convolution, then S, [states][inner].  Step sizes, decays and the state are fp32
whatever the activations' type (csrc/selective_scan.hip).

The narrow row is laid out for the kernels: dt, then B and C in as many columns each as the scan keeps in registers, zeros in
between and up to a multiple of ``ROW_MULTIPLE``; the third projection reads the whole row, with zeros where B and C stand.
"""
from __future__ import annotations

import math
from typing import Dict, Optional

import torch

from ..kernels import api as K
from .base import CacheView, Mixer, Runtime, StateSpec, StepContext, WeightSpec, register_part
from .linear import emit_linear, linear, prepare_weights

ROW_MULTIPLE = 64       # inner dimension of the products that read the narrow row


class Mamba1Mixer(Mixer):
    graph_safe = True

    def __init__(self, rt: Runtime, hidden_size: int, inner: int, state_size: int, dt_rank: int, conv_taps: int,
                 init_std: float = 0.02):
        super().__init__(rt)
        self.hidden_size, self.inner, self.Ns, self.rank = int(hidden_size), int(inner), int(state_size), int(dt_rank)
        self.taps, self.init_std = int(conv_taps), init_std
        if self.taps < 1:
            raise ValueError(f"a convolution needs at least one tap, got {conv_taps}")
        if K.selective_columns(self.Ns) == 0:
            raise ValueError(f"mamba1: a state of {self.Ns} values a channel, at most 128")
        self.conv_floats = (self.taps - 1) * self.inner
        cols = K.selective_columns(self.Ns)
        self.b_col = -(-self.rank // 8) * 8
        self.c_col = self.b_col + cols
        self.row = -(-(self.c_col + cols) // ROW_MULTIPLE) * ROW_MULTIPLE

    # ---- what it needs ---------------------------------------------------
    def state_spec(self) -> StateSpec:
        return StateSpec((self.conv_floats + self.Ns * self.inner,))

    def weights(self) -> Dict[str, WeightSpec]:
        H, I, Ns, R, small = self.hidden_size, self.inner, self.Ns, self.rank, dict(follows_compute_dtype=False)
        return {
            "in": WeightSpec((2 * I, H), ("normal", self.init_std)),
            "conv": WeightSpec((I, self.taps), ("normal", self.taps ** -0.5), **small),
            "conv.b": WeightSpec((I,), ("normal", 0.1), **small),
            "x": WeightSpec((R + 2 * Ns, I), ("normal", I ** -0.5)),
            "dt": WeightSpec((I, R), ("normal", R ** -0.5)),
            "dt.b": WeightSpec((I,), ("uniform", -4.5, -1.0), **small),
            "A_log": WeightSpec((I, Ns), ("uniform", -0.7, 2.7), **small),
            "D": WeightSpec((I,), ("uniform", 0.5, 1.5), **small),
            "o": WeightSpec((H, I), ("normal", self.init_std)),
        }

    def load(self, tensors: Dict[str, torch.Tensor]) -> None:
        f32 = lambda name: tensors[name].to(torch.float32).contiguous()            # noqa: E731
        R, Ns = self.rank, self.Ns
        self.w_in, self.w_o = tensors["in"].contiguous(), tensors["o"].contiguous()
        self.w_conv, self.b_conv = f32("conv").t().contiguous(), f32("conv.b")        # tap by tap: [taps, channels]
        low = tensors["x"]
        self.w_low = low.new_zeros((self.row, self.inner))
        self.w_low[:R], self.w_low[self.b_col:self.b_col + Ns], self.w_low[self.c_col:self.c_col + Ns] = \
            low[:R], low[R:R + Ns], low[R + Ns:]
        self.w_dt = low.new_zeros((self.inner, self.row))
        self.w_dt[:, :R] = tensors["dt"]
        self.dt_bias, self.skip = f32("dt.b"), f32("D")
        self.a2 = (-torch.exp(f32("A_log")) * math.log2(math.e)).t().contiguous()     # [states, channels]
        prepare_weights(self.rt, [(self.w_in, None, False), (self.w_low, None, False), (self.w_dt, None, False),
                                  (self.w_o, None, True)])

    def _state(self, cache: CacheView) -> torch.Tensor:
        if cache is None or cache.state is None:
            raise K.KernelError("mamba1 needs a state slot")
        return cache.state

    # ---- one step --------------------------------------------------------
    def forward(self, x: torch.Tensor, ctx: StepContext, cache: CacheView):
        n, I, kn = x.shape[0], self.inner, self.rt.kernels
        conv_state = self._state(cache)
        state = conv_state[:, self.conv_floats:]
        proj = linear(x, self.w_in, kernels=kn)                                   # [n, x | z]
        u, z = proj[:, :I], proj[:, I:]
        c = torch.empty((n, I), dtype=self.rt.dtype, device=x.device)
        if self.taps > 1 and ctx.num_decode == ctx.num_seqs:            # every request brings one token
            K.causal_conv_single(u, self.w_conv, conv_state, ctx.token_seq, ctx.state_slots, c, bias_out=self.b_conv,
                                 activation="silu", tap_major=True)
        else:
            K.causal_conv(u, self.w_conv, conv_state, ctx.token_seq, ctx.seq_starts, ctx.state_slots, c,
                          bias_out=self.b_conv, activation="silu", tap_major=True)
            if self.taps > 1:
                K.conv_state_update(u, self.taps, conv_state, ctx.seq_starts, ctx.state_slots)
        low = linear(c, self.w_low, kernels=kn)                                   # [n, dt | B | C]
        dt = linear(low, self.w_dt, out_dtype=torch.float32, kernels=kn)
        y = torch.empty((n, I), dtype=self.rt.dtype, device=x.device)
        same = (c, z, low, self.b_col, self.c_col, dt, self.dt_bias, self.a2, self.skip, state, y, ctx.seq_starts, ctx.state_slots)
        nd = ctx.num_decode
        if nd > 0:
            K.selective_scan(*same, 0, nd, 1)
        if ctx.num_seqs > nd:
            rows = ctx.q_lens[nd:]
            K.selective_scan(*same, nd, ctx.num_seqs - nd, max(rows), K.selective_segment(rows, I, x.device))
        return linear(y, self.w_o, keep_split=True, kernels=kn)

    def native(self, program, view: CacheView) -> None:
        if type(self).forward is not Mamba1Mixer.forward:
            return super().native(program, view)
        from ..engine.program import ALWAYS, STREAM, Guard
        rt, I, taps, dev = self.rt, self.inner, self.taps, self.rt.device
        act, ab, N, T = program.act_code, program.act_bytes, program.N, program.T
        state = self._state(view)
        stride = int(state.stride(0))
        ssm = state[:, self.conv_floats:]
        program.keep(state, ssm, self.w_conv, self.b_conv, self.dt_bias, self.a2, self.skip)
        proj = emit_linear(program, program.x, N, self.w_in, rt.dtype, None, False, "mamba1.proj", "mamba1.in").tensor()
        c = program.buffer("mamba1.c", T * I * ab)
        portions = Guard.between(program.NP, 1) if taps > 1 else ALWAYS
        program.op("core", "ia_causal_conv", [proj, act, 2 * I, None, self.w_conv, self.b_conv, 1, c, act, I, state, stride,
                                              program.token_seq, program.seq_starts, program.state_slots, N, I, taps, 1,
                                              STREAM], portions)
        if taps > 1:
            program.op("core", "ia_conv_state_update", [proj, act, 2 * I, None, state, stride, program.seq_starts,
                                                        program.state_slots, program.B, I, taps, STREAM], portions)
            program.op("core", "ia_causal_conv_single", [proj, act, 2 * I, None, self.w_conv, self.b_conv, 1, c, act, I, state,
                                                         stride, program.token_seq, program.state_slots, N, I, taps, 1,
                                                         STREAM], ~portions)
        low = emit_linear(program, c, N, self.w_low, rt.dtype, None, False, "mamba1.low", "mamba1.x").tensor()
        dt = emit_linear(program, low, N, self.w_dt, torch.float32, None, False, "mamba1.dt", "mamba1.dtp").tensor()
        y = program.buffer("mamba1.y", T * I * ab)
        same = [c, act, I, proj.at(I * ab), 2 * I, low, self.row, self.b_col, self.c_col, dt, I, self.dt_bias, self.a2, self.skip,
                ssm, stride, y, I, program.seq_starts, program.state_slots]
        program.op("core", "ia_selective_scan", [*same, 0, program.ND, I, self.Ns, 1, 1, None, None, STREAM],
                   Guard.between(program.ND, 1))
        # a request holds a state slot, and a segment but a request's last so many rows: so many segments a step has at most
        most = T // K.SELECTIVE_SEGMENTS[0] + int(state.shape[0])
        records = program.buffer("mamba1.records", most * self.Ns * I * 4)
        sums = program.buffer("mamba1.sums", most * I * 4)
        longest = program.scalar("mamba1: rows of the longest portion", lambda ctx: max(ctx.q_lens[ctx.num_decode:], default=1))
        seg = program.scalar(("mamba1: rows of a segment", I),
                             lambda ctx: K.selective_segment(ctx.q_lens[ctx.num_decode:], I, dev))
        program.op("core", "ia_selective_scan", [*same, program.ND, program.NP, I, self.Ns, longest, seg, records, sums, STREAM],
                   Guard.between(program.NP, 1))
        program.pending = emit_linear(program, y, N, self.w_o, rt.dtype, None, True, "mamba1.out", "mamba1.o")


register_part("mixer", "mamba1", Mamba1Mixer)
