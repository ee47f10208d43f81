"""A linear recurrence with one real number of state a channel and a decay that the input sets
(``RealGatedRecurrenceSpec``).

    y = act(W_y h + b_y),  u = filter(W_x h + b_x)                 a short causal filter per channel, with a bias
    r = logistic(A_b u_b + ..), i = logistic(I_b u_b + ..)          block by block of the channels
    a = exp(-strength * r * softplus(lam)),  S <- a S + sqrt(1 - a^2) * i * u
    output  W_o (S * y)

W_y h | W_x h is one product in the compute dtype and u is rounded to it as well; the square matrices' sums, the logistic
functions, the decay and its logarithm, the root, the products that enter S and S itself are 32-bit.  A request's state is
one 32-bit row [ S: channels | the filter's last taps - 1 inputs ]; the kernels find it through ``ctx.state_slots`` on the
device, so decode steps can be recorded.
"""
from __future__ import annotations

import torch

from ..kernels import ops
from .base import Mixer, StateNeed, StepContext, register_mixer, to_matrix, to_vector


class RealGatedRecurrence(Mixer):
    graph_safe = True
    can_store = True

    def __init__(self, spec, params, dtype, device):
        self.spec = spec
        E, C, B, K = spec.width, spec.channels, spec.blocks, spec.conv_taps
        self.channels, self.blocks, self.taps = C, B, K
        if B < 1 or C % B != 0:
            raise ValueError(f"{C} channels do not fall into {B} equal blocks")
        if not (1 <= K <= ops.CONV_MAX_TAPS):
            raise ValueError(f"a filter of {K} taps is outside 1..{ops.CONV_MAX_TAPS}")
        if spec.activation not in ops.ACTIVATIONS or spec.activation == "glu_capped":
            raise ValueError(f"unknown activation {spec.activation!r}")
        self.activation = spec.activation
        n = self.block = C // B

        def shaped(name, shape):
            t = params[name]
            if tuple(t.shape) != tuple(shape):
                raise ValueError(f"{name} is {list(t.shape)}, expected {list(shape)}")
            return t

        self.in_weight = to_matrix(shaped("in_weight", (2 * C, E)), dtype, device)        # y | x
        self.in_bias = to_vector(shaped("in_bias", (2 * C,)), dtype, device)
        self.conv_weight = to_vector(shaped("conv_weight", (C, K)), dtype, device)
        self.conv_bias = to_vector(shaped("conv_bias", (C,)), dtype, device)
        # the same for the serving form: 32-bit, a tap a row
        self.conv_rows = self.conv_weight.to(torch.float32).t().contiguous()
        self.conv_bias32 = self.conv_bias.to(torch.float32).contiguous()
        self.gate_weight = to_matrix(shaped("gate_weight", (B, 2 * n, n)), dtype, device)     # block by block: r's rows | i's
        self.gate_bias = shaped("gate_bias", (B, 2 * n)).to(device=device, dtype=torch.float32).contiguous()
        lam = shaped("lam", (C,)).to(dtype=torch.float64)
        self.rate = (-float(spec.decay_strength) * torch.nn.functional.softplus(lam)).to(device=device, dtype=torch.float32).contiguous()
        self.out_weight = to_matrix(shaped("out_weight", (E, C)), dtype, device)
        self.conv_off = C                            # where the filter's inputs start in a state row

    def kernel_units(self, dtype):
        return ("rglru",) if dtype == torch.bfloat16 and ops.rglru_block_fits(self.block) else ("rglru", "ssm")

    def cache_need(self):
        return StateNeed(self.channels * self.taps)

    normed_into = True

    def forward_normed(self, ctx: StepContext, norm, x: torch.Tensor, call, into=None) -> bool:
        """Small steps of a layer without a feed-forward beside it: the layer norm in front and the first product in one
        kernel."""
        N, ln = x.shape[0], norm.fusable_params()
        if ln is None or not ops.can_fuse_ln(N, x, self.in_weight):
            return False
        yx = ctx.buf("rglru_in", N, 2 * self.channels, ctx.dtype)
        ops.linear_ln(x, None, N, ln[0], ln[1], ln[2], self.in_weight, self.in_bias, yx)
        self._recur(ctx, yx, x if into is None else into, call)
        return True

    def forward(self, ctx: StepContext, h: torch.Tensor, x: torch.Tensor, call) -> None:
        yx = ctx.buf("rglru_in", h.shape[0], 2 * self.channels, ctx.dtype)
        ops.linear(h, self.in_weight, self.in_bias, yx)
        self._recur(ctx, yx, x, call)

    def _recur(self, ctx: StepContext, yx: torch.Tensor, x: torch.Tensor, call) -> None:
        N, C, n = yx.shape[0], self.channels, self.block
        state = ctx.cache.state[call.cache]                          # [slots, C + (taps - 1) C]
        out = ctx.buf("rglru_out", N, C, ctx.dtype)
        if ops.rglru_serve_takes(yx, n):
            ops.rglru_serve(ctx, yx, self.conv_rows, self.conv_bias32, self.gate_weight, self.gate_bias, self.rate,
                            self.activation, state, out, write=call.write)
        else:
            u = ctx.buf("rglru_u", N, C, ctx.dtype)
            ops.conv_causal(ctx, yx[:, C:], state, self.conv_off, self.conv_weight, self.conv_bias, None, u)
            if call.write:
                ops.conv_state_update(ctx, yx[:, C:], state, self.conv_off, C, self.taps)
            raw = ctx.buf("rglru_gates", N, 2 * C, torch.float32)    # before the logistic functions, unrounded
            for b in range(self.blocks):
                ops.linear(u[:, b * n:(b + 1) * n], self.gate_weight[b], self.gate_bias[b], raw[:, 2 * b * n:2 * (b + 1) * n])
            ops.rglru_walk(ctx, u, raw, n, self.rate, yx[:, :C], self.activation, state, out, write=call.write)
        ops.linear(out, self.out_weight, None, x, accumulate=ctx.part_accumulate)


register_mixer("real_gated_recurrence", RealGatedRecurrence)
