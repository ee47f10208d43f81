"""Gated linear attention as a mixer (``GatedLinearSpec``): linear attention whose decay the input sets.

Per head a matrix S [head_dim, v_head_dim] is carried from token to token in 32-bit:

    S <- diag(a) S + k v^T      a = logistic(z)^(1 / tau), one a key channel (a row of S); z = W_a2 (W_a1 h) + b
    o  = S^T q                  (sees the token's own write; q times head_dim^-1/2)

There is no softmax and no denominator.  Each head's o is divided by its root mean square, multiplied by a gain shared by
the heads and by the gate (SiLU of one more projection), and projected back.  What enters the recurrence besides q, k and
v is 32-bit: z as the unrounded sum of its product, the logarithm of the decay, its exponential, the state.  A request's
state is one 32-bit row [ S: heads x v_head_dim x head_dim ]; kernels find it through ``ctx.state_slots`` on the device,
so decode steps can be recorded.

Products of a step: [q | k | v | gate | the decay's low rank] in the compute dtype (one product), the low rank's second
factor (in bfloat16 serving inside the recurrence's kernels for ranks up to 32), and the output projection.
"""
from __future__ import annotations

import torch

from ..kernels import ops
from .base import Mixer, StateNeed, StepContext, register_mixer, to_matrix, to_vector


class GatedLinearAttention(Mixer):
    graph_safe = True
    can_store = True

    def __init__(self, spec, params, dtype, device):
        self.spec = spec
        E, H, D, Dv = spec.width, spec.n_heads, spec.head_dim, spec.v_head_dim
        self.H, self.D, self.Dv = H, D, Dv
        if not (1 <= D <= ops.GLA_MAX_DIM):
            raise ValueError(f"a key size of {D} is outside 1..{ops.GLA_MAX_DIM}")
        if not (float(spec.tau) > 0.0):
            raise ValueError(f"tau {spec.tau} must be positive")
        if spec.gate != "silu":
            raise ValueError(f"the gate of a gated linear mixer is 'silu', not {spec.gate!r}")
        self.eps, self.tau = float(spec.norm_eps), float(spec.tau)
        self.qk_cols, self.v_cols = H * D, H * Dv

        def shaped(name, shape):
            t = params[name]
            if t.dim() != len(shape) or any(e not in (-1, f) for e, f in zip(shape, t.shape)):
                raise ValueError(f"{name} is {list(t.shape)}, expected {list(shape)}")
            return t

        down = shaped("decay_down", (spec.decay_rank, E))
        self.rank = down.shape[0]                    # a rank that the spec leaves open is what the matrices share
        self.decay_up = to_matrix(shaped("decay_up", (self.qk_cols, self.rank)), dtype, device)
        self.decay_bias = shaped("decay_bias", (self.qk_cols,)).to(device=device, dtype=torch.float32).contiguous()
        self.in_weight = to_matrix(torch.cat([shaped("q_weight", (self.qk_cols, E)), shaped("k_weight", (self.qk_cols, E)),
                                              shaped("v_weight", (self.v_cols, E)), shaped("gate_weight", (self.v_cols, E)),
                                              down], 0), dtype, device)
        self.out_norm = to_vector(shaped("out_norm", (Dv,)), dtype, device)
        self.out_weight = to_matrix(shaped("out_weight", (E, self.v_cols)), dtype, device)
        self.q_scale = float(D) ** -0.5
        self.v_off, self.gate_off = 2 * self.qk_cols, 2 * self.qk_cols + self.v_cols
        self.low_off = self.gate_off + self.v_cols

    def kernel_units(self, dtype):
        serve = dtype == torch.bfloat16 and self.D % 4 == 0 and max(self.D, self.Dv) <= ops.GLA_SERVE_MAX_DIM
        return ("gla",) if serve else ("gla", "delta")

    def cache_need(self):
        return StateNeed(self.H * self.Dv * self.D)

    def forward(self, ctx: StepContext, h: torch.Tensor, x: torch.Tensor, call) -> None:
        N = h.shape[0]
        proj = ctx.buf("gla_in", N, self.in_weight.shape[0], ctx.dtype)
        ops.linear(h, self.in_weight, None, proj)
        state = ctx.cache.state[call.cache]
        y = ctx.buf("gla_y", N, self.v_cols, ctx.dtype)
        serve = ops.gla_serve_takes(proj, state, self.D, self.Dv)
        raw = None
        if not (serve and ops.gla_low_takes(self.rank, self.decay_up)):
            raw = ctx.buf("gla_decay", N, self.qk_cols, torch.float32)      # unrounded sums
            ops.linear(proj[:, self.low_off:self.low_off + self.rank], self.decay_up, None, raw)
        if serve:
            # the decays, the recurrence, the read-out's norm and the gate together
            ops.gla_serve(ctx, proj, 0, self.qk_cols, self.v_off, self.gate_off, self.low_off,
                          self.decay_up if raw is None else None, raw, self.decay_bias, self.tau, self.q_scale, self.out_norm,
                          self.eps, state, y, self.H, self.D, self.Dv, write=call.write)
        else:
            o = ctx.buf("gla_o", N, self.v_cols, torch.float32)
            ops.gla_walk(ctx, proj, 0, self.qk_cols, self.v_off, raw, self.decay_bias, self.tau, self.q_scale, state, o,
                         self.H, self.D, self.Dv, write=call.write)
            ops.delta_gate_norm(o, proj[:, self.gate_off:self.gate_off + self.v_cols], self.out_norm, self.eps, "silu",
                                self.H, self.Dv, y)
        if ctx.debug_hook is not None:
            ctx.emit(call.layer, "attention_value", y)
        ops.linear(y, self.out_weight, None, x, accumulate=ctx.part_accumulate)


register_mixer("gated_linear", GatedLinearAttention)
