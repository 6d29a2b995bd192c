"""A selective state-space mixer (Mamba-2's form): it keeps, per request, a matrix per head instead of keys and values.

One stacked product reads h: ``[z | x | B | C | dt]``.  x, B and C together pass a short causal convolution per channel
with a bias, and silu; ``dt <- softplus(dt + dt_bias)``, one number a head.  Per head, with the B and C of its group,
``S <- exp(-exp(A_log) dt) S + dt B x^T`` from S = 0 and ``y = S^T C + D x``.  The heads side by side are multiplied by
silu(z), every one of ``norm_groups`` equal parts is divided by its own root mean square, a weight multiplies the row,
and the output projection follows.

The products are in the storage type; their 32-bit sums go straight into the convolution, whose activated result is
rounded once to the storage type; everything from there to the norm's one rounding is 32-bit arithmetic in either storage
type.  The state (the matrices and the convolution's last
inputs) is one row of 32-bit numbers in the request's slot, zero when a request takes the slot; a step of any cut
continues from it.  Long portions in bfloat16 storage run as chunks of products on the matrix cores, with the same sums
in another order.
"""

from __future__ import annotations

import torch

from tokasaurus_amd.kernels import ops
from tokasaurus_amd.parts.base import BIAS, CONV, MIXERS, NORM_WEIGHT, VECTOR, Mixer, StateNeed, StepContext, TensorSpec
from tokasaurus_amd.parts.linear import Linear, Placer


@MIXERS.register("mamba2")
class Mamba2(Mixer):
    def __init__(self, hidden_size: int, num_heads: int, value_dim: int, state_dim: int, groups: int, taps: int, norm_groups: int,
                 norm_eps: float, names: dict[str, str]):
        """``names``: checkpoint names under in ([2 inner + 2 groups * state_dim + heads, hidden] with inner = heads *
        value_dim: rows z, x, B, C, dt), conv ([inner + 2 groups * state_dim, taps], the last column is the current
        token's), conv_bias, dt_bias, A_log, D ([heads]), norm ([inner]), o ([hidden, inner])."""
        if num_heads % groups:
            raise ValueError(f"{num_heads} heads are no multiple of {groups} groups that share B and C")
        self.num_heads, self.value_dim, self.state_dim = int(num_heads), int(value_dim), int(state_dim)
        self.groups, self.taps, self.norm_groups = int(groups), int(taps), int(norm_groups)
        self.norm_eps = float(norm_eps)
        self.names = dict(names)
        self.inner = self.num_heads * self.value_dim
        self.channels = self.inner + 2 * self.groups * self.state_dim
        if self.inner % self.norm_groups:
            raise ValueError(f"{self.inner} channels do not form {self.norm_groups} equal parts")
        self.inp = Linear(hidden_size, [names["in"]], [self.inner + self.channels + self.num_heads])
        self.out = Linear(self.inner, [names["o"]], [hidden_size])
        self.conv_w = self.conv_b = self.dt_bias = self.a_log = self.d_skip = self.norm_w = None

    def tensor_specs(self) -> list[TensorSpec]:
        n, H = self.names, self.num_heads
        return self.inp.tensor_specs() + self.out.tensor_specs() + [
            TensorSpec(n["conv"], (self.channels, self.taps), CONV), TensorSpec(n["conv_bias"], (self.channels,), BIAS),
            TensorSpec(n["dt_bias"], (H,), VECTOR), TensorSpec(n["A_log"], (H,), VECTOR), TensorSpec(n["D"], (H,), VECTOR),
            TensorSpec(n["norm"], (self.inner,), NORM_WEIGHT)]

    def state_need(self) -> StateNeed:
        return StateNeed((ops.state_space_sizes(self.num_heads, self.groups, self.state_dim, self.value_dim, self.taps)[0],), torch.float32)

    def load(self, tensors: dict[str, torch.Tensor], placer: Placer) -> None:
        self.inp.load(tensors, placer)
        self.out.load(tensors, placer)
        n = self.names

        def f32(name: str) -> torch.Tensor:
            return placer.place(("vector_f32", name), lambda: tensors[name].to(torch.float32).contiguous().to(placer.device))

        # tap by tap, [taps, channels]: neighbouring channels' weights of one tap lie together
        self.conv_w = placer.place(("conv_f32_by_tap", n["conv"]), lambda: tensors[n["conv"]].to(torch.float32).t().contiguous().to(placer.device))
        self.conv_b, self.dt_bias, self.a_log = f32(n["conv_bias"]), f32(n["dt_bias"]), f32(n["A_log"])
        self.d_skip, self.norm_w = f32(n["D"]), f32(n["norm"])

    def _run(self, h: torch.Tensor, ctx: StepContext, state: torch.Tensor, rows: torch.Tensor | None) -> torch.Tensor:
        assert state is not None, "a state-space mixer keeps its state in the request's slot"
        proj = self.inp(h, out_f32=True)
        y = ops.state_space(proj, self.inner, self.inner + self.channels, self.conv_w, self.conv_b, self.a_log, self.dt_bias,
                            self.d_skip, state, ctx.q_start, ctx.token_req, ctx.slots, ctx.positions, self.num_heads, self.groups,
                            self.state_dim, self.value_dim, longest=ctx.max_q_len, storage=h.dtype)
        out = ops.gate_group_norm(y, proj[:, : self.inner], self.norm_w, self.norm_eps, self.norm_groups, h.dtype)
        return out if rows is None else ops.gather_rows(out, rows)

    def mix(self, h, ctx, cache, state, rows, out_f32: bool = False):
        return self.out(self._run(h, ctx, state, rows), out_f32=out_f32)

    def forward(self, h, residual, ctx, cache, state, rows):
        return self.out(self._run(h, ctx, state, rows), residual=residual)
