"""Linear attention with a decay: mixers that keep, per request, a matrix per head instead of keys and
values.  Per head ``S_t = diag(a_t) S_(t-1) + k_t v_t^T`` and ``o_t = S_t^T q_t``, from ``S = 0``.

``lightning_attention``: q, k and v are projections through silu; a_t is one constant a head (``decays``); the
heads' results side by side pass one RMS norm with a plain weight, are multiplied by sigmoid(W_g h) and projected.

``hgrn2``: q is a projection through silu and v a plain projection; a forget gate per head and row of S,
``f = low + (1 - low) * sigmoid(W_f h + b)`` with a learned lower bound ``low``, decays the state (a_t = f) and its
complement is what is written (k_t = 1 - f); every head's result passes an RMS norm over its own elements with
one weight for all heads, and the output projection follows.

``gated_linear_attention``: q (scaled), k and v are plain projections; a_t is a decay per head and row of S,
``sigmoid(W_a2 (W_a1 h) + b)^(1 / tau)``; every head's result passes an RMS norm over its own elements with one weight for
all heads, the row is multiplied by silu(W_g h) and projected.

``matrix_memory`` (xLSTM's mLSTM): q (scaled), k and v are plain projections; two numbers a head and token, an input gate
and a forget gate kept as logarithms, a_t = exp(f) and exp(i) k_t v_t^T is written, both relative to a running maximum that
is part of the state, as is the sum n of the written keys; the read-out is divided by max(|n . q|, exp(-maximum)) + 1e-6,
every head's result by its root mean square; a weight multiplies the row, then sigmoid(W_g h), and it is projected.

Everything that reads h is one stacked product whose 32-bit sums go straight into the recurrence: activations,
gates, the state, the read-out and the norms are 32-bit arithmetic in either storage type.  The state is one
row of 32-bit numbers in the request's slot, zero when a request takes the slot; a step of any cut continues
from it with the sums of the token-by-token recurrence.

A mixer here also gives its result in front of the output projection (``inner_rows``), with a factor, into a
view that the caller names: for a mixer that runs two side by side through one stacked output product.
"""

from __future__ import annotations

import torch

from tokasaurus_amd.kernels import ops
from tokasaurus_amd.kernels.upload import upload
from tokasaurus_amd.parts.base import BIAS, MATRIX, MIXERS, NORM_WEIGHT, UNIT_INTERVAL, VECTOR, Mixer, StateNeed, StepContext, TensorSpec
from tokasaurus_amd.parts.linear import Linear, Placer


def chunk_plan(ctx: StepContext, memory: bool, key_dim: int) -> "ops.ChunkPlan | None":
    """The step's rows in chunks, made once a step and shared by the layers; None for steps of short portions."""
    if not ops.linear_attention_takes_chunks(memory, key_dim, ctx.max_q_len):
        return None
    plan = ctx.extras.get("chunk_plan")
    if plan is None:
        size = ops.linear_attention_chunk_tokens()
        req, row0, first = [], [], [0]
        for r in range(ctx.num_requests):
            rows = range(ctx.host_q_start[r], ctx.host_q_start[r + 1], size)
            req += [r] * len(rows)
            row0 += rows
            first.append(len(req))
        dev, n = upload(req + row0 + first, torch.int32, ctx.device), len(req)
        plan = ctx.extras["chunk_plan"] = ops.ChunkPlan(dev[:n], dev[n : 2 * n], dev[2 * n :])
    return plan


class _LinearAttention(Mixer):
    """What the forms share: the state, the output projection, and how a result leaves."""

    hidden_size: int
    num_heads: int
    key_dim: int
    value_dim: int
    out: Linear
    keeps_memory = False  # the state is the matrix memory's

    @property
    def inner_size(self) -> int:
        return self.num_heads * self.value_dim

    def state_need(self) -> StateNeed:
        return StateNeed((ops.linear_attention_state_words(self.num_heads, self.key_dim, self.value_dim, self.keeps_memory),), torch.float32)

    def inner_rows(self, h, ctx: StepContext, cache, state, out: torch.Tensor | None = None, scale: float = 1.0) -> torch.Tensor:
        raise NotImplementedError

    def mix(self, h, ctx, cache, state, rows, out_f32: bool = False):
        y = self.inner_rows(h, ctx, cache, state)
        return self.out(y if rows is None else ops.gather_rows(y, rows), out_f32=out_f32)

    def forward(self, h, residual, ctx, cache, state, rows):
        y = self.inner_rows(h, ctx, cache, state)
        return self.out(y if rows is None else ops.gather_rows(y, rows), residual=residual)


@MIXERS.register("lightning_attention")
class LightningAttention(_LinearAttention):
    def __init__(self, hidden_size: int, num_heads: int, key_dim: int, value_dim: int, decays: list[float], norm_eps: float,
                 names: dict[str, str]):
        """``decays``: one number a head.  ``names``: checkpoint names under q, k ([heads * key_dim, hidden]), v, g
        ([heads * value_dim, hidden]), norm ([heads * value_dim]) and o ([hidden, heads * value_dim])."""
        self.hidden_size, self.num_heads = hidden_size, int(num_heads)
        self.key_dim, self.value_dim = int(key_dim), int(value_dim)
        self.decays = [float(a) for a in decays]
        if len(self.decays) != self.num_heads:
            raise ValueError(f"{len(self.decays)} decays for {self.num_heads} heads")
        self.norm_eps = float(norm_eps)
        self.names = dict(names)
        qk, v = self.num_heads * self.key_dim, self.num_heads * self.value_dim
        self.inp = Linear(hidden_size, [names[x] for x in ("q", "k", "v", "g")], [qk, qk, v, v])
        self.out = Linear(v, [names["o"]], [hidden_size])
        self.decay: torch.Tensor | None = None
        self.norm_w: torch.Tensor | None = None

    def tensor_specs(self) -> list[TensorSpec]:
        return self.inp.tensor_specs() + self.out.tensor_specs() + [TensorSpec(self.names["norm"], (self.inner_size,), NORM_WEIGHT)]

    def load(self, tensors: dict[str, torch.Tensor], placer: Placer) -> None:
        self.inp.load(tensors, placer)
        self.out.load(tensors, placer)
        n = self.names["norm"]
        self.norm_w = placer.place(("vector_f32", n), lambda: tensors[n].to(torch.float32).contiguous().to(placer.device))
        self.decay = placer.place(("constant_f32", *self.decays), lambda: torch.tensor(
            self.decays, dtype=torch.float64).to(torch.float32).to(placer.device))

    def inner_rows(self, h, ctx, cache, state, out=None, scale: float = 1.0):
        assert state is not None, "linear attention keeps its state in the request's slot"
        H, dk, dv = self.num_heads, self.key_dim, self.value_dim
        proj = self.inp(h, out_f32=True)
        o = ops.linear_attention(proj, 0, H * dk, 2 * H * dk, state, ctx.q_start, ctx.slots, H, dk, dv, decay=self.decay, longest=ctx.max_q_len)
        gate = proj[:, 2 * H * dk + H * dv :]
        return ops.group_norm_gate(o, self.norm_w, self.norm_eps, 1, h.dtype, gate=gate, scale=scale, out=out)


@MIXERS.register("hgrn2")
class HGRN2(_LinearAttention):
    def __init__(self, hidden_size: int, num_heads: int, key_dim: int, value_dim: int, norm_eps: float, names: dict[str, str]):
        """``names``: checkpoint names under q, f ([heads * key_dim, hidden]), f_bias, lower ([heads * key_dim]), v
        ([heads * value_dim, hidden]), norm ([value_dim], shared by the heads) and o ([hidden, heads * value_dim])."""
        self.hidden_size, self.num_heads = hidden_size, int(num_heads)
        self.key_dim, self.value_dim = int(key_dim), int(value_dim)
        self.norm_eps = float(norm_eps)
        self.names = dict(names)
        qk, v = self.num_heads * self.key_dim, self.num_heads * self.value_dim
        self.inp = Linear(hidden_size, [names[x] for x in ("q", "f", "v")], [qk, qk, v])
        self.out = Linear(v, [names["o"]], [hidden_size])
        self.f_bias = self.f_low = self.norm_w = None

    def tensor_specs(self) -> list[TensorSpec]:
        qk = self.num_heads * self.key_dim
        return self.inp.tensor_specs() + self.out.tensor_specs() + [
            TensorSpec(self.names["f_bias"], (qk,), BIAS), TensorSpec(self.names["lower"], (qk,), UNIT_INTERVAL),
            TensorSpec(self.names["norm"], (self.value_dim,), NORM_WEIGHT)]

    def load(self, tensors: dict[str, torch.Tensor], placer: Placer) -> None:
        self.inp.load(tensors, placer)
        self.out.load(tensors, placer)

        def f32(name: str) -> torch.Tensor:
            return placer.place(("vector_f32", name), lambda: tensors[name].to(torch.float32).contiguous().to(placer.device))

        self.f_bias, self.f_low, self.norm_w = f32(self.names["f_bias"]), f32(self.names["lower"]), f32(self.names["norm"])

    def inner_rows(self, h, ctx, cache, state, out=None, scale: float = 1.0):
        assert state is not None, "linear attention keeps its state in the request's slot"
        H, dk, dv = self.num_heads, self.key_dim, self.value_dim
        proj = self.inp(h, out_f32=True)
        o = ops.linear_attention(proj, 0, H * dk, 2 * H * dk, state, ctx.q_start, ctx.slots, H, dk, dv,
                                 forget_bias=self.f_bias, forget_low=self.f_low, longest=ctx.max_q_len)
        return ops.group_norm_gate(o, self.norm_w, self.norm_eps, H, h.dtype, scale=scale, out=out)


@MIXERS.register("gated_linear_attention")
class GatedLinearAttention(_LinearAttention):
    def __init__(self, hidden_size: int, num_heads: int, key_dim: int, value_dim: int, rank: int, tau: float, norm_eps: float,
                 names: dict[str, str], q_scale: float = 1.0):
        """``names``: checkpoint names under q, k ([heads * key_dim, hidden]), v, g ([heads * value_dim, hidden]), a1 ([rank,
        hidden]), a2 ([heads * key_dim, rank]), a2_bias ([heads * key_dim]), norm ([value_dim], shared by the heads) and o
        ([hidden, heads * value_dim])."""
        self.hidden_size, self.num_heads = hidden_size, int(num_heads)
        self.key_dim, self.value_dim, self.rank = int(key_dim), int(value_dim), int(rank)
        self.tau, self.norm_eps, self.q_scale = float(tau), float(norm_eps), float(q_scale)
        if not self.tau > 0:
            raise ValueError("the decays' tau must be positive")
        self.names = dict(names)
        qk, v = self.num_heads * self.key_dim, self.num_heads * self.value_dim
        self.inp = Linear(hidden_size, [names[x] for x in ("q", "k", "v", "g", "a1")], [qk, qk, v, v, self.rank])
        self.out = Linear(v, [names["o"]], [hidden_size])
        self.low_up = self.low_bias = self.norm_w = None

    def tensor_specs(self) -> list[TensorSpec]:
        qk, n = self.num_heads * self.key_dim, self.names
        return self.inp.tensor_specs() + self.out.tensor_specs() + [
            TensorSpec(n["a2"], (qk, self.rank), MATRIX), TensorSpec(n["a2_bias"], (qk,), BIAS),
            TensorSpec(n["norm"], (self.value_dim,), NORM_WEIGHT)]

    def load(self, tensors: dict[str, torch.Tensor], placer: Placer) -> None:
        self.inp.load(tensors, placer)
        self.out.load(tensors, placer)
        n = self.names

        def f32(name: str) -> torch.Tensor:
            return placer.place(("vector_f32", name), lambda: tensors[name].to(torch.float32).contiguous().to(placer.device))

        # [rank, channels]: neighbouring channels' weights lie together
        self.low_up = placer.place(("transposed_f32", n["a2"]), lambda: tensors[n["a2"]].to(torch.float32).t().contiguous().to(placer.device))
        self.low_bias, self.norm_w = f32(n["a2_bias"]), f32(n["norm"])

    def inner_rows(self, h, ctx, cache, state, out=None, scale: float = 1.0):
        assert state is not None, "linear attention keeps its state in the request's slot"
        H, dk, dv = self.num_heads, self.key_dim, self.value_dim
        qk, v = H * dk, H * dv
        proj = self.inp(h, out_f32=True)
        o = ops.gated_linear_attention(proj, 0, qk, 2 * qk, 2 * (qk + v), self.low_up, self.low_bias, self.tau, self.q_scale, state,
                                       ctx.q_start, ctx.slots, H, dk, dv, longest=ctx.max_q_len,
                                       chunks=chunk_plan(ctx, False, dk))
        return ops.group_norm_gate(o, self.norm_w, self.norm_eps, H, h.dtype, gate=proj[:, 2 * qk + v : 2 * (qk + v)], scale=scale, out=out,
                                   silu_gate=True)


@MIXERS.register("matrix_memory")
class MatrixMemory(_LinearAttention):
    keeps_memory = True

    def __init__(self, hidden_size: int, num_heads: int, key_dim: int, value_dim: int, gate_cap: float, norm_eps: float,
                 names: dict[str, str], q_scale: float = 1.0):
        """``gate_cap``: both gates' sums pass cap * tanh(. / cap).  ``names``: checkpoint names under q, k ([heads * key_dim,
        hidden]), v, g ([heads * value_dim, hidden]), i, f ([heads, hidden]), i_bias, f_bias ([heads]), norm ([heads *
        value_dim]) and o ([hidden, heads * value_dim])."""
        self.hidden_size, self.num_heads = hidden_size, int(num_heads)
        self.key_dim, self.value_dim = int(key_dim), int(value_dim)
        self.gate_cap, self.norm_eps, self.q_scale = float(gate_cap), float(norm_eps), float(q_scale)
        if not self.gate_cap > 0:
            raise ValueError("the gates' cap must be positive")
        self.names = dict(names)
        qk, v, H = self.num_heads * self.key_dim, self.num_heads * self.value_dim, self.num_heads
        self.inp = Linear(hidden_size, [names[x] for x in ("q", "k", "v", "g", "i", "f")], [qk, qk, v, v, H, H])
        self.out = Linear(v, [names["o"]], [hidden_size])
        self.i_bias = self.f_bias = self.norm_w = None

    def tensor_specs(self) -> list[TensorSpec]:
        n, H = self.names, self.num_heads
        return self.inp.tensor_specs() + self.out.tensor_specs() + [
            TensorSpec(n["i_bias"], (H,), VECTOR), TensorSpec(n["f_bias"], (H,), VECTOR), TensorSpec(n["norm"], (self.inner_size,), NORM_WEIGHT)]

    def load(self, tensors: dict[str, torch.Tensor], placer: Placer) -> None:
        self.inp.load(tensors, placer)
        self.out.load(tensors, placer)

        def f32(name: str) -> torch.Tensor:
            return placer.place(("vector_f32", name), lambda: tensors[name].to(torch.float32).contiguous().to(placer.device))

        self.i_bias, self.f_bias, self.norm_w = f32(self.names["i_bias"]), f32(self.names["f_bias"]), f32(self.names["norm"])

    def inner_rows(self, h, ctx, cache, state, out=None, scale: float = 1.0):
        assert state is not None, "a matrix memory keeps its state in the request's slot"
        H, dk, dv = self.num_heads, self.key_dim, self.value_dim
        qk, v = H * dk, H * dv
        proj = self.inp(h, out_f32=True)
        o, floor = ops.matrix_memory(proj, 0, qk, 2 * qk, 2 * (qk + v), 2 * (qk + v) + H, self.i_bias, self.f_bias, self.gate_cap,
                                     self.q_scale, state, ctx.q_start, ctx.slots, ctx.positions, H, dk, dv, longest=ctx.max_q_len,
                                     chunks=chunk_plan(ctx, True, dk))
        return ops.group_norm_gate(o, self.norm_w, self.norm_eps, H, h.dtype, gate=proj[:, 2 * qk + v : 2 * (qk + v)], scale=scale, out=out,
                                   size=dv, floor=floor)
