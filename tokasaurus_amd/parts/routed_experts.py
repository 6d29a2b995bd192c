"""A feed-forward made of many small gated experts of which every token uses a few.

The router is 32-bit arithmetic: logits ``W_router h`` over the routed experts and the identity
experts together, ``s = softmax(logits)`` or (``scores="sigmoid"``) each its own logit's sigmoid; the choice is made by
``s + correction`` (a learned vector that moves the choice and not the weight) or, without one, by ``s``; the experts form ``groups`` equal groups of
neighbours, a group's mark is its largest choice score, and only experts of the ``keep`` groups
with the largest marks can be chosen; the ``top`` largest choice scores win and the chosen experts'
``s`` are their weights, as they are or (``normalize_scale``) divided by their sum (+ 1e-20) and multiplied by a
constant.  A weight multiplies its expert's output or (``weights_on_input``) what the expert reads.  A routed expert is ``W_down (silu(W_gate h) * (W_up h))``;
the last ``identity`` router outputs have no tensors, their output is ``h`` itself.  A shared
expert of the same form may run for every token; its output is multiplied by
``sigmoid(w_sg . h)``, one number a token, where the checkpoint has such a gate, and added.

Or there is no router at all (``table_experts``): a table of integers gives each token id its experts, in equal parts.  The
choice then rests on the step's token ids alone and is looked up once a step for all layers.  An expert's activation may be the
form with clamps, ``g sigmoid(alpha g) (u + 1)`` of ``g = min(gate, limit)`` and ``u = clamp(up, -limit, limit)``.

One kernel routes (and computes the shared expert's gate); the experts' products run pair by
pair (token, chosen expert), each a function of its own token only, and are summed per token
in the order of the choice: a token's result does not depend on what else is in the batch.
"""

from __future__ import annotations

import torch

from tokasaurus_amd.kernels import ops
from tokasaurus_amd.parts.base import FEED_FORWARDS, INT_TABLE, MATRIX, SMALL_VECTOR, FeedForward, StepContext, TensorSpec
from tokasaurus_amd.parts.linear import Linear, Placer


class _Experts(FeedForward):
    """The experts' matrices, one tensor for all experts of a layer."""

    hidden_size: int
    expert_size: int
    num_experts: int
    names: dict[str, str]
    w_gate_up: torch.Tensor | None = None  # [experts, gate rows | up rows, hidden]
    w_down: torch.Tensor | None = None  # [experts, hidden, expert_size]

    def _expert(self, e: int, which: str) -> str:
        return f"{self.names['expert'].format(e=e)}.{which}"

    def _expert_specs(self) -> list[TensorSpec]:
        W, F = self.hidden_size, self.expert_size
        return [TensorSpec(self._expert(e, which), shape, MATRIX) for e in range(self.num_experts)
                for which, shape in (("gate", (F, W)), ("up", (F, W)), ("down", (W, F)))]

    def _load_experts(self, tensors: dict[str, torch.Tensor], placer: Placer) -> None:
        n, E = self.names["expert"], range(self.num_experts)
        self.w_gate_up = placer.place(("experts_gate_up", n), lambda: torch.stack(
            [torch.cat([tensors[self._expert(e, "gate")], tensors[self._expert(e, "up")]], dim=0) for e in E]).to(
                placer.dtype).contiguous().to(placer.device))
        self.w_down = placer.place(("experts_down", n), lambda: torch.stack([tensors[self._expert(e, "down")] for e in E]).to(
            placer.dtype).contiguous().to(placer.device))


@FEED_FORWARDS.register("routed_experts")
class RoutedExperts(_Experts):
    def __init__(self, hidden_size: int, expert_size: int, num_experts: int, top: int, names: dict[str, str],
                 identity: int = 0, groups: int = 1, keep: int = 1, shared_size: int | None = None,
                 normalize_scale: float | None = None, scores: str = "softmax", weights_on_input: bool = False):
        """``names``: ``router`` ([experts + identity, hidden]), optionally ``correction`` ([experts + identity]),
        ``expert``: a pattern with ``{e}`` for the expert's number that gives the prefix of its
        ``.gate``, ``.up`` ([expert_size, hidden]) and ``.down`` ([hidden, expert_size]); with a
        shared expert also ``shared`` (the prefix of its three matrices) and, where it has a gate,
        ``shared_gate`` ([1, hidden]).  ``normalize_scale``: the chosen experts' weights are divided by their sum
        and multiplied by this number.  ``scores``: "softmax" or "sigmoid".  ``weights_on_input``: the output is the
        sum of expert(weight * h)."""
        if scores not in ("softmax", "sigmoid"):
            raise ValueError(f"a router's scores are softmax or sigmoid, not {scores!r}")
        self.sigmoid_scores, self.weights_on_input = scores == "sigmoid", bool(weights_on_input)
        self.normalize_scale = float(normalize_scale) if normalize_scale else None
        self.hidden_size, self.expert_size = hidden_size, int(expert_size)
        self.num_experts, self.top, self.identity = int(num_experts), int(top), int(identity)
        self.groups, self.keep = int(groups), int(keep)
        self.n_all = self.num_experts + self.identity
        if self.n_all % self.groups or not 0 < self.keep <= self.groups or not 0 < self.top <= self.n_all:
            raise ValueError(f"{self.n_all} experts in {self.groups} groups, {self.keep} kept, {self.top} chosen")
        self.names = dict(names)
        self.shared_size = int(shared_size) if shared_size else None
        self.shared_gate_up = self.shared_down = None
        if self.shared_size:
            sp = names["shared"]
            self.shared_gate_up = Linear(hidden_size, [f"{sp}.gate", f"{sp}.up"], [self.shared_size] * 2)
            self.shared_down = Linear(self.shared_size, [f"{sp}.down"], [hidden_size])
        self.router = self.correction = self.shared_gate = None

    def tensor_specs(self) -> list[TensorSpec]:
        W = self.hidden_size
        specs = [TensorSpec(self.names["router"], (self.n_all, W), MATRIX)]
        if self.names.get("correction"):
            specs.append(TensorSpec(self.names["correction"], (self.n_all,), SMALL_VECTOR))
        specs += self._expert_specs()
        if self.shared_size:
            specs += self.shared_gate_up.tensor_specs() + self.shared_down.tensor_specs()
            if self.names.get("shared_gate"):
                specs.append(TensorSpec(self.names["shared_gate"], (1, W), MATRIX))
        return specs

    def load(self, tensors: dict[str, torch.Tensor], placer: Placer) -> None:
        n = self.names

        def place(key, make):
            return placer.place(key, lambda: make().contiguous().to(placer.device))

        self.router = place(("row_major", n["router"]), lambda: tensors[n["router"]].to(placer.dtype))
        if n.get("correction"):
            self.correction = place(("vector_f32", n["correction"]), lambda: tensors[n["correction"]].to(torch.float32))
        self._load_experts(tensors, placer)
        if self.shared_size:
            self.shared_gate_up.load(tensors, placer)
            self.shared_down.load(tensors, placer)
            if n.get("shared_gate"):
                self.shared_gate = place(("row_major", n["shared_gate"]), lambda: tensors[n["shared_gate"]].to(placer.dtype).reshape(-1))

    def transform(self, h: torch.Tensor, out_f32: bool = False) -> torch.Tensor:
        ids, weights, gate = ops.expert_route(h, self.router, self.correction, self.groups, self.keep, self.top, self.shared_gate,
                                              normalize_scale=self.normalize_scale,
                                              unit_gate=bool(self.shared_size) and self.shared_gate is None,
                                              sigmoid_scores=self.sigmoid_scores)
        shared = self.shared_down(self.shared_gate_up(h, swiglu=True), out_f32=True) if self.shared_size else None
        y = ops.expert_mix(h, self.w_gate_up, self.w_down, ids, weights, shared, gate, weights_on_input=self.weights_on_input)
        return y if out_f32 else y.to(h.dtype)

    def forward(self, h: torch.Tensor, residual: torch.Tensor):
        return ops.add(self.transform(h), residual.contiguous())


class TokenTables:
    """The tables of a model's layers whose experts go by token id: they are read once a step, for all layers, in front
    of the embedding, and the choices sorted by expert there too where the layers' products want that."""

    KEY = "experts_by_token"  # in ``StepContext.extras``: per table the step's ids [tokens, top] and, or None, their sorted pairs

    def __init__(self):
        self.layers: list[TableExperts] = []
        self._ready: "ops.ExpertTables | None" = None

    def add(self, layer: "TableExperts") -> int:
        self.layers.append(layer)
        self._ready = None
        return len(self.layers) - 1

    def __call__(self, ctx: StepContext) -> None:
        if self._ready is None:
            self._ready = ops.ExpertTables([x.table for x in self.layers])
        ids = ops.expert_lookup(ctx.token_ids, ctx.last_token, self._ready)
        tiled = [i for i, x in enumerate(self.layers) if ops.experts_go_in_tiles(ctx.num_tokens, ctx.dtype, x.hidden_size, x.expert_size)]
        made = dict(zip(tiled, ops.expert_sort([(ids[i], self.layers[i].num_experts) for i in tiled]))) if tiled else {}
        ctx.extras[self.KEY] = [(x, made.get(i)) for i, x in enumerate(ids)]


@FEED_FORWARDS.register("table_experts")
class TableExperts(_Experts):
    reads_tokens = True

    def __init__(self, hidden_size: int, vocab_size: int, expert_size: int, num_experts: int, top: int, names: dict[str, str],
                 glu: tuple[float, float] | None = None, shared: dict | None = None):
        """``names``: ``table`` (integers [vocab_size, top], the entries of a row differ) and ``expert`` as in
        ``routed_experts``.  ``glu``: (limit, alpha) of the activation with clamps (None: silu)."""
        self.hidden_size, self.vocab_size, self.expert_size = hidden_size, int(vocab_size), int(expert_size)
        self.num_experts, self.top = int(num_experts), int(top)
        if not 0 < self.top <= self.num_experts:
            raise ValueError(f"{self.top} of {self.num_experts} experts")
        self.names = dict(names)
        self.glu = tuple(float(x) for x in glu) if glu else None
        shared = shared if shared is not None else {}
        if "token_tables" not in shared:
            shared["token_tables"] = TokenTables()
            shared.setdefault("step_starts", []).append(shared["token_tables"])
        self.tables: TokenTables = shared["token_tables"]
        self.table: torch.Tensor | None = None
        self.index: int | None = None

    def tensor_specs(self) -> list[TensorSpec]:
        return [TensorSpec(self.names["table"], (self.vocab_size, self.top), INT_TABLE, below=self.num_experts), *self._expert_specs()]

    def load(self, tensors: dict[str, torch.Tensor], placer: Placer) -> None:
        self._load_experts(tensors, placer)
        name = self.names["table"]
        self.table = placer.place(("int_table", name), lambda: tensors[name].to(torch.int32).contiguous().to(placer.device))
        self.index = self.tables.add(self)

    def transform(self, h: torch.Tensor, out_f32: bool = False, ctx: StepContext | None = None, rows: torch.Tensor | None = None):
        ids, pairs = ctx.extras[TokenTables.KEY][self.index]
        if rows is not None:
            ids, pairs = ids.index_select(0, rows), None
        y = ops.expert_mix(h, self.w_gate_up, self.w_down, ids, None, glu=self.glu, pairs=pairs)
        return y if out_f32 else y.to(h.dtype)

    def forward(self, h: torch.Tensor, residual: torch.Tensor, ctx: StepContext | None = None, rows: torch.Tensor | None = None):
        return ops.add(self.transform(h, ctx=ctx, rows=rows), residual.contiguous())
