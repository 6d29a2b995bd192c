"""The configuration of a Tefavik model, read from its ``config.json``.

The file lists the layers one by one; every size and every constant that may differ between
two models of the design is taken from it.  Keys:

    architecture: "Tefavik"       vocab, width       norm.eps
    loop: absent or null | {start, stop, times}   layers start .. stop-1 run ``times`` times in a row
    layers[i].type: "gla" | "parallel"
    layers[i].mlp: null | {"kind": "moe", "expert": {ff, limit}, "router": {experts, top}}
    gla mixer:              heads, dim, vdim, tau
    parallel mixer, left:   heads, kv_heads, dim, vdim, scale, softcap (null: none), rot: {base, dims} | null,
                            mask: {size} | null (a query sees its own chunk of so many positions; null: all before it)
    parallel mixer, right:  heads, dim, vdim, gate_cap

The inner size of a gla layer's decay projections is the checkpoint's (``with_tensor_shapes``).
"""

from __future__ import annotations

from dataclasses import dataclass, replace
from typing import Any

from tokasaurus_amd.config.kupuzen_config import _need
from tokasaurus_amd.config.model_config import ConfigError
from tokasaurus_amd.config.taborax_config import Loop


@dataclass(frozen=True)
class GatedLinearLayer:
    heads: int
    dim: int
    vdim: int
    tau: float
    rank: int | None = None  # inner size of the decays' two projections; None: not known yet


@dataclass(frozen=True)
class ChunkAttentionBranch:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    softcap: float | None
    chunk: int  # positions that see each other; 0: all
    rot_base: float | None
    rot_dims: int


@dataclass(frozen=True)
class MatrixMemoryBranch:
    heads: int
    dim: int
    vdim: int
    gate_cap: float


@dataclass(frozen=True)
class ParallelLayer:
    left: ChunkAttentionBranch
    right: MatrixMemoryBranch


@dataclass(frozen=True)
class TokenExperts:
    ff: int  # inner size of an expert
    limit: float
    experts: int
    top: int


@dataclass(frozen=True)
class TefavikLayer:
    kind: str
    mixer: GatedLinearLayer | ParallelLayer
    ff: TokenExperts | None


def _size(d: dict[str, Any], key: str, where: str) -> int:
    n = int(_need(d, key, where))
    if n <= 0:
        raise ConfigError(f"config.json: {where}.{key} must be positive, got {n}")
    return n


def _positive(d: dict[str, Any], key: str, where: str) -> float:
    x = float(_need(d, key, where))
    if not x > 0:
        raise ConfigError(f"config.json: {where}.{key} must be positive, got {x}")
    return x


def _attention_branch(m: dict[str, Any], where: str) -> ChunkAttentionBranch:
    rot, mask = m.get("rot"), m.get("mask")
    b = ChunkAttentionBranch(
        heads=_size(m, "heads", where), kv_heads=_size(m, "kv_heads", where), dim=_size(m, "dim", where), vdim=_size(m, "vdim", where),
        scale=float(_need(m, "scale", where)), softcap=_positive(m, "softcap", where) if m.get("softcap") is not None else None,
        chunk=_size(mask, "size", f"{where}.mask") if mask else 0,
        rot_base=float(_need(rot, "base", f"{where}.rot")) if rot else None, rot_dims=int(_need(rot, "dims", f"{where}.rot")) if rot else 0)
    if b.heads % b.kv_heads:
        raise ConfigError(f"config.json: {where}: {b.heads} heads are no multiple of {b.kv_heads} kv_heads")
    if rot and (b.rot_dims <= 0 or b.rot_dims % 2 or b.rot_dims > b.dim):
        raise ConfigError(f"config.json: {where}.rot.dims must be an even number of at most dim, got {b.rot_dims}")
    return b


def _experts(mlp: dict[str, Any] | None, where: str) -> TokenExperts | None:
    if mlp is None:
        return None
    if mlp.get("kind", "moe") != "moe":
        raise ConfigError(f"config.json: {where} has kind {mlp.get('kind')!r}; known: moe")
    e, r = _need(mlp, "expert", where), _need(mlp, "router", where)
    ff = TokenExperts(ff=_size(e, "ff", f"{where}.expert"), limit=_positive(e, "limit", f"{where}.expert"),
                      experts=_size(r, "experts", f"{where}.router"), top=_size(r, "top", f"{where}.router"))
    if ff.top > ff.experts:
        raise ConfigError(f"config.json: {where}: {ff.top} of {ff.experts} experts")
    return ff


@dataclass(frozen=True)
class TefavikConfig:
    vocab: int
    width: int
    norm_eps: float
    layers: tuple[TefavikLayer, ...]
    loop: Loop | None = None
    eos_token_ids: tuple[int, ...] = ()

    @classmethod
    def from_dict(cls, d: dict[str, Any]) -> "TefavikConfig":
        layers = []
        for i, layer in enumerate(_need(d, "layers", "the file")):
            where = f"layers[{i}]"
            kind = _need(layer, "type", where)
            m = _need(layer, "mixer", where)
            mw = f"{where}.mixer"
            if kind == "gla":
                mixer: Any = GatedLinearLayer(heads=_size(m, "heads", mw), dim=_size(m, "dim", mw), vdim=_size(m, "vdim", mw),
                                              tau=_positive(m, "tau", mw), rank=_size(m, "rank", mw) if m.get("rank") is not None else None)
            elif kind == "parallel":
                right, rw = _need(m, "right", mw), f"{mw}.right"
                mixer = ParallelLayer(
                    left=_attention_branch(_need(m, "left", mw), f"{mw}.left"),
                    right=MatrixMemoryBranch(heads=_size(right, "heads", rw), dim=_size(right, "dim", rw), vdim=_size(right, "vdim", rw),
                                             gate_cap=_positive(right, "gate_cap", rw)))
            else:
                raise ConfigError(f"config.json: {where} has type {kind!r}; known: gla, parallel")
            layers.append(TefavikLayer(kind, mixer, _experts(layer.get("mlp"), f"{where}.mlp")))
        if not layers:
            raise ConfigError("config.json: a model needs at least one layer")
        loop = d.get("loop")
        if loop:
            loop = Loop(int(_need(loop, "start", "loop")), int(_need(loop, "stop", "loop")), int(_need(loop, "times", "loop")))
            if not (0 <= loop.start < loop.stop <= len(layers) and loop.times >= 1):
                raise ConfigError(f"config.json: loop {loop} names no run of the {len(layers)} layers")
        eos = d.get("eos_token_id")
        return cls(vocab=_size(d, "vocab", "the file"), width=_size(d, "width", "the file"),
                   norm_eps=float(_need(_need(d, "norm", "the file"), "eps", "norm")), layers=tuple(layers), loop=loop or None,
                   eos_token_ids=() if eos is None else tuple(int(e) for e in (eos if isinstance(eos, (list, tuple)) else [eos])))

    def with_tensor_shapes(self, shapes: dict[str, tuple[int, ...]]) -> "TefavikConfig":
        """With the inner sizes of the decays' projections, which only the checkpoint's tensors say."""
        layers = []
        for i, layer in enumerate(self.layers):
            name = f"l{i}.mix.a1"
            if isinstance(layer.mixer, GatedLinearLayer) and name in shapes:
                layer = replace(layer, mixer=replace(layer.mixer, rank=int(shapes[name][0])))
            layers.append(layer)
        return replace(self, layers=tuple(layers))

    def run_order(self) -> list[tuple[int, bool]]:
        """(layer, whether the embedding's output is added to the stream in front of it) in the order the layers run: that
        happens once at the start of every pass of the loop but the first."""
        n = len(self.layers)
        if self.loop is None:
            return [(i, False) for i in range(n)]
        a, b = self.loop.start, self.loop.stop
        inside = [(i, t > 0 and i == a) for t in range(self.loop.times) for i in range(a, b)]
        return [(i, False) for i in range(a)] + inside + [(i, False) for i in range(b, n)]
