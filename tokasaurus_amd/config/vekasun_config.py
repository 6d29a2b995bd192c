"""The configuration of a Vekasun model, read from its ``config.json``.

The file lists the layers one by one; every size and every constant that may differ between
two models of the design is taken from it.  Keys:

    architecture: "Vekasun"       vocab, width       norm.eps       logit_scale (absent: 1)
    loop: absent or null | {start, stop, times}   layers start .. stop-1 run ``times`` times in a row
    layers[i].type: "mamba2" | "latent_attention"
    layers[i].mlp: null | {"kind": "moe", "expert": {ff}, "router": {experts, top}}
    mamba2 mixer:           heads, vdim, state, groups, conv (taps), norm_groups
    latent_attention mixer: heads, dim, rot_dim, vdim, q_rank, kv_rank, scale, rot: {base, dims} (dims = rot_dim)
"""

from __future__ import annotations

from dataclasses import dataclass
from typing import Any

from tokasaurus_amd.config.kupuzen_config import _need
from tokasaurus_amd.config.model_config import ConfigError
from tokasaurus_amd.config.taborax_config import Loop


@dataclass(frozen=True)
class StateSpaceLayer:
    heads: int
    vdim: int
    state: int
    groups: int
    taps: int
    norm_groups: int


@dataclass(frozen=True)
class SinkLatentAttentionLayer:
    heads: int
    dim: int
    rot_dim: int
    vdim: int
    q_rank: int
    kv_rank: int
    scale: float
    rot_base: float


@dataclass(frozen=True)
class InputWeightedExperts:
    ff: int  # inner size of an expert
    experts: int
    top: int


@dataclass(frozen=True)
class VekasunLayer:
    kind: str
    mixer: StateSpaceLayer | SinkLatentAttentionLayer
    ff: InputWeightedExperts | None


@dataclass(frozen=True)
class VekasunConfig:
    vocab: int
    width: int
    norm_eps: float
    logit_scale: float
    layers: tuple[VekasunLayer, ...]
    loop: Loop | None = None
    eos_token_ids: tuple[int, ...] = ()

    @classmethod
    def from_dict(cls, d: dict[str, Any]) -> "VekasunConfig":
        layers = []
        for i, layer in enumerate(_need(d, "layers", "the file")):
            where = f"layers[{i}]"
            kind = _need(layer, "type", where)
            m = _need(layer, "mixer", where)
            mw = f"{where}.mixer"

            def size(key: str) -> int:
                n = int(_need(m, key, mw))
                if n <= 0:
                    raise ConfigError(f"config.json: {mw}.{key} must be positive, got {n}")
                return n

            if kind == "mamba2":
                mixer: Any = StateSpaceLayer(heads=size("heads"), vdim=size("vdim"), state=size("state"), groups=size("groups"),
                                             taps=size("conv"), norm_groups=size("norm_groups"))
                if mixer.heads % mixer.groups:
                    raise ConfigError(f"config.json: {mw}: {mixer.heads} heads are no multiple of {mixer.groups} groups")
                if (mixer.heads * mixer.vdim) % mixer.norm_groups:
                    raise ConfigError(f"config.json: {mw}: {mixer.heads} heads of {mixer.vdim} do not form {mixer.norm_groups} equal norm_groups")
            elif kind == "latent_attention":
                rot = _need(m, "rot", mw)
                mixer = SinkLatentAttentionLayer(
                    heads=size("heads"), dim=size("dim"), rot_dim=size("rot_dim"), vdim=size("vdim"), q_rank=size("q_rank"),
                    kv_rank=size("kv_rank"), scale=float(_need(m, "scale", mw)), rot_base=float(_need(rot, "base", f"{mw}.rot")))
                if mixer.rot_dim % 2 or int(_need(rot, "dims", f"{mw}.rot")) != mixer.rot_dim:
                    raise ConfigError(f"config.json: {mw}: rot.dims must be rot_dim, an even number")
            else:
                raise ConfigError(f"config.json: {where} has type {kind!r}; known: mamba2, latent_attention")
            mlp = layer.get("mlp")
            ff = None
            if mlp is not None:
                fw = f"{where}.mlp"
                if mlp.get("kind", "moe") != "moe":
                    raise ConfigError(f"config.json: {fw} has kind {mlp.get('kind')!r}; known: moe")
                r = _need(mlp, "router", fw)
                ff = InputWeightedExperts(ff=int(_need(_need(mlp, "expert", fw), "ff", f"{fw}.expert")),
                                          experts=int(_need(r, "experts", f"{fw}.router")), top=int(_need(r, "top", f"{fw}.router")))
                if ff.ff <= 0 or not 0 < ff.top <= ff.experts:
                    raise ConfigError(f"config.json: {fw}: {ff.top} of {ff.experts} experts of size {ff.ff}")
            layers.append(VekasunLayer(kind, mixer, ff))
        if not layers:
            raise ConfigError("config.json: a model needs at least one layer")
        loop = d.get("loop")
        if loop:
            loop = Loop(int(_need(loop, "start", "loop")), int(_need(loop, "stop", "loop")), int(_need(loop, "times", "loop")))
            if not (0 <= loop.start < loop.stop <= len(layers) and loop.times >= 1):
                raise ConfigError(f"config.json: loop {loop} names no run of the {len(layers)} layers")
        eos = d.get("eos_token_id")
        cfg = cls(
            vocab=int(_need(d, "vocab", "the file")), width=int(_need(d, "width", "the file")),
            norm_eps=float(_need(_need(d, "norm", "the file"), "eps", "norm")),
            logit_scale=float(d.get("logit_scale") if d.get("logit_scale") is not None else 1.0),
            layers=tuple(layers), loop=loop or None,
            eos_token_ids=() if eos is None else tuple(int(e) for e in (eos if isinstance(eos, (list, tuple)) else [eos])))
        if cfg.vocab <= 0 or cfg.width <= 0:
            raise ConfigError("config.json: vocab and width must be positive")
        return cfg

    def run_order(self) -> list[tuple[int, int | None]]:
        """(layer, number of the loop's pass that begins with it or None) in the order the layers run."""
        n = len(self.layers)
        if self.loop is None:
            return [(i, None) for i in range(n)]
        a, b = self.loop.start, self.loop.stop
        inside = [(i, t if i == a else None) for t in range(self.loop.times) for i in range(a, b)]
        return [(i, None) for i in range(a)] + inside + [(i, None) for i in range(b, n)]
