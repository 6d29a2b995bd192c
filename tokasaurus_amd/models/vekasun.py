"""Vekasun as a choice of parts: a plain embedding into a 32-bit residual stream; blocks with a layer norm (weight, no
bias) in front of each sublayer; per layer a selective state-space mixer (Mamba-2: a short convolution, a matrix per head
with a decay per head and token, a gate and a norm in equal parts behind it) or attention over a cached latent beside a
rotated key part that all heads share (queries through a latent of their own, a rotation of halves, a learned sink per
head, a sigmoid gate per element); per layer a mixture of gated experts with sigmoid scores whose weights multiply what
the experts read, or none; a run of layers that is passed several times with the same weights, each pass with caches and
states of its own and begun by adding a learned row of the pass to the stream; a final layer norm and a head whose logits
are scaled.  Checkpoint names: ``embed``, ``loop.step``, ``l<i>.norm1|norm2``, ``l<i>.mix.*``, ``l<i>.mlp.*``,
``final.norm``, ``head``.
"""

from __future__ import annotations

from tokasaurus_amd.config.vekasun_config import StateSpaceLayer, VekasunConfig
from tokasaurus_amd.models.spec import ModelSpec, RunEntry
from tokasaurus_amd.parts.base import PartSpec

MAX_POSITIONS = 1 << 30  # the rotation computes its angles from the position: no table ends them


def vekasun_spec(cfg: VekasunConfig) -> ModelSpec:
    def norm(name: str) -> PartSpec:
        return PartSpec("stream_layernorm", {"size": cfg.width, "eps": cfg.norm_eps, "name": name})

    layers, unused = [], []
    for i, layer in enumerate(cfg.layers):
        m, p = layer.mixer, f"l{i}.mix"
        if isinstance(m, StateSpaceLayer):
            mixer = PartSpec("mamba2", {
                "hidden_size": cfg.width, "num_heads": m.heads, "value_dim": m.vdim, "state_dim": m.state, "groups": m.groups,
                "taps": m.taps, "norm_groups": m.norm_groups, "norm_eps": cfg.norm_eps,
                "names": {"in": f"{p}.in", "conv": f"{p}.conv", "conv_bias": f"{p}.conv.b", "dt_bias": f"{p}.dt_bias",
                          "A_log": f"{p}.A_log", "D": f"{p}.D", "norm": f"{p}.norm", "o": f"{p}.o"}})
        else:
            mixer = PartSpec("latent_attention", {
                "hidden_size": cfg.width, "num_heads": m.heads, "key_dim": m.dim, "value_dim": m.vdim, "q_rank": m.q_rank,
                "kv_rank": m.kv_rank, "rot_dim": m.rot_dim, "scale": m.scale, "norm_eps": cfg.norm_eps,
                "position": PartSpec("rotary_halves", {"dims": m.rot_dim, "base": m.rot_base}),
                "names": {"dq": f"{p}.dq", "dq_norm": f"{p}.dq.norm", "uq": f"{p}.uq", "dkv": f"{p}.dkv",
                          "dkv_norm": f"{p}.dkv.norm", "uk": f"{p}.uk", "uv": f"{p}.uv", "sink": f"{p}.sink", "g": f"{p}.g",
                          "o": f"{p}.o"}})
        params = {"mixer_norm": norm(f"l{i}.norm1"), "mixer": mixer}
        if layer.ff is None:
            unused.append(f"l{i}.norm2")
        else:
            q = f"l{i}.mlp"
            params["ff_norm"] = norm(f"l{i}.norm2")
            params["feed_forward"] = PartSpec("routed_experts", {
                "hidden_size": cfg.width, "expert_size": layer.ff.ff, "num_experts": layer.ff.experts, "top": layer.ff.top,
                "scores": "sigmoid", "weights_on_input": True, "names": {"router": f"{q}.router", "expert": q + ".e{e}"}})
        layers.append(PartSpec("stream_pre_norm", params))
    times = cfg.loop.times if cfg.loop is not None else 0
    return ModelSpec(
        vocab_size=cfg.vocab,
        embedding=PartSpec("token_embedding", {"vocab_size": cfg.vocab, "hidden_size": cfg.width, "name": "embed", "stream_f32": True}),
        head=PartSpec("norm_linear", {"vocab_size": cfg.vocab, "hidden_size": cfg.width, "name": "head", "norm": norm("final.norm"),
                                      "scale": cfg.logit_scale}),
        layers=tuple(layers),
        # a layer that is passed again is named again: every use has a cache and a state of its own
        run_order=tuple(RunEntry(i, before=t) for i, t in cfg.run_order()),
        connectors=tuple(PartSpec("add_row", {"hidden_size": cfg.width, "name": "loop.step", "rows": times, "row": t}) for t in range(times)),
        max_positions=MAX_POSITIONS,
        eos_token_ids=cfg.eos_token_ids,
        # a layer without a feed-forward may still carry the norm in front of it
        ignorable_tensors=tuple(unused),
    )
