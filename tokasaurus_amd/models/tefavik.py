"""Tefavik as a choice of parts: a plain embedding into a 32-bit residual stream; blocks with an RMS norm in front of each
sublayer; per layer gated linear attention (a decay per key channel from a projection of low rank, a norm head by head, a silu
gate), or two mixers side by side, each output with a norm of its own, in equal halves: soft-capped attention inside chunks of
positions (norms of queries and keys head by head, a rotation of neighbours, biases, one added to the softmax's denominator)
and a matrix memory (mLSTM: exponential gates behind a soft cap, relative to a running maximum); per layer a mixture of
experts with clamped activations that a table chooses by token id, or none; a run of layers that is passed several times with
the same weights, each pass with caches and states of its own and every one but the first begun by adding the embedding's
output to the stream; a final norm and a head whose matrix is the embedding's.  Checkpoint names: ``embed``,
``l<i>.norm1|norm2``, ``l<i>.mix.*``, ``l<i>.mlp.*``, ``final.norm``.
"""

from __future__ import annotations

from tokasaurus_amd.config.tefavik_config import GatedLinearLayer, TefavikConfig
from tokasaurus_amd.models.spec import ModelSpec, RunEntry
from tokasaurus_amd.parts.base import PartSpec

MAX_POSITIONS = 1 << 30  # the rotation computes its angles from the position: no table ends them
DEFAULT_RANK = 16  # inner size of the decays' projections when no checkpoint says
GLU_ALPHA = 1.702


def tefavik_spec(cfg: TefavikConfig) -> ModelSpec:
    W = cfg.width

    def norm(name: str) -> PartSpec:
        return PartSpec("stream_rmsnorm", {"size": W, "eps": cfg.norm_eps, "name": name})

    layers, unused = [], []
    for i, layer in enumerate(cfg.layers):
        m, p = layer.mixer, f"l{i}.mix"
        if isinstance(m, GatedLinearLayer):
            mixer = PartSpec("gated_linear_attention", {
                "hidden_size": W, "num_heads": m.heads, "key_dim": m.dim, "value_dim": m.vdim, "rank": m.rank or DEFAULT_RANK,
                "tau": m.tau, "norm_eps": cfg.norm_eps, "q_scale": m.dim ** -0.5,
                "names": {"q": f"{p}.q", "k": f"{p}.k", "v": f"{p}.v", "g": f"{p}.g", "a1": f"{p}.a1", "a2": f"{p}.a2",
                          "a2_bias": f"{p}.a2.b", "norm": f"{p}.norm", "o": f"{p}.o"}})
        else:
            a, b, pl, pr = m.left, m.right, f"{p}.left", f"{p}.right"
            position = None
            if a.rot_base is not None:
                position = PartSpec("rotary_interleaved", {"dims": a.rot_dims, "base": a.rot_base})
            left = PartSpec("grouped_attention", {
                "hidden_size": W, "num_heads": a.heads, "num_kv_heads": a.kv_heads, "key_dim": a.dim, "value_dim": a.vdim,
                "scale": a.scale, "softcap": a.softcap, "section": a.chunk, "position": position, "sink_value": 0.0, "key_chunk": 256,
                "head_norm": {"q": f"{pl}.q.norm", "k": f"{pl}.k.norm", "eps": cfg.norm_eps},
                "bias_names": {"q": f"{pl}.q.b", "k": f"{pl}.k.b", "v": f"{pl}.v.b"},
                "names": {"q": f"{pl}.q", "k": f"{pl}.k", "v": f"{pl}.v", "o": f"{pl}.o"}})
            right = PartSpec("matrix_memory", {
                "hidden_size": W, "num_heads": b.heads, "key_dim": b.dim, "value_dim": b.vdim, "gate_cap": b.gate_cap,
                "norm_eps": cfg.norm_eps, "q_scale": b.dim ** -0.5,
                "names": {"q": f"{pr}.q", "k": f"{pr}.k", "v": f"{pr}.v", "g": f"{pr}.g", "i": f"{pr}.i", "i_bias": f"{pr}.i.b",
                          "f": f"{pr}.f", "f_bias": f"{pr}.f.b", "norm": f"{pr}.norm", "o": f"{pr}.o"}})
            mixer = PartSpec("mixer_pair", {"hidden_size": W, "left": left, "right": right, "left_scale": 0.5, "right_scale": 0.5,
                                            "out_norms": {"left": f"{pl}.out", "right": f"{pr}.out", "eps": cfg.norm_eps}})
        params = {"mixer_norm": norm(f"l{i}.norm1"), "mixer": mixer}
        if layer.ff is None:
            unused.append(f"l{i}.norm2")
        else:
            q, f = f"l{i}.mlp", layer.ff
            params["ff_norm"] = norm(f"l{i}.norm2")
            params["feed_forward"] = PartSpec("table_experts", {
                "hidden_size": W, "vocab_size": cfg.vocab, "expert_size": f.ff, "num_experts": f.experts, "top": f.top,
                "glu": (f.limit, GLU_ALPHA), "names": {"table": f"{q}.table", "expert": q + ".e{e}"}})
        layers.append(PartSpec("stream_pre_norm", params))
    order = cfg.run_order()
    return ModelSpec(
        vocab_size=cfg.vocab,
        embedding=PartSpec("token_embedding", {"vocab_size": cfg.vocab, "hidden_size": W, "name": "embed", "stream_f32": True}),
        # the head names the embedding's tensor: one buffer
        head=PartSpec("norm_linear", {"vocab_size": cfg.vocab, "hidden_size": W, "name": "embed", "norm": norm("final.norm")}),
        layers=tuple(layers),
        # a layer that is passed again is named again: every use has a cache and a state of its own
        run_order=tuple(RunEntry(i, before=0 if add else None) for i, add in order),
        connectors=(PartSpec("add_embedding"),) if any(add for _, add in order) else (),
        max_positions=MAX_POSITIONS,
        eos_token_ids=cfg.eos_token_ids,
        # a layer without a feed-forward may still carry the norm in front of it
        ignorable_tensors=tuple(unused),
    )
