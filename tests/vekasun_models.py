"""Small Vekasun configurations of the tests' own, their model folders, and the plain model's rows for
them.  The configurations differ from one another in every size and option: state-space layers with one
group and as many groups as heads, norms over the whole row and head by head, states and values off every
multiple of sixteen, convolutions of one, two, three and six taps; latent attention with latents of sizes the matrix-core kernels
take and do not take, one head and many; experts of which one, some and all are chosen, and layers without;
runs of layers that are passed once, twice and three times, at the start, inside and over the whole model, and
none; a model without any attention (no cache group) and one without any recurrence.
"""

from __future__ import annotations

import json
from pathlib import Path

import torch
from safetensors import safe_open
from safetensors.torch import save_file

import plain_vekasun
from tokasaurus_amd.weights import write_random_model


def mamba_layer(heads, vdim, state, groups, norm_groups, taps, mlp=None):
    return {"type": "mamba2", "mlp": mlp, "mixer": {"heads": heads, "vdim": vdim, "state": state, "groups": groups,
                                                    "norm_groups": norm_groups, "conv": taps}}


def latent_layer(heads, dim, rot_dim, vdim, q_rank, kv_rank, scale, base=10000.0, mlp=None):
    return {"type": "latent_attention", "mlp": mlp, "mixer": {
        "heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "q_rank": q_rank, "kv_rank": kv_rank, "scale": scale,
        "rot": {"base": base, "dims": rot_dim}}}


def moe(ff, experts, top):
    return {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top}}


def model(vocab, width, layers, eps=1e-5, loop=None, logit_scale=1.0):
    cfg = {"architecture": "Vekasun", "vocab": vocab, "width": width, "norm": {"eps": eps}, "logit_scale": logit_scale, "layers": layers}
    if loop:
        cfg["loop"] = dict(zip(("start", "stop", "times"), loop))
    return cfg


# every mechanism in one model; the loop begins behind the first layer and ends in front of the last
MIXED = model(160, 96, [
    mamba_layer(6, 16, 32, 3, 2, 4, mlp=moe(40, 6, 2)),
    latent_layer(4, 32, 16, 48, 64, 48, 0.2, mlp=moe(24, 5, 3)),
    mamba_layer(3, 32, 16, 1, 1, 3),
    latent_layer(6, 16, 8, 16, 24, 32, 0.3, base=500.0, mlp=moe(56, 3, 1)),
], loop=(1, 3, 2), logit_scale=0.7)
# sizes that fit nothing: a width that is no multiple of 4, odd heads, a cached key that is no multiple of 8, an odd number
# of experts, all of them chosen, two taps; the loop is the model
AWKWARD = model(131, 90, [
    latent_layer(3, 20, 6, 10, 18, 27, 0.25, base=77.0, mlp=moe(33, 3, 3)),
    mamba_layer(5, 6, 10, 5, 3, 2, mlp=moe(21, 7, 2)),
], eps=1e-4, loop=(0, 2, 3), logit_scale=2.0)
# heads of the sizes of large models; a loop of one layer at the end
LARGE_HEADS = model(120, 128, [
    mamba_layer(4, 64, 128, 2, 4, 4, mlp=moe(64, 8, 2)),
    latent_layer(8, 64, 32, 64, 96, 128, 0.1, mlp=moe(48, 4, 4)),
    mamba_layer(2, 128, 160, 1, 1, 4),
], loop=(2, 3, 2))
# no attention at all (no cache group, no pages), a loop passed once; and no recurrence at all (no state in any slot), no loop
ONLY_STATES = model(64, 48, [mamba_layer(2, 8, 24, 2, 2, 1, mlp=moe(16, 4, 1)), mamba_layer(4, 24, 8, 1, 1, 6)], loop=(0, 1, 1))
ONLY_ATTENTION = model(70, 64, [
    latent_layer(1, 16, 16, 16, 16, 16, 0.25, mlp=moe(48, 2, 1)),
    latent_layer(16, 24, 4, 32, 40, 300, 0.3, base=100.0),  # a latent larger than the matrix-core attention takes
])
CONFIGS = {"mixed": MIXED, "awkward": AWKWARD, "large_heads": LARGE_HEADS, "only_states": ONLY_STATES, "only_attention": ONLY_ATTENTION}


def make_folder(folder: Path, config: dict, seed: int, edits: dict | None = None, steady_choice: bool = False) -> Path:
    """Random weights with the parts scaled so that each mechanism matters to the logits: projections of order one a
    row, added rows as large as the tokens' rows, decays from fast to slow, convolution biases, sinks and skips of order
    one, routers whose scores differ clearly.  ``edits``: name suffix -> function of the tensor, applied last.
    ``steady_choice``: every token's row has one direction in common and a router reads that direction only, its experts'
    logits far apart in a shuffled order, so that the choice of experts (not their weights) is the same for every token
    and no comparison in bfloat16 rests on which of two nearly equal scores is larger; the 32-bit runs use the
    data-dependent choice."""
    write_random_model(folder, config, seed)
    path = folder / "model.safetensors"
    gen = torch.Generator().manual_seed(seed + 1000)
    common = torch.randn(config["width"], generator=gen)
    common = common - common.mean()
    tensors = {}
    with safe_open(str(path), framework="pt") as f:
        for name in sorted(f.keys()):
            t = f.get_tensor(name).float()
            if t.dim() == 2 and not name.endswith(".conv"):
                t = t * (1.0 / (0.02 * t.shape[1] ** 0.5))  # N(0, 1/in): outputs of order one
            if name in ("embed", "loop.step"):
                t = t * (t.shape[1] ** 0.5)
            if steady_choice and name == "embed":
                t = t + 1.5 * common
            if name.endswith(".router"):
                t = t * 2.0
                if steady_choice:
                    n = t.shape[0]
                    a = torch.linspace(-1.5, 1.5, n)[torch.randperm(n, generator=gen)] if n > 1 else torch.ones(1)
                    t = a[:, None] * common[None, :] / common.norm() * 4.0 / config["width"] ** 0.5
            if name.endswith(".A_log"):
                t = 2.0 * t - 1.5
            if name.endswith(".conv.b"):
                t = t * 25.0
            if name.endswith((".sink", ".D")):
                t = t * 2.0
            for suffix, fn in (edits or {}).items():
                if name.endswith(suffix):
                    t = fn(t)
            tensors[name] = t.to(torch.bfloat16).contiguous()
    save_file(tensors, str(path))
    return folder


def load_plain(folder: Path, dtype=torch.float64):
    config = json.loads((Path(folder) / "config.json").read_text())
    w = {}
    with safe_open(str(Path(folder) / "model.safetensors"), framework="pt") as f:
        for name in f.keys():
            w[name] = f.get_tensor(name).to(dtype)
    return config, w


def plain_rows(folder: Path, requests: dict[str, list[int]]) -> dict[str, torch.Tensor]:
    config, w = load_plain(folder)
    return {rid: plain_vekasun.forward(toks, w, config).float() for rid, toks in requests.items()}


def row_error(row: torch.Tensor, ref: torch.Tensor) -> float:
    return float((row - ref).pow(2).mean().sqrt() / ref.pow(2).mean().sqrt().clamp_min(1e-9))


def rounding_limits(folder: Path, requests: dict[str, list[int]]) -> dict[tuple[str, int], float]:
    """Three times what rounding alone does to every row.  A part of few numbers that nearly cancel in front of its norm
    makes some rows of a small model move many times further than others."""
    config, w = load_plain(folder)
    out = {}
    for rid, toks in requests.items():
        exact = plain_vekasun.forward(toks, w, config)
        with plain_vekasun.rounding():
            rounded = plain_vekasun.forward(toks, w, config)
        for pos in range(len(toks)):
            out[rid, pos] = 3.0 * row_error(rounded[pos], exact[pos])
    return out


def compare_rows(got: dict, plain: dict[str, torch.Tensor], tol: float, limits: dict | None = None) -> float:
    """Every collected row against the plain row: the root mean square of the difference over the
    vocabulary, relative to that of the plain row (a row may have a wider limit of its own).  Names the first wrong
    (request, position)."""
    worst = 0.0
    for (rid, pos), row in sorted(got.items()):
        err = row_error(row, plain[rid][pos])
        allowed = max(tol, (limits or {}).get((rid, pos), 0.0))
        assert err <= allowed, f"request {rid} position {pos}: relative error {err:.3e} (allowed {allowed:.1e})"
        worst = max(worst, err)
    return worst


# relative error of a row of logits: summation order in 32-bit; roundings to 8 bits of mantissa in bfloat16
TOL = {"float32": 3e-4, "bfloat16": 6e-2}
# in bfloat16 a router's choice between two experts of nearly equal score can fall the other way than in the
# plain model: the bfloat16 runs use folders with a steady choice
STEADY = {"float32": False, "bfloat16": True}
