"""Small Tefavik configurations of the tests' own, their model folders, and the plain model's rows for
them.  The configurations differ from one another in every size and option: gated linear attention with one head and many,
keys and values of sizes that fit nothing, decays through small and large tau and ranks of one to forty; attention in chunks
of one position, of fewer than a page, across pages and longer than any request, one to many query heads a key/value head,
rotations of a part and of the whole head; memories with few and many rows; experts of which one, some and all are chosen,
and layers without; runs of layers that are passed once, twice and three times, at the start, inside and over the whole
model, and none; a model without any attention (no cache group).
"""

from __future__ import annotations

import json
from pathlib import Path

import torch
from safetensors import safe_open
from safetensors.torch import save_file

import plain_tefavik
from tokasaurus_amd.weights import write_random_model


def gla_layer(heads, dim, vdim, tau, rank, mlp=None):
    # (the rank is read from a checkpoint's shapes; a model that is drawn is told it)
    return {"type": "gla", "mlp": mlp, "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "tau": tau, "rank": rank}}


def attention_branch(heads, kv_heads, dim, vdim, chunk, rot_dims=None, scale=0.3, softcap=20.0, base=10000.0):
    return {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale, "softcap": softcap, "mask": {"size": chunk},
            "rot": {"base": base, "dims": dim if rot_dims is None else rot_dims}}


def memory_branch(heads, dim, vdim, cap=9.0):
    return {"heads": heads, "dim": dim, "vdim": vdim, "gate_cap": cap}


def pair_layer(left, right, mlp=None):
    return {"type": "parallel", "mlp": mlp, "mixer": {"left": left, "right": right}}


def moe(ff, experts, top, limit=1.5):
    return {"kind": "moe", "expert": {"ff": ff, "limit": limit}, "router": {"experts": experts, "top": top}}


def model(vocab, width, layers, eps=1e-5, loop=None):
    cfg = {"architecture": "Tefavik", "vocab": vocab, "width": width, "norm": {"eps": eps}, "layers": layers}
    if loop:
        cfg["loop"] = dict(zip(("start", "stop", "times"), loop))
    return cfg


# every mechanism in one model; the loop begins behind the first layer and ends in front of the last
MIXED = model(150, 96, [
    gla_layer(3, 32, 48, 8.0, 12, mlp=moe(40, 6, 2)),
    pair_layer(attention_branch(4, 2, 32, 16, 24, rot_dims=16), memory_branch(2, 24, 32), mlp=moe(24, 5, 3, limit=0.7)),
    gla_layer(2, 16, 64, 16.0, 24),
    pair_layer(attention_branch(6, 1, 16, 32, 40, base=500.0), memory_branch(6, 16, 16, cap=5.0), mlp=moe(56, 3, 1)),
], loop=(1, 3, 2))
# sizes that fit nothing: a width that is no multiple of 4, odd heads, keys off every multiple of 8, values off 16, all
# experts chosen; the loop is the model
AWKWARD = model(131, 90, [
    pair_layer(attention_branch(3, 3, 20, 10, 7, rot_dims=6, base=77.0), memory_branch(5, 6, 9, cap=3.0), mlp=moe(33, 3, 3)),
    gla_layer(5, 7, 10, 3.0, 5, mlp=moe(21, 7, 2, limit=0.4)),
], eps=1e-4, loop=(0, 2, 3))
# heads of the sizes of large models; a loop of one layer at the end
LARGE_HEADS = model(120, 128, [
    pair_layer(attention_branch(8, 2, 64, 128, 64, scale=0.125), memory_branch(2, 128, 128), mlp=moe(64, 8, 2)),
    gla_layer(2, 128, 96, 16.0, 16, mlp=moe(48, 4, 4)),
    pair_layer(attention_branch(16, 1, 128, 64, 160, scale=0.1), memory_branch(1, 160, 70), mlp=moe(16, 2, 1)),
], loop=(2, 3, 2))
# no attention at all (no cache group, no pages), a loop passed once; and no loop, no feed-forward
ONLY_STATES = model(64, 48, [gla_layer(2, 24, 8, 16.0, 1, mlp=moe(16, 4, 1)), gla_layer(4, 8, 24, 1.0, 40)], loop=(0, 1, 1))
ONLY_PAIRS = model(70, 64, [
    pair_layer(attention_branch(1, 1, 16, 16, 1), memory_branch(1, 16, 16)),
    pair_layer(attention_branch(4, 4, 8, 16, 16), memory_branch(8, 8, 8, cap=1.0), mlp=moe(48, 2, 1, limit=30.0)),
])
CONFIGS = {"mixed": MIXED, "awkward": AWKWARD, "large_heads": LARGE_HEADS, "only_states": ONLY_STATES, "only_pairs": ONLY_PAIRS}


def make_folder(folder: Path, config: dict, seed: int, edits: dict | None = None) -> Path:
    """Random weights with the parts scaled so that each mechanism matters to the logits: projections of order one a
    row, biases of order a half, forget gates that keep and decays from fast to slow, input gates on both sides of zero.
    ``edits``: name suffix -> function of the tensor, applied last."""
    write_random_model(folder, config, seed)
    path = folder / "model.safetensors"
    tensors = {}
    with safe_open(str(path), framework="pt") as f:
        for name in sorted(f.keys()):
            t = f.get_tensor(name)
            if t.dtype == torch.int32:
                tensors[name] = t
                continue
            t = t.float()
            if t.dim() == 2:
                t = t * (1.0 / (0.02 * t.shape[1] ** 0.5))  # N(0, 1/in): outputs of order one
            if name == "embed":
                t = t * (t.shape[1] ** 0.5)
            if name.endswith((".q.b", ".k.b", ".v.b")):
                t = t * 25.0
            if name.endswith(".a2.b"):
                t = t * 75.0 + 1.0
            if name.endswith(".i.b"):
                t = t * 3.0
            if name.endswith(".f.b"):
                t = t * 2.0 + 2.5
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
            t = f.get_tensor(name)
            w[name] = t if t.dtype == torch.int32 else t.to(dtype)
    return config, w


def plain_rows(folder: Path, requests: dict[str, list[int]]) -> dict[str, torch.Tensor]:
    config, w = load_plain(folder)
    return {rid: plain_tefavik.forward(toks, w, config).float() for rid, toks in requests.items()}


def row_error(row: torch.Tensor, ref: torch.Tensor) -> float:
    return float((row - ref).pow(2).mean().sqrt() / ref.pow(2).mean().sqrt().clamp_min(1e-9))


def rounding_limits(folder: Path, requests: dict[str, list[int]]) -> dict[tuple[str, int], float]:
    """Three times what rounding alone does to every row.  A head's few numbers that nearly cancel in front of its norm
    make some rows of a small model move many times further than others."""
    config, w = load_plain(folder)
    out = {}
    for rid, toks in requests.items():
        exact = plain_tefavik.forward(toks, w, config)
        with plain_tefavik.rounding():
            rounded = plain_tefavik.forward(toks, w, config)
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
