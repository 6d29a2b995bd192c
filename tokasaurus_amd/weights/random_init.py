"""Random weights: writes a model folder (config.json, model.safetensors) from a
configuration and a seed.  The reference has no such mode (it only fabricates
inputs, tokasaurus/manager/input_building.py:14-100).

Every matrix is drawn from N(0, 0.02), every norm weight from 1 + N(0, 0.01) (from N(0, 0.01)
when it is stored around zero, as is a vector that only nudges), other learned vectors from N(0, 0.5),
in 32-bit on the host, in the sorted order of the tensor names, from one
generator seeded with ``seed``; integer tables are drawn uniformly (rows of different
numbers where the table names rows' choices from a few).  Tensors are
stored in bfloat16, so the 32-bit engine, the bfloat16 engine and any plain
implementation read exactly the same values.  A tied head is not drawn.
"""

from __future__ import annotations

import json
from pathlib import Path
from typing import Any

import torch
from safetensors.torch import save_file

from tokasaurus_amd.models.registry import architecture_of
from tokasaurus_amd.parts.base import (AVERAGE_WEIGHT, BIAS, CONV, INT_TABLE, MATRIX, NORM_OFFSET, NORM_WEIGHT, SMALL_VECTOR, UNIT_INTERVAL,
                                       VECTOR, TensorSpec)

MATRIX_STD = 0.02
NORM_STD = 0.01
VECTOR_STD = 0.5


def draw_tensors(
    specs: list[TensorSpec],
    seed: int,
    store_dtype: torch.dtype = torch.bfloat16,
    device: str | torch.device = "cpu",
) -> dict[str, torch.Tensor]:
    """Seeded tensors for every spec.  On the host (the default) the values are
    a function of the seed alone; ``device`` draws them with that device's
    generator instead (large benchmark models, where no folder is written)."""
    gen = torch.Generator(device=device)
    gen.manual_seed(int(seed))
    out: dict[str, torch.Tensor] = {}
    for spec in sorted(specs, key=lambda s: s.name):
        if spec.kind in (MATRIX, BIAS):
            t = torch.randn(spec.shape, generator=gen, dtype=torch.float32, device=device) * MATRIX_STD
        elif spec.kind == NORM_WEIGHT:
            t = 1.0 + torch.randn(spec.shape, generator=gen, dtype=torch.float32, device=device) * NORM_STD
        elif spec.kind in (NORM_OFFSET, SMALL_VECTOR):
            t = torch.randn(spec.shape, generator=gen, dtype=torch.float32, device=device) * NORM_STD
        elif spec.kind in (VECTOR, CONV):
            t = torch.randn(spec.shape, generator=gen, dtype=torch.float32, device=device) * VECTOR_STD
        elif spec.kind == UNIT_INTERVAL:
            t = 0.05 + 0.9 * torch.rand(spec.shape, generator=gen, dtype=torch.float32, device=device)
        elif spec.kind == AVERAGE_WEIGHT:
            n = max(1, spec.shape[-1])
            t = (1.0 + 0.1 * torch.randn(spec.shape, generator=gen, dtype=torch.float32, device=device)) / n
        elif spec.kind == INT_TABLE and spec.below:
            # every row: the first columns of a random order of 0 .. below - 1
            keys = torch.rand((*spec.shape[:-1], spec.below), generator=gen, dtype=torch.float32, device=device)
            out[spec.name] = keys.argsort(dim=-1)[..., : spec.shape[-1]].to(torch.int32).contiguous()
            continue
        elif spec.kind == INT_TABLE:
            out[spec.name] = torch.randint(0, 1 << 15, spec.shape, generator=gen, dtype=torch.int32, device=device)
            continue
        else:
            raise ValueError(f"tensor {spec.name}: unknown kind {spec.kind!r}")
        out[spec.name] = t.to(store_dtype)
    return out


def write_random_model(
    folder: str | Path,
    config: dict[str, Any],
    seed: int,
    store_dtype: torch.dtype = torch.bfloat16,
) -> Path:
    """Write ``config.json`` and ``model.safetensors`` for the architecture that
    ``config['model_type']`` names; returns the folder."""
    from tokasaurus_amd.models.registry import build_model

    folder = Path(folder)
    folder.mkdir(parents=True, exist_ok=True)
    arch = architecture_of(config)
    cfg = arch.config_from_dict(config)
    model = build_model(arch, cfg)
    tensors = draw_tensors(model.tensor_specs(), seed, store_dtype)
    (folder / "config.json").write_text(json.dumps(config, indent=2) + "\n")
    save_file({k: v.contiguous() for k, v in tensors.items()}, str(folder / "model.safetensors"))
    return folder
