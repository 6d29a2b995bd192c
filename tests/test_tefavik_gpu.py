"""Tefavik through the engine against the plain model: every mechanism alone, prompts against
token-by-token decoding, portions down to two tokens and one, unequal requests in one batch on pages
and slots that are used again, keys on both sides of a chunk's border and of a page's, tokens far back in
the recurrences, first tokens, long decoding, and greedy generation through ``Engine.generate``."""

from __future__ import annotations

import json
import os
import random
import subprocess
import sys

import numpy as np
import pytest
import torch

import plain_tefavik as pt
from replay_helpers import mixed_trace, portions, run_steps, tail_one_by_one, whole
from tefavik_models import (CONFIGS, MIXED, TOL, attention_branch, compare_rows, gla_layer, load_plain, make_folder, memory_branch, model,
                            moe, pair_layer, plain_rows, rounding_limits)
from tiny_models import random_tokens
from tokasaurus_amd.engine.batch import StepEntry, layout, to_device
from tokasaurus_amd.engine.runner import ModelRunner
from tokasaurus_amd.kernels import ops

pytestmark = pytest.mark.gpu
PAGE = 16


@pytest.fixture(scope="module")
def tefavik_folders(tmp_path_factory):
    root = tmp_path_factory.mktemp("tefavik")
    return {name: make_folder(root / name, cfg, seed=5 + i) for i, (name, cfg) in enumerate(sorted(CONFIGS.items()))}


def runner_for(folder, dtype, tokens=512, slots=4, **kw):
    return ModelRunner.from_folder(str(folder), dtype, page_size=PAGE, num_pages=tokens // PAGE, max_slots=slots, **kw)


def i32(v):
    return torch.tensor(v, dtype=torch.int32, device="cuda")


# ---------------------------------------------------------------------------------- kernels alone


def cuts_of(lens):
    """The same requests' tokens as steps: whole; two portions; portions of a few tokens and single tokens."""
    yield [list(lens)]
    yield [[max(1, n // 2) for n in lens], [n - max(1, n // 2) for n in lens]]
    if max(lens) <= 48:
        steps, left, k = [], list(lens), 0
        while any(left):
            size = (3, 1, 1, 17, 2)[k % 5]
            steps.append([min(size, n) for n in left])
            left = [n - s for n, s in zip(left, steps[-1])]
            k += 1
        yield steps


def walk(run, proj, lens, slots, steps, in_chunks):
    """Hand ``run`` the rows of every step (rows, q_start, slots, positions, longest, chunks) and put its results back in the order of proj."""
    starts = [sum(lens[:r]) for r in range(len(lens))]
    held = [0] * len(lens)
    out = None
    for sizes in steps:
        idx, q_start, used, pos = [], [0], [], []
        for r, n in enumerate(sizes):
            if n == 0:
                continue
            idx += [starts[r] + held[r] + j for j in range(n)]
            pos += [held[r] + j for j in range(n)]
            q_start.append(len(idx))
            used.append(slots[r])
            held[r] += n
        req, row0, first = [], [], [0]
        for r, (a, b) in enumerate(zip(q_start, q_start[1:])):
            req += [r] * len(range(a, b, 64))
            row0 += range(a, b, 64)
            first.append(len(req))
        chunks = ops.ChunkPlan(i32(req), i32(row0), i32(first)) if in_chunks else None
        got = run(proj[idx].contiguous().cuda(), i32(q_start), i32(used), i32(pos), max(sizes), chunks)
        got = [g.cpu() for g in got]
        if out is None:
            out = [torch.zeros(proj.shape[0], g.shape[1]) for g in got]
        for o, g in zip(out, got):
            o[idx] = g
    return out


LINEAR_CASES = [  # heads, key size, value size, lengths of the requests
    (2, 16, 16, [1, 1, 1]), (3, 12, 10, [3, 40, 1, 9]), (1, 50, 20, [33, 2]), (4, 64, 64, [48, 30, 17]), (2, 128, 128, [130, 1, 20]),
    (5, 7, 9, [25]), (1, 160, 17, [70, 129]), (1, 256, 33, [100, 16]), (1, 300, 8, [40, 3]), (1, 512, 5, [6, 20]), (2, 1, 1, [19]),
]


@pytest.mark.parametrize("heads, dk, dv, lens", LINEAR_CASES)
@pytest.mark.parametrize("rank", [1, 16, 37])
@pytest.mark.parametrize("in_chunks", [False, True])
def test_gated_linear_attention_kernel(heads, dk, dv, lens, rank, in_chunks):
    """Decays from a projection of low rank and the recurrence, whole and in every cutting, token by token and (longer portions)
    in chunks, against the plain functions."""
    torch.manual_seed(dk + dv + rank)
    H, n, tau, scale = heads, sum(lens), 5.0, 0.3
    low_off = 3 + 2 * H * dk + H * dv
    proj = torch.randn(n, low_off + rank + 2)
    up, bias = torch.randn(rank, H * dk) * rank ** -0.5, torch.randn(H * dk) * 2.0 + 1.0
    bias[0] = 40.0  # a channel that forgets nothing
    bias[-1] = -300.0  # and one that forgets at once
    slots = list(range(len(lens)))[::-1]
    want, at = [], 0
    for ln in lens:
        p = proj[at : at + ln].double()
        q, k, v = (p[:, o : o + H * w].reshape(ln, H, w) for o, w in ((3, dk), (3 + H * dk, dk), (3 + 2 * H * dk, dv)))
        a = pt.decays(p[:, low_off : low_off + rank] @ up.double() + bias.double(), tau).view(ln, H, dk)
        want.append(pt.decayed_outer_products(q * scale, k, v, a).reshape(ln, H * dv))
        at += ln
    want = torch.cat(want).float()
    ops_args = (up.cuda(), bias.cuda(), tau, scale)
    for steps in cuts_of(lens):
        state = torch.zeros(len(lens) + 1, ops.linear_attention_state_words(H, dk, dv), device="cuda")
        (o,) = walk(lambda rows, qs, sl, pos, longest, chunks: (ops.gated_linear_attention(
            rows, 3, 3 + H * dk, 3 + 2 * H * dk, low_off, *ops_args, state, qs, sl, H, dk, dv, longest=longest,
            chunks=chunks),), proj, lens, slots, steps, in_chunks)
        torch.testing.assert_close(o, want, atol=2e-4, rtol=2e-4)
        assert float(state[len(lens)].abs().max()) == 0.0  # nobody's slot


@pytest.mark.parametrize("heads, dk, dv, lens", LINEAR_CASES + [(2, 8, 8, [1100, 513]), (1, 24, 16, [512, 511, 1])])
@pytest.mark.parametrize("sharp", [False, True])
@pytest.mark.parametrize("in_chunks", [False, True])
def test_matrix_memory_kernel(heads, dk, dv, lens, sharp, in_chunks):
    """Gates, the running maximum, the state and its read-out, whole and in every cutting, against the plain function;
    ``sharp``: gates near their caps, so that the maximum jumps and falls."""
    torch.manual_seed(dk + dv)
    H, n, cap, scale = heads, sum(lens), 9.0, 0.4
    i_off = 2 + 2 * H * dk + H * dv
    f_off = i_off + H + 1
    proj = torch.randn(n, f_off + H + 1)
    if sharp:
        proj[:, i_off : i_off + H] *= 12.0
        proj[:, f_off : f_off + H] *= 6.0
    i_bias, f_bias = torch.randn(H), torch.randn(H) + 2.0
    slots = list(range(len(lens)))[::-1]
    # the read-outs of S and n, and the maxima, apart: their quotient is the plain function's
    sums, keys, tops, at = [], [], [], 0
    for ln in lens:
        p = proj[at : at + ln].double()
        q, k, v = (p[:, o : o + H * w].reshape(ln, H, w) for o, w in ((2, dk), (2 + H * dk, dk), (2 + 2 * H * dk, dv)))
        i = pt.soft_cap(p[:, i_off : i_off + H] + i_bias.double(), cap)
        f = pt.log_sigmoid(pt.soft_cap(p[:, f_off : f_off + H] + f_bias.double(), cap))
        m = torch.zeros(ln + 1, H, dtype=torch.float64)
        for t in range(ln):
            m[t + 1] = torch.maximum(f[t] + m[t], i[t])
        keep, write = torch.exp(f + m[:-1] - m[1:])[..., None].expand(ln, H, dk), torch.exp(i - m[1:])[..., None]
        sums.append(pt.decayed_outer_products(q * scale, k * write, v, keep))
        keys.append(pt.decayed_outer_products(q * scale, k * write, torch.ones(ln, H, 1, dtype=torch.float64), keep)[..., 0])
        tops.append(m[1:])
        whole = sums[-1] / (torch.maximum(keys[-1].abs(), torch.exp(-m[1:])) + 1e-6)[..., None]
        assert torch.allclose(whole, pt.matrix_memory(q * scale, k, v, i, f))
        at += ln
    want = torch.cat([torch.cat(sums), torch.cat(keys)[..., None]], dim=-1)
    size = want.abs().amax(-1, keepdim=True).amax(1, keepdim=True) + 0.1
    for steps in cuts_of(lens):
        state = torch.zeros(len(lens) + 1, ops.linear_attention_state_words(H, dk, dv, memory=True), device="cuda")
        o, floor = walk(lambda rows, qs, sl, pos, longest, chunks: ops.matrix_memory(
            rows, 2, 2 + H * dk, 2 + 2 * H * dk, i_off, f_off, i_bias.cuda(), f_bias.cuda(), cap, scale, state, qs, sl, pos, H, dk, dv,
            longest=longest, chunks=chunks), proj, lens, slots, steps, in_chunks)
        o = o.view(n, H, -1).double()
        assert float(((o[..., : dv + 1] - want).abs() / size).max()) < 1e-4
        torch.testing.assert_close(floor.double(), torch.exp(-torch.cat(tops)), atol=1e-7, rtol=1e-4)
        assert float(state[len(lens)].abs().max()) == 0.0


@pytest.mark.parametrize("groups, size", [(3, 10), (4, 64), (2, 256), (1, 300), (2, 1024), (8, 16)])
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_group_norm_with_a_floor_a_weight_for_all_and_either_gate(groups, size, dtype):
    torch.manual_seed(size)
    n, pad = 5, -(-(size + 1) // 4) * 4
    o, floor = torch.randn(n, groups, pad), torch.rand(n, groups) + 0.05
    o[..., size] *= 0.5
    gate = torch.randn(n, groups * size + 3)[:, 3:]
    x = o[..., :size] / (torch.maximum(o[..., size].abs(), floor) + 1e-6)[..., None]
    for w in (torch.rand(size), torch.rand(groups * size)):
        ww = w.view(-1, size)
        normed = (pt.rms(x.double(), 1e-5) * ww.double()).reshape(n, groups * size)
        for silu in (False, True):
            want = normed * (torch.sigmoid(gate) * (gate if silu else 1.0)).double()
            got = ops.group_norm_gate(o.view(n, -1).cuda(), w.cuda(), 1e-5, groups, dtype, gate=gate.cuda(), size=size, floor=floor.cuda(),
                                      silu_gate=silu)
            tol = dict(atol=1e-5, rtol=1e-4) if dtype == torch.float32 else dict(atol=1e-2, rtol=1e-2)
            torch.testing.assert_close(got.float().cpu(), want.float(), **tol)


@pytest.mark.parametrize("hidden", [90, 96, 2048, 8200])
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_two_normed_branches_in_one_pass(hidden, dtype):
    torch.manual_seed(hidden)
    x, a, b = (torch.randn(7, hidden) * s for s in (1.0, 30.0, 0.01))
    wa, wb, wn = torch.rand(hidden), torch.rand(hidden), torch.rand(hidden)
    both = 0.5 * (pt.rms(a.double(), 1e-5) * wa.double() + pt.rms(b.double(), 1e-5) * wb.double())
    new = x.double() + both
    got, h = ops.post_norm_residual(x.cuda(), a.cuda(), wa.cuda(), 1e-5, wn.cuda(), 1e-3, dtype, in_place=False,
                                    second=(b.cuda(), wb.cuda()), mult=0.5)
    torch.testing.assert_close(got.cpu(), new.float(), atol=1e-5, rtol=1e-5)
    torch.testing.assert_close(h.float().cpu(), (pt.rms(new, 1e-3) * wn.double()).float(),
                               **(dict(atol=1e-5, rtol=1e-4) if dtype == torch.float32 else dict(atol=1e-2, rtol=1e-2)))
    alone, _ = ops.post_norm_residual(None, a.cuda(), wa.cuda(), 1e-5, in_place=False, second=(b.cuda(), wb.cuda()), mult=0.5)
    torch.testing.assert_close(alone.cpu(), both.float(), atol=1e-5, rtol=1e-5)


def test_lookup_of_experts_for_all_layers_at_once():
    torch.manual_seed(0)
    vocab, tops = 50, (1, 3, 2)
    tables = [torch.stack([torch.randperm(9)[:t] for _ in range(vocab)]).to(torch.int32) for t in tops]
    last = torch.tensor([7, 49, 0, 21], dtype=torch.int32)
    for n in (1, 5, 700):
        ids = torch.randint(0, vocab, (n,), dtype=torch.int32)
        ids[n // 2] = -2  # the token that slot 1 sampled
        got = ops.expert_lookup(ids.cuda(), last.cuda(), ops.ExpertTables([t.cuda() for t in tables]))
        real = ids.clone()
        real[n // 2] = 49
        for t, g in zip(tables, got):
            assert torch.equal(g.cpu(), t[real.long()])


@pytest.mark.parametrize("n", [1, 7, 40, 300])
@pytest.mark.parametrize("width, ff, experts, top", [(64, 48, 5, 2), (90, 33, 3, 3), (128, 64, 8, 1)])
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_experts_with_clamps_in_equal_parts(n, width, ff, experts, top, dtype):
    torch.manual_seed(n + ff)
    h = (torch.randn(n, width) * 2).to(dtype).float()
    gu, dn = (torch.randn(experts, 2 * ff, width) * width ** -0.5).to(dtype).float(), (torch.randn(experts, width, ff) * ff ** -0.5).to(dtype).float()
    ids = torch.stack([torch.randperm(experts)[:top] for _ in range(n)]).to(torch.int32)
    limit = 0.8
    got = ops.expert_mix(h.to(dtype).cuda(), gu.to(dtype).cuda(), dn.to(dtype).cuda(), ids.cuda(), None, glu=(limit, 1.702)).cpu()
    want = torch.zeros(n, width, dtype=torch.float64)
    for t in range(n):
        for e in ids[t].tolist():
            g, u = (gu[e].double() @ h[t].double()).split(ff)
            want[t] += dn[e].double() @ pt.clamped_gate(g, u, limit) / top
    tol = dict(atol=1e-4, rtol=1e-4) if dtype == torch.float32 else dict(atol=4e-2, rtol=2e-2)
    torch.testing.assert_close(got, want.float(), **tol)


# ---------------------------------------------------------------------------------- one layer alone

PLAIN_MEMORY = memory_branch(2, 8, 8)
PLAIN_LEFT = attention_branch(2, 1, 16, 16, 20)
SINGLE_LAYERS = {
    "gla": gla_layer(2, 16, 16, 16.0, 16),
    "gla_one_head": gla_layer(1, 64, 32, 4.0, 3),
    "gla_odd_sizes": gla_layer(3, 10, 7, 1.0, 5),
    "gla_large": gla_layer(2, 128, 128, 16.0, 16),
    "gla_of_one_row_and_column": gla_layer(2, 1, 1, 2.0, 1),
    "memory": pair_layer(PLAIN_LEFT, memory_branch(2, 16, 16)),
    "memory_one_head": pair_layer(PLAIN_LEFT, memory_branch(1, 32, 48, cap=2.0)),
    "memory_odd_sizes": pair_layer(PLAIN_LEFT, memory_branch(3, 7, 10)),
    "memory_large": pair_layer(PLAIN_LEFT, memory_branch(2, 128, 128, cap=15.0)),
    "memory_of_one_row_and_column": pair_layer(PLAIN_LEFT, memory_branch(2, 1, 1)),
    "chunks_of_one": pair_layer(attention_branch(2, 1, 16, 16, 1), PLAIN_MEMORY),
    "chunks_of_two": pair_layer(attention_branch(4, 4, 16, 16, 2), PLAIN_MEMORY),
    "chunks_of_a_page": pair_layer(attention_branch(4, 2, 16, 32, 16), PLAIN_MEMORY),
    "chunks_off_the_pages": pair_layer(attention_branch(8, 1, 24, 48, 21, rot_dims=8), PLAIN_MEMORY),
    "chunk_longer_than_all": pair_layer(attention_branch(2, 2, 32, 16, 1000, scale=1.0, softcap=2.0), PLAIN_MEMORY),
    "heads_no_tile_takes": pair_layer(attention_branch(3, 3, 9, 7, 10, rot_dims=4), PLAIN_MEMORY),
    "heads_larger_than_the_tile_s": pair_layer(attention_branch(1, 1, 320, 16, 24, scale=0.05), PLAIN_MEMORY),
    "large_heads": pair_layer(attention_branch(4, 2, 128, 64, 24, scale=0.09), PLAIN_MEMORY),
    "experts": gla_layer(1, 8, 8, 4.0, 2, mlp=moe(24, 7, 2)),
    "experts_one_of_many": pair_layer(PLAIN_LEFT, PLAIN_MEMORY, mlp=moe(10, 20, 1)),
    "experts_all": gla_layer(1, 8, 8, 4.0, 2, mlp=moe(33, 3, 3, limit=0.2)),
    "one_expert": gla_layer(1, 8, 8, 4.0, 2, mlp=moe(16, 1, 1, limit=50.0)),
}


@pytest.mark.parametrize("name", sorted(SINGLE_LAYERS))
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_one_layer_alone(tmp_path, name, dtype):
    """A model of one layer: whole, token by token and in portions of two and three tokens; run once, and passed twice
    with the embedding's output added in between."""
    for loop in (None, (0, 1, 2)):
        config = model(61, 64, [SINGLE_LAYERS[name]], loop=loop)
        folder = make_folder(tmp_path / f"one{bool(loop)}", config, seed=3)
        reqs = {"a": random_tokens(50, 61, 1), "b": random_tokens(19, 61, 2)}
        plain = plain_rows(folder, reqs)
        limits = rounding_limits(folder, reqs) if dtype == "bfloat16" else None
        runner = runner_for(folder, dtype, tokens=128)
        for rid, toks in reqs.items():
            compare_rows(run_steps(runner, whole(rid, toks)), plain, TOL[dtype], limits)
        compare_rows(run_steps(runner, tail_one_by_one("a", reqs["a"], tail=30)), plain, TOL[dtype], limits)
        compare_rows(run_steps(runner, portions("a", reqs["a"], [2, 3])), plain, TOL[dtype], limits)
        compare_rows(run_steps(runner, mixed_trace(reqs, 1, max_live=2)), plain, TOL[dtype], limits)


def test_the_stream_after_every_layer_run(tefavik_folders):
    """The stream that every run of a layer leaves (before the embedding's output is added for the next pass) against the
    plain model's."""
    for name in ("mixed", "awkward"):
        folder = tefavik_folders[name]
        cfg, w = load_plain(folder)
        tokens = random_tokens(37, cfg["vocab"], 6)
        want: list = []
        pt.forward(tokens, w, cfg, want)
        runner = runner_for(folder, "float32")
        planned = runner.plan([StepEntry("tap", tokens, [])])
        runner.storage.reset_slots(runner.manager.take_fresh_slots())
        hb = layout(planned, runner.model.spec.vocab_size, len(runner.groups), runner.manager.slot_tables)
        ctx, _, tables = to_device(hb, runner.model.dtype, runner.model.device, runner.storage.last_token)
        ctx.extras["kv_bound"] = runner.kv_bound(ctx.max_kv_len)
        tap: list = []
        ctx.extras["model_tap"] = tap
        runner.model.forward(ctx, runner.cache_views(tables), runner.storage.states, None)
        runner.release("tap")
        assert len(tap) == len(want)
        for got, ref in zip(tap, want):
            assert float((got.cpu().double() - ref).abs().max()) < 2e-4 * max(1.0, float(ref.abs().max()))


# ---------------------------------------------------------------------------------- cuttings, batches, reuse


@pytest.mark.parametrize("name", sorted(CONFIGS))
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_every_cutting_gives_the_plain_rows(tefavik_folders, name, dtype):
    """Whole prompts, a tail decoded token by token (through recorded steps), portions of changing sizes down to
    two tokens and one, and unequal requests mixed in one batch on a pool so small that pages and slots are used
    again."""
    folder, vocab = tefavik_folders[name], CONFIGS[name]["vocab"]
    reqs = {f"r{i}": random_tokens(n, vocab, 50 + i) for i, n in enumerate((70, 3, 41, 1, 97, 26))}
    plain = plain_rows(folder, reqs)
    limits = rounding_limits(folder, reqs) if dtype == "bfloat16" else None
    runner = runner_for(folder, dtype, tokens=256)
    tol = TOL[dtype]
    for rid, toks in reqs.items():
        compare_rows(run_steps(runner, whole(rid, toks)), plain, tol, limits)
    compare_rows(run_steps(runner, tail_one_by_one("r4", reqs["r4"], tail=40)), plain, tol, limits)
    compare_rows(run_steps(runner, portions("r4", reqs["r4"], [2, 3, 16, 2, 1, 31, 5])), plain, tol, limits)
    compare_rows(run_steps(runner, portions("r0", reqs["r0"], [15, 17, 1, 2])), plain, tol, limits)
    for seed in (1, 2):
        compare_rows(run_steps(runner, mixed_trace(reqs, seed, max_live=4)), plain, tol, limits)
    assert runner.manager.requests == {}
    if dtype == "float32":
        # the same position from different cuttings: the same up to the order of 32-bit sums
        a = run_steps(runner, whole("r2", reqs["r2"]))
        b = run_steps(runner, portions("r2", reqs["r2"], [2, 7]))
        for key in a:
            assert float((a[key] - b[key]).abs().max()) < 2e-4 * max(1.0, float(a[key].abs().max()))


@pytest.mark.parametrize("name", ["mixed", "large_heads"])
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_long_prompts_in_one_step(tefavik_folders, name, dtype):
    """Steps of hundreds of rows, the same step again and again: every row is the plain one's, and the steps' rows are equal
    bit for bit."""
    folder, vocab = tefavik_folders[name], CONFIGS[name]["vocab"]
    reqs = {f"l{i}": random_tokens(n, vocab, 60 + i) for i, n in enumerate((230, 20, 131))}
    plain = plain_rows(folder, reqs)
    limits = rounding_limits(folder, reqs) if dtype == "bfloat16" else None
    runner = runner_for(folder, dtype, tokens=512)
    steps = [{"entries": [(rid, toks, list(range(len(toks)))) for rid, toks in reqs.items()], "end": list(reqs)}]
    first = run_steps(runner, steps)
    compare_rows(first, plain, TOL[dtype], limits)
    for _ in range(3):
        again = run_steps(runner, steps)
        assert all(torch.equal(again[key], row) for key, row in first.items())


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_only_the_last_row_is_wanted(tefavik_folders, dtype):
    """The last block goes on with the wanted rows alone: their experts are their own tokens'."""
    folder, vocab = tefavik_folders["only_pairs"], CONFIGS["only_pairs"]["vocab"]
    reqs = {f"w{i}": random_tokens(n, vocab, 40 + i) for i, n in enumerate((30, 9, 21))}
    plain = plain_rows(folder, reqs)
    limits = rounding_limits(folder, reqs) if dtype == "bfloat16" else None
    runner = runner_for(folder, dtype, tokens=256)
    steps = [{"entries": [(rid, toks, [len(toks) - 1, 2]) for rid, toks in reqs.items()], "end": list(reqs)}]
    compare_rows(run_steps(runner, steps), plain, TOL[dtype], limits)


def test_batch_rows_do_not_depend_on_their_neighbours(tefavik_folders):
    """A request's rows beside other requests are those it has alone (32-bit: up to the order of sums)."""
    folder, vocab = tefavik_folders["mixed"], MIXED["vocab"]
    reqs = {f"r{i}": random_tokens(n, vocab, 70 + i) for i, n in enumerate((33, 5, 18))}
    runner = runner_for(folder, "float32", tokens=256)
    alone = {}
    for rid, toks in reqs.items():
        alone.update(run_steps(runner, whole(rid, toks)))
    together = run_steps(runner, [{"entries": [(rid, toks, list(range(len(toks)))) for rid, toks in reqs.items()], "end": list(reqs)}])
    for key, row in together.items():
        assert float((row - alone[key]).abs().max()) < 2e-4 * max(1.0, float(row.abs().max())), key


@pytest.mark.parametrize("name", ["mixed", "only_states", "awkward"])
def test_slots_and_pages_are_clean_for_their_next_holder(tefavik_folders, name):
    """Two slots and few pages: a request that takes a slot after another finds zero states (the matrices, the keys' sums,
    the running maxima) in every pass of a loop, and its own keys only."""
    folder, vocab = tefavik_folders[name], CONFIGS[name]["vocab"]
    reqs = {f"q{i}": random_tokens(n, vocab, 90 + i) for i, n in enumerate((40, 25, 31, 12, 37))}
    plain = plain_rows(folder, reqs)
    runner = runner_for(folder, "float32", tokens=96, slots=2)
    compare_rows(run_steps(runner, mixed_trace(reqs, 5, max_live=2)), plain, TOL["float32"])
    for rid, toks in reqs.items():
        compare_rows(run_steps(runner, tail_one_by_one(rid, toks, tail=3)), plain, TOL["float32"])


# ---------------------------------------------------------------------------------- marked tokens


def score_of_tokens(w, cfg, last_token: int, distance: int) -> torch.Tensor:
    """The score of every token as a key ``distance`` in front of the last query, of a one-layer model with one head."""
    m, eps = cfg["layers"][0]["mixer"]["left"], cfg["norm"]["eps"]
    p, dims, base = "l0.mix.left", m["rot"]["dims"], m["rot"]["base"]
    h = pt.rms(w["embed"], eps) * w["l0.norm1"]
    q = pt.rms(h[last_token] @ w[f"{p}.q"].T + w[f"{p}.q.b"], eps) * w[f"{p}.q.norm"]
    k = pt.rms(h @ w[f"{p}.k"].T + w[f"{p}.k.b"], eps) * w[f"{p}.k.norm"]
    f = torch.tensor([base ** (-2.0 * i / dims) for i in range(dims // 2)], dtype=torch.float64) * distance
    u, v = q[0:dims:2].clone(), q[1:dims:2].clone()
    q = q.clone()
    q[0:dims:2], q[1:dims:2] = u * torch.cos(f) + v * torch.sin(f), v * torch.cos(f) - u * torch.sin(f)  # turned back by the distance
    return pt.soft_cap(k @ q * m["scale"], m["softcap"])


@pytest.mark.parametrize("chunk, n", [(48, 130), (21, 62), (128, 240), (300, 590)])
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_a_key_that_stands_out_just_inside_and_just_outside_its_chunk(tmp_path, chunk, n, dtype):
    """A sharp attention whose queries prefer one token, put at the first place of the last query's chunk and at the place in
    front of it, at page borders inside the chunk and beside the query: inside, the plain last row moves by it; outside it does
    not (and would, if the chunk were longer); the engine's last rows are the plain model's in a whole prompt, decoded at the
    end, in portions, and with the key itself decoded alone."""
    config = model(64, 32, [pair_layer(attention_branch(1, 1, 16, 32, chunk, rot_dims=4, scale=1.6, softcap=14.0, base=50.0), memory_branch(1, 4, 4))])
    longer = json.loads(json.dumps(config))
    longer["layers"][0]["mixer"]["left"]["mask"]["size"] = 10 * n
    folder = make_folder(tmp_path / "sharp", config, seed=8, edits={
        ".right.out": lambda t: t * 0, ".left.out": lambda t: t * 6.0, ".left.k.b": lambda t: t * 0})
    cfg, w = load_plain(folder)
    runner = runner_for(folder, dtype, tokens=-(-n // 16) * 16 + 16)
    first = (n - 1) // chunk * chunk  # of the last query's chunk
    last = 5
    # tokens whose keys score low wherever they stand
    anywhere = torch.stack([score_of_tokens(w, cfg, last, d) for d in range(n)]).amax(0)
    dull = [t for t in torch.argsort(anywhere).tolist()[:10] if t != last]
    for at in sorted({first, first - 1, first + 1, first - 16, (n - 1) // 16 * 16, (n - 1) // 16 * 16 - 1, n - 2}):
        score = score_of_tokens(w, cfg, last, n - 1 - at)
        score[last] = -1e9
        g = random.Random(at)
        tokens = [g.choice(dull) for _ in range(n - 1)] + [last]

        def marked(token, config):
            return pt.forward(tokens[:at] + [token] + tokens[at + 1 :], w, config)

        # of the best keys the one whose values change the last row most, where the query sees it
        unmarked, sees = pt.forward(tokens, w, cfg), cfg if at >= first else longer
        before = pt.forward(tokens, w, sees)[-1]
        moved, mark = max((float((marked(t, sees)[-1] - before).norm() / before.norm()), t) for t in torch.topk(score, 4).indices.tolist())
        assert moved > 0.2, at
        plain = marked(mark, cfg).float()
        if at < first:
            assert torch.equal(plain[-1], unmarked[-1].float())
        tokens[at] = mark
        cuts = [whole("e", tokens), tail_one_by_one("e", tokens, tail=3), portions("e", tokens, [2, 61])]
        if n - at < 60:
            cuts.append(tail_one_by_one("e", tokens, tail=n - at + 1))
        for steps in cuts:
            got = run_steps(runner, steps)
            compare_rows({k: v for k, v in got.items() if k[1] >= n - 3}, {"e": plain}, TOL[dtype])


def test_one_in_the_denominator_counts_once_however_the_keys_are_cut(tmp_path):
    """A chunk so long that a decoded token's keys are cut among workgroups, with scores far below zero, so that the one in
    the denominator takes most of the weight: without it, or counted twice, the rows would differ."""
    n = 700
    config = model(64, 32, [pair_layer(attention_branch(2, 1, 16, 32, 690, scale=1.0, softcap=8.0), memory_branch(1, 4, 4))])
    # keys against the queries: their biases have opposite directions
    v = torch.randn(16, generator=torch.Generator().manual_seed(1))
    folder = make_folder(tmp_path / "one", config, seed=12, edits={
        ".right.out": lambda t: t * 0, ".left.q.b": lambda t: v.repeat(2) * 6.0, ".left.k.b": lambda t: v * -6.0})
    cfg, w = load_plain(folder)
    tokens = random_tokens(n, 64, 3)
    plain = {"s": pt.forward(tokens, w, cfg).float()}
    runner = runner_for(folder, "float32", tokens=720)
    for steps in (whole("s", tokens), tail_one_by_one("s", tokens, tail=30), portions("s", tokens, [2, 130, 1])):
        compare_rows(run_steps(runner, steps), plain, TOL["float32"])


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("kind", ["gla", "memory"])
def test_a_token_far_back_shows_through_the_recurrence(tmp_path, kind, dtype):
    """A recurrence that hardly forgets: the first token's mark is still in the last row 300 tokens on, in a whole prompt,
    token by token and across portions."""
    if kind == "gla":
        layer, edits = gla_layer(2, 16, 16, 16.0, 4), {".a2.b": lambda t: t * 0 + 9.0, ".a2": lambda t: t * 0.1}
    else:
        layer = pair_layer(attention_branch(1, 1, 8, 8, 4), memory_branch(2, 16, 16))
        edits = {".f.b": lambda t: t * 0 + 30.0, ".left.out": lambda t: t * 0}
    config = model(64, 32, [layer])
    folder = make_folder(tmp_path / "slow", config, seed=3, edits=edits)
    cfg, w = load_plain(folder)
    n = 300
    tokens = [t % 63 for t in random_tokens(n, 64, 9)]
    unmarked = pt.forward(tokens, w, cfg)[-1]
    tokens[0] = 63
    plain = pt.forward(tokens, w, cfg).float()
    assert float((plain[-1] - unmarked).norm() / unmarked.norm()) > 5e-3
    runner = runner_for(folder, dtype, tokens=448)
    for steps in (whole("e", tokens), tail_one_by_one("e", tokens, tail=250), portions("e", tokens, [2, 61, 1])):
        got = run_steps(runner, steps)
        compare_rows({k: v for k, v in got.items() if k[1] >= n - 3}, {"e": plain}, 3e-5 if dtype == "float32" else 2e-2)


@pytest.mark.parametrize("bias", [-7.0, 0.0, 7.0])
def test_the_running_maximum_starts_at_zero_and_is_carried(tmp_path, bias):
    """Input gates far below zero (the maximum stays near its start and the read-out is divided by its exponential), around
    zero and far above: from the first token on, in every cutting."""
    config = model(64, 32, [pair_layer(attention_branch(1, 1, 8, 8, 4), memory_branch(3, 8, 8, cap=20.0))])
    folder = make_folder(tmp_path / "max", config, seed=6, edits={".i.b": lambda t: t * 0 + bias, ".left.out": lambda t: t * 0})
    tokens = random_tokens(60, 64, 4)
    plain = plain_rows(folder, {"c": tokens})
    runner = runner_for(folder, "float32", tokens=64)
    for steps in (whole("c", tokens), portions("c", tokens, [1]), portions("c", tokens, [2, 1, 5]), tail_one_by_one("c", tokens, tail=59)):
        compare_rows(run_steps(runner, steps), plain, TOL["float32"])


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_portions_on_both_sides_of_the_recurrences_borders(tmp_path, dtype):
    """Prompts that end at, one before and one behind the borders of the recurrences' groups of tokens, and cuts that move
    them: every row is the plain one's."""
    config = model(64, 48, [pair_layer(attention_branch(2, 1, 16, 16, 33), memory_branch(2, 32, 24)), gla_layer(2, 24, 48, 16.0, 8)])
    folder = make_folder(tmp_path / "chunks", config, seed=6)
    tokens = random_tokens(200, 64, 4)
    plain = plain_rows(folder, {"c": tokens})
    limits = rounding_limits(folder, {"c": tokens}) if dtype == "bfloat16" else None
    runner = runner_for(folder, dtype, tokens=256)
    for n in (15, 16, 17, 63, 64, 65, 80, 127, 128, 129, 193):
        compare_rows(run_steps(runner, whole("c", tokens[:n])), plain, TOL[dtype], limits)
    for sizes in ([64], [63, 1], [65], [16], [17, 15], [1, 64, 128], [100, 2]):
        compare_rows(run_steps(runner, portions("c", tokens, sizes)), plain, TOL[dtype], limits)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_first_tokens_of_a_sequence(tefavik_folders, dtype):
    """Requests of one, two and three tokens, whole and token by token: states and maxima that start at zero, one key, the
    first page half empty."""
    for name in sorted(CONFIGS):
        folder, vocab = tefavik_folders[name], CONFIGS[name]["vocab"]
        reqs = {f"s{n}": random_tokens(n, vocab, 30 + n) for n in (1, 2, 3, 6)}
        plain = plain_rows(folder, reqs)
        limits = rounding_limits(folder, reqs) if dtype == "bfloat16" else None
        runner = runner_for(folder, dtype, tokens=64)
        for rid, toks in reqs.items():
            compare_rows(run_steps(runner, whole(rid, toks)), plain, TOL[dtype], limits)
            compare_rows(run_steps(runner, portions(rid, toks, [1])), plain, TOL[dtype], limits)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_long_decoding(tefavik_folders, dtype):
    """A short prompt and 400 tokens decoded one by one through recorded steps."""
    folder, vocab = tefavik_folders["mixed"], MIXED["vocab"]
    tokens = random_tokens(420, vocab, 77)
    plain = plain_rows(folder, {"d": tokens})
    limits = rounding_limits(folder, {"d": tokens}) if dtype == "bfloat16" else None
    runner = runner_for(folder, dtype, tokens=448)
    got = run_steps(runner, tail_one_by_one("d", tokens, tail=400))
    compare_rows(got, plain, TOL[dtype], limits)
    assert all(step.captured for step in runner.recorded.values()) and runner.recorded


# ---------------------------------------------------------------------------------- the entry points


@pytest.mark.parametrize("name", ["mixed", "awkward", "only_states"])
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_greedy_generation_through_the_engine(tefavik_folders, dtype, name):
    """``Engine.generate``: the scheduler cuts prompts into portions beside decoding requests, whose tokens (and so their
    experts) are read from what was sampled; the tokens are the plain model's greedy tokens (in bfloat16: each token is, for
    the plain logits of its own history, within rounding of the best)."""
    from tokasaurus_amd.config.engine_config import EngineConfig
    from tokasaurus_amd.engine.engine import Engine
    from tokasaurus_amd.sampling import SamplingParams

    folder, vocab = tefavik_folders[name], CONFIGS[name]["vocab"]
    prompts = [random_tokens(n, vocab, 10 + n) for n in (5, 40, 23, 1, 64)]
    engine = Engine(EngineConfig(model=str(folder), dtype=dtype, page_size=PAGE, kv_cache_num_tokens=512, max_seqs_per_forward=3,
                                 max_tokens_per_forward=24, allocator_sanity_checks=True))
    done = engine.generate(prompts, SamplingParams(temperature=0.0, max_tokens=12, ignore_eos=True))
    cfg, w = load_plain(folder)
    for prompt, c in zip(prompts, done):
        assert len(c.tokens) == 12 and c.finish_reason == "length"
        ids = list(prompt)
        for tok in c.tokens:
            logits = pt.forward(ids, w, cfg)[-1]
            if dtype == "float32":
                assert tok == int(logits.argmax()), f"token {tok}, plain {int(logits.argmax())}"
            else:
                assert float(logits.max() - logits[tok]) < 0.15 * float(logits.std()), f"{tok} lies below the best"
            ids.append(tok)
    assert engine.runner.manager.requests == {}


def test_command_line_and_trace_replay(tefavik_folders, tmp_path):
    """``bin/toka`` generates with the design and ``bin/trace_run`` replays a trace of it."""
    root = os.path.join(os.path.dirname(os.path.abspath(__file__)), "..")
    folder, vocab = tefavik_folders["mixed"], MIXED["vocab"]
    proc = subprocess.run([sys.executable, os.path.join(root, "bin", "toka"), f"model={folder}", "dtype=float32",
                           "prompt_ids=([[1, 2, 3]])", "max_tokens=4", "kv_cache_num_tokens=256"],
                          capture_output=True, text=True, timeout=300)
    assert proc.returncode == 0, proc.stderr[-2000:]
    a, b = random_tokens(21, vocab, 1), random_tokens(40, vocab, 2)
    steps = [
        {"step": 0, "entries": [{"id": "a", "tokens": a[:17], "want": [0, 16]}], "end": []},
        {"step": 1, "entries": [{"id": "a", "tokens": a[17:18], "want": [0]}, {"id": "b", "tokens": b[:33], "want": [32]}], "end": []},
        {"step": 2, "entries": [{"id": "b", "tokens": b[33:35], "want": []}, {"id": "a", "tokens": a[18:], "want": [2]}], "end": ["a"]},
        {"step": 3, "entries": [{"id": "b", "tokens": b[35:], "want": [4]}], "end": ["b"]},
    ]
    out = tmp_path / "out"
    proc = subprocess.run([sys.executable, os.path.join(root, "bin", "trace_run"), "--model", str(folder), "--dtype", "float32",
                           "--out", str(out), "--max-tokens", "128"], input="\n".join(json.dumps(s) for s in steps) + "\n",
                          capture_output=True, text=True, timeout=300)
    assert proc.returncode == 0, proc.stderr[-2000:]
    assert [l for l in proc.stdout.splitlines() if l.startswith("done")] == [f"done {i}" for i in range(4)]
    plain = plain_rows(folder, {"a": a, "b": b})
    want = {0: [("a", 0), ("a", 16)], 1: [("a", 17), ("b", 32)], 2: [("a", 20)], 3: [("b", 39)]}
    for step, rows in want.items():
        got = torch.from_numpy(np.fromfile(out / f"{step}.f32", dtype="<f4").reshape(len(rows), vocab).copy())
        compare_rows({key: got[i] for i, key in enumerate(rows)}, plain, TOL["float32"])


# ---------------------------------------------------------------------------------- drawn configurations


def random_config(seed: int) -> dict:
    """A model drawn from lists of comfortable and awkward sizes."""
    rng = random.Random(seed)
    width = rng.choice([32, 48, 90, 64, 100])
    layers = []
    for _ in range(rng.choice([1, 2, 3, 4])):
        experts = rng.choice([1, 2, 5, 8])
        mlp = rng.choice([None, moe(rng.choice([8, 20, 32, 33]), experts, rng.randint(1, experts), limit=rng.choice([0.5, 2.0, 7.0])),
                          moe(rng.choice([16, 40]), 8, rng.choice([1, 2]))])
        if rng.random() < 0.5:
            layers.append(gla_layer(rng.choice([1, 2, 3, 6]), rng.choice([4, 15, 16, 31, 64, 100]), rng.choice([4, 9, 16, 20, 48]),
                                    rng.choice([1.0, 4.0, 16.0]), rng.choice([1, 8, 16, 33]), mlp=mlp))
        else:
            kv_heads = rng.choice([1, 2, 3])
            dim = rng.choice([4, 8, 15, 16, 32])
            left = attention_branch(kv_heads * rng.choice([1, 2, 4]), kv_heads, dim, rng.choice([5, 8, 16, 32, 48]),
                                    rng.choice([1, 3, 8, 16, 29, 64, 100]), rot_dims=2 * rng.randint(1, dim // 2), scale=rng.choice([0.1, 0.5]),
                                    softcap=rng.choice([3.0, 30.0]), base=rng.choice([50.0, 10000.0]))
            right = memory_branch(rng.choice([1, 2, 5]), rng.choice([4, 15, 16, 31, 64]), rng.choice([4, 9, 16, 20, 48]), cap=rng.choice([2.0, 15.0]))
            layers.append(pair_layer(left, right, mlp=mlp))
    n = len(layers)
    start = rng.randrange(n)
    loop = rng.choice([None, (start, rng.randint(start + 1, n), rng.choice([1, 2, 3]))])
    return model(rng.choice([40, 97, 130]), width, layers, eps=rng.choice([1e-6, 1e-5]), loop=loop)


@pytest.mark.parametrize("seed", range(12))
def test_random_configurations(tmp_path, seed):
    config = random_config(seed)
    reqs = {f"r{i}": random_tokens(n, config["vocab"], 20 * seed + i) for i, n in enumerate((90, 2, 37, 130))}
    folder = make_folder(tmp_path / "drawn", config, seed=seed)
    plain = plain_rows(folder, reqs)
    for dtype in ("float32", "bfloat16"):
        limits = rounding_limits(folder, reqs) if dtype == "bfloat16" else None
        runner = runner_for(folder, dtype, tokens=320)
        for rid, toks in reqs.items():
            compare_rows(run_steps(runner, whole(rid, toks)), plain, TOL[dtype], limits)
        compare_rows(run_steps(runner, tail_one_by_one("r3", reqs["r3"], tail=70)), plain, TOL[dtype], limits)
        compare_rows(run_steps(runner, portions("r3", reqs["r3"], [2, 3, 16, 2, 1, 31, 5])), plain, TOL[dtype], limits)
        compare_rows(run_steps(runner, mixed_trace(reqs, seed, max_live=3)), plain, TOL[dtype], limits)
        assert runner.manager.requests == {}
