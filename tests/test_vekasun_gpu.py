"""Vekasun through the engine against the plain model: every mechanism alone, prompts against
token-by-token decoding, portions down to two tokens and one, unequal requests in one batch on pages
and slots that are used again, keys at page borders and far back, tokens on both sides of the borders of the
recurrence's chunks, first tokens, long decoding, and greedy generation through ``Engine.generate``."""

from __future__ import annotations

import json
import os
import random
import subprocess
import sys

import numpy as np
import pytest
import torch

import plain_vekasun as pv
from replay_helpers import mixed_trace, portions, run_steps, tail_one_by_one, whole
from tiny_models import random_tokens
from tokasaurus_amd.engine.batch import StepEntry, layout, to_device
from tokasaurus_amd.engine.runner import ModelRunner
from tokasaurus_amd.kernels import ops
from vekasun_models import (CONFIGS, MIXED, STEADY, TOL, compare_rows, latent_layer, load_plain, make_folder, mamba_layer, model, moe,
                            plain_rows, rounding_limits)

pytestmark = pytest.mark.gpu
PAGE = 16


@pytest.fixture(scope="module")
def vekasun_folders(tmp_path_factory):
    root = tmp_path_factory.mktemp("vekasun")
    return {(name, steady): make_folder(root / f"{name}{int(steady)}", cfg, seed=5 + i, steady_choice=steady)
            for i, (name, cfg) in enumerate(sorted(CONFIGS.items())) for steady in (False, True)}


def runner_for(folder, dtype, tokens=512, slots=4, **kw):
    return ModelRunner.from_folder(str(folder), dtype, page_size=PAGE, num_pages=tokens // PAGE, max_slots=slots, **kw)


def i32(v):
    return torch.tensor(v, dtype=torch.int32, device="cuda")


def step_arrays(lens, slots, held=None):
    """q_start, each token's request, slots and positions of a step that brings ``lens`` tokens behind ``held``."""
    starts = [0]
    for n in lens:
        starts.append(starts[-1] + n)
    held = held or [0] * len(lens)
    req = [r for r, n in enumerate(lens) for _ in range(n)]
    pos = [h + i for n, h in zip(lens, held) for i in range(n)]
    return i32(starts), i32(req), i32(slots), i32(pos)


# ---------------------------------------------------------------------------------- kernels alone


SPACE_CASES = [  # heads, groups, state, value size, taps, lengths of the requests
    (2, 1, 16, 16, 4, [1, 1, 1]), (4, 2, 12, 6, 3, [3, 40, 1, 9]), (2, 2, 50, 20, 2, [33, 2]), (1, 1, 64, 64, 4, [64, 65, 63]),
    (8, 2, 128, 64, 4, [130, 1, 20]), (3, 1, 96, 24, 1, [200]), (2, 1, 160, 17, 5, [70, 129]), (1, 1, 256, 33, 4, [100, 16]),
    (2, 1, 300, 8, 4, [40, 3]), (1, 1, 512, 5, 3, [6, 20]), (16, 8, 10, 9, 6, [1, 1]), (2, 1, 200, 70, 4, [1, 1, 1, 1]),
]


@pytest.mark.parametrize("heads, groups, N, dv, taps, lens", SPACE_CASES)
@pytest.mark.parametrize("storage", [torch.float32, torch.bfloat16])
def test_state_space_kernel(heads, groups, N, dv, taps, lens, storage):
    """Convolution, step sizes and the recurrence on random sums, from random matrices and inputs in shuffled slots,
    against the plain functions; then the same tokens cut in two steps; then the last token alone."""
    torch.manual_seed(N + dv)
    H, G, n = heads, groups, sum(lens)
    C = H * dv + 2 * G * N
    proj = torch.randn(n, 7 + C + H + 2)
    x_off, dt_off = 7, 7 + C
    conv_w, conv_b = torch.randn(taps, C) * 0.5, torch.randn(C) * 0.3
    a_log, dt_bias, skip = torch.randn(H) - 1.0, torch.randn(H) * 0.5, torch.randn(H)
    a_log[0] = -6.0  # a head that hardly forgets
    slots = list(range(len(lens)))[::-1]
    size, ring = ops.state_space_sizes(H, G, N, dv, taps)
    # requests that hold tokens already: random matrices, and their last inputs in the places of their positions
    held = [5 + 3 * r for r in range(len(lens))]
    before = [torch.randn(max(held), C) for _ in lens]
    state0 = torch.zeros(len(lens) + 1, size)
    state0[:, : H * dv * N] = torch.randn(len(lens) + 1, H * dv * N) * 0.3
    if taps > 1:
        for r, s in enumerate(slots):
            for p in range(held[r] - taps + 1, held[r]):
                if p >= 0:
                    state0[s, ring + (p % taps) * C : ring + (p % taps + 1) * C] = before[r][p]

    def run(state, rows, lens_, slots_, held_, longest=None):
        q_start, req, slot_t, pos = step_arrays(lens_, slots_, held_)
        return ops.state_space(rows.cuda(), x_off, dt_off, conv_w.cuda(), conv_b.cuda(), a_log.cuda(), dt_bias.cuda(), skip.cuda(), state,
                               q_start, req, slot_t, pos, H, G, N, dv, longest=longest, storage=storage).cpu()

    state = state0.clone().cuda()
    y = run(state, proj, lens, slots, held, max(lens))
    d = lambda t: t.double()  # noqa: E731
    tol = dict(atol=3e-4, rtol=3e-4)
    at, matrices = 0, []
    for r, ln in enumerate(lens):
        inputs = torch.cat([before[r][max(held[r] - taps + 1, 0) : held[r]], proj[at : at + ln, x_off : x_off + C]])
        u = pv.silu(pv.causal_convolution(d(inputs), d(conv_w).t(), d(conv_b)))[inputs.shape[0] - ln :]
        if storage == torch.bfloat16:
            u = u.float().bfloat16().double()
        x, B, Cc = torch.split(u, [H * dv, G * N, G * N], dim=-1)
        x, B, Cc = x.view(ln, H, dv), B.view(ln, G, N), Cc.view(ln, G, N)
        dt = pv.softplus(d(proj[at : at + ln, dt_off : dt_off + H]) + d(dt_bias))
        S = d(state0[slots[r], : H * dv * N]).view(H, dv, N).clone()
        want = torch.zeros(ln, H, dv, dtype=torch.float64)
        for t in range(ln):
            Bt, Ct = B[t].repeat_interleave(H // G, 0), Cc[t].repeat_interleave(H // G, 0)
            S = torch.exp(-torch.exp(d(a_log)) * dt[t])[:, None, None] * S + dt[t][:, None, None] * x[t][:, :, None] * Bt[:, None, :]
            want[t] = (S * Ct[:, None, :]).sum(-1) + d(skip)[:, None] * x[t]
        scale = float(want.abs().max())
        # (in bfloat16 a few numbers of the convolution round the other way than the plain function's)
        slack = (2e-2 if storage == torch.bfloat16 else 1e-4) * scale
        assert float((d(y[at : at + ln]) - want.view(ln, -1)).abs().max()) < slack, r
        rms = float((d(y[at : at + ln]) - want.view(ln, -1)).pow(2).mean().sqrt() / want.pow(2).mean().sqrt())
        assert rms < (1e-3 if storage == torch.bfloat16 else 1e-5), (r, rms)
        got = d(state[slots[r], : H * dv * N].cpu()).view(H, dv, N)
        assert float((got - S).pow(2).mean().sqrt() / S.pow(2).mean().sqrt()) < (1e-3 if storage == torch.bfloat16 else 1e-5)
        if taps > 1:  # the last inputs in the places of their positions
            end = held[r] + ln
            for p in range(max(end - taps, held[r]), end):
                entry = state[slots[r], ring + (p % taps) * C : ring + (p % taps + 1) * C].cpu()
                assert torch.equal(entry, proj[at + p - held[r], x_off : x_off + C])
        matrices.append(got)
        at += ln
    assert torch.equal(state[len(lens)].cpu(), state0[len(lens)])  # a slot of no request stays as it was
    # the same tokens in two steps, cut inside every request that has two tokens or more, then once more with the last alone
    for cut in ([max(1, ln // 3) if ln > 1 else 1 for ln in lens], [max(1, ln - 1) for ln in lens]):
        state2 = state0.clone().cuda()
        base = [sum(lens[:r]) for r in range(len(lens))]
        first = torch.cat([proj[b : b + c] for b, c in zip(base, cut)])
        y1 = run(state2, first, cut, slots, held, max(cut))
        keep = [r for r in range(len(lens)) if lens[r] > cut[r]]
        if keep:
            second = torch.cat([proj[base[r] + cut[r] : base[r] + lens[r]] for r in keep])
            rest = [lens[r] - cut[r] for r in keep]
            y2 = run(state2, second, rest, [slots[r] for r in keep], [held[r] + cut[r] for r in keep], max(rest))
        a1 = a2 = 0
        for r, ln in enumerate(lens):
            assert torch.allclose(y1[a1 : a1 + cut[r]], y[base[r] : base[r] + cut[r]], **tol)
            a1 += cut[r]
            if r in keep:
                assert torch.allclose(y2[a2 : a2 + ln - cut[r]], y[base[r] + cut[r] : base[r] + ln], **tol), (r, cut)
                a2 += ln - cut[r]
        assert torch.allclose(state2, state, **tol)
        if storage == torch.float32:  # token by token in every form: the same bits
            assert torch.equal(state2, state)


@pytest.mark.parametrize("storage", [torch.float32, torch.bfloat16])
def test_steep_decays_stay_finite(storage):
    """Decays whose logarithms sum to hundreds over a chunk: nothing overflows, and only the last tokens show."""
    torch.manual_seed(9)
    H, G, N, dv, taps, ln = 2, 1, 32, 16, 2, 150
    C = H * dv + 2 * N
    proj = torch.randn(ln, C + H) + 1.0
    size, _ = ops.state_space_sizes(H, G, N, dv, taps)
    w, b, a_log, bias, skip = torch.randn(taps, C), torch.randn(C), torch.tensor([2.5, 4.5]), torch.tensor([3.0, 6.0]), torch.zeros(H)
    q_start, req, slots, pos = step_arrays([ln], [0])
    y = ops.state_space(proj.cuda(), 0, C, w.cuda(), b.cuda(), a_log.cuda(), bias.cuda(), skip.cuda(), torch.zeros(2, size).cuda(), q_start,
                        req, slots, pos, H, G, N, dv, storage=storage).cpu().double()
    u = pv.silu(pv.causal_convolution(proj[:, :C].double(), w.double().t(), b.double()))
    if storage == torch.bfloat16:
        u = u.float().bfloat16().double()
    x, B, Cc = torch.split(u, [H * dv, N, N], dim=-1)
    dt = pv.softplus(proj[:, C:].double() + bias.double())
    want = pv.state_space(x.view(ln, H, dv), B[:, None], Cc[:, None], dt, a_log.double(), skip.double()).view(ln, -1)
    assert torch.isfinite(y).all()
    assert float((y - want).pow(2).mean().sqrt() / want.pow(2).mean().sqrt()) < (2e-3 if storage == torch.bfloat16 else 1e-5)


@pytest.mark.parametrize("groups, size", [(1, 1024), (2, 300), (3, 20), (8, 512), (1, 9000), (5, 7)])
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_gate_then_norm_kernel(groups, size, dtype):
    torch.manual_seed(size)
    n = 5
    y, z, w = torch.randn(n, groups * size), torch.randn(n, groups * size + 24), torch.randn(groups * size)
    for off in (0, 5, 8):  # gates that start at a multiple of 16 bytes and that do not
        got = ops.gate_group_norm(y.cuda(), z.cuda()[:, off : off + groups * size], w.cuda(), 1e-5, groups, dtype)
        want = pv.gate_then_norm(y.double(), z[:, off : off + groups * size].double(), w.double(), groups, 1e-5)
        tol = 1e-5 if dtype == torch.float32 else 2e-2
        assert torch.allclose(got.cpu().double(), want, atol=tol, rtol=tol)


@pytest.mark.parametrize("width", [70, 256, 1028, 9000])
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_layer_norm_of_the_updated_stream(width, dtype):
    """x + branch + row and the layer norm's rows of it in one pass, on rows with a large mean; the RMS norm with the
    same row; every piece alone."""
    torch.manual_seed(width)
    x, a, row, w = torch.randn(6, width) + 20.0, torch.randn(6, width), torch.randn(width), torch.randn(width)
    tol = 2e-5 if dtype == torch.float32 else 2e-2
    for branch in (None, a):
        for add in (None, row):
            want = x.double() + (branch.double() if branch is not None else 0) + (add.double() if add is not None else 0)
            for center in (True, False):
                xs, h, _ = ops.residual_norm(x.clone().cuda(), (branch.cuda() if branch is not None else None, None), weights=(w.cuda(), None),
                                             eps=1e-5, out_dtype=dtype, add_row=add.cuda() if add is not None else None, center=center)
                ref = pv.layer_norm(want, w.double(), 1e-5) if center else pv.rms(want, 1e-5) * w.double()
                assert torch.allclose(xs.cpu().double(), want, atol=1e-5)
                assert torch.allclose(h.cpu().double(), ref, atol=tol * 3, rtol=tol), (branch is not None, add is not None, center)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_rotation_of_a_head_s_leading_part(dtype):
    torch.manual_seed(7)
    heads, d, rot = 3, 20, 8
    x = torch.randn(6, heads * d + 4).to(dtype)
    freq = torch.tensor([30.0 ** (-2.0 * i / rot) for i in range(rot // 2)], dtype=torch.float32)
    got = ops.rotate_heads_(x.clone().cuda(), i32(list(range(6))), freq.cuda(), heads, d, True).cpu().double()
    want = x.double().clone()
    for h in range(heads):
        want[:, h * d : h * d + rot] = pv.rotate_halves(x.double()[:, h * d : h * d + rot], 30.0)
    tol = 1e-5 if dtype == torch.float32 else 2e-2
    assert torch.allclose(got, want, atol=tol, rtol=tol)
    assert torch.equal(got[:, heads * d :], x.double()[:, heads * d :])
    near = ops.rotate_heads_(x.clone().cuda(), i32([2] * 6), freq.cuda(), heads, d, False).cpu().double()  # neighbouring elements
    c, s = np.cos(2.0), np.sin(2.0)
    assert torch.allclose(near[:, 0], x[:, 0].double() * c - x[:, 1].double() * s, atol=tol * 3)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_a_matrix_a_head_with_a_rotation_and_a_gate(dtype):
    """The leading part turned instead of multiplied by its identity block: the bits of turning first and multiplying
    then; the result times a gate's sigmoid.  Neighbouring pairs and halves, a rotated part longer than a block of rows."""
    torch.manual_seed(8)
    for heads, dr, d, r, halves in ((3, 6, 10, 20, True), (2, 40, 8, 32, True), (2, 48, 8, 30, False), (1, 2, 3, 5, False)):
        n = 7
        w = torch.zeros(heads, dr + r, dr + d)
        w[:, :dr, :dr] = torch.eye(dr)
        w[:, dr:, dr:] = torch.randn(heads, r, d)
        w, x, pos = w.to(dtype).cuda(), torch.randn(n, heads * (dr + d) + 3).to(dtype).cuda(), i32([0, 5, 9, 100, 3, 2, 1])
        freq = torch.tensor([50.0 ** (-2.0 * i / dr) for i in range(dr // 2)], dtype=torch.float32).cuda()
        want = ops.head_linear(ops.rotate_heads_(x.clone(), pos, freq, heads, dr + d, halves, 1.25), w)
        got = ops.head_linear(x, w, positions=pos, freq=freq, pair_halves=halves, rotation_scale=1.25)
        assert torch.equal(got, want)
        gate = torch.randn(n, heads * (dr + r) + 5).to(dtype).cuda()[:, 5:]
        gated = ops.head_linear(x, w, gate=gate).double().cpu()
        ref = torch.einsum("thi,hoi->tho", x[:, : heads * (dr + d)].double().cpu().view(n, heads, dr + d), w.double().cpu()).reshape(n, -1)
        tol = 1e-5 if dtype == torch.float32 else 2e-2
        assert torch.allclose(gated, ref * torch.sigmoid(gate.double().cpu()), atol=tol, rtol=tol)


def test_router_with_sigmoid_scores():
    torch.manual_seed(4)
    for experts, top, width in ((6, 3, 40), (1, 1, 16), (130, 8, 64), (5, 5, 24)):
        h, wr = torch.randn(70, width), torch.randn(experts, width) * 0.3
        want_ids, want_w = pv.route(h.double(), {"p.router": wr.double()}, "p", {"top": top})
        ids, wts, gate = ops.expert_route(h.cuda(), wr.cuda(), None, 1, 1, top, sigmoid_scores=True)
        assert gate is None and torch.equal(ids.cpu().long(), want_ids) and torch.allclose(wts.cpu().double(), want_w, atol=1e-6)
        corr = torch.randn(experts) * 0.5  # with a correction the choice is by the sum, the weights are the scores
        ids, wts, _ = ops.expert_route(h.cuda(), wr.cuda(), corr.cuda(), 1, 1, top, sigmoid_scores=True)
        s = torch.sigmoid(h.double() @ wr.double().t())
        assert torch.equal(ids.cpu().long(), torch.topk(s + corr.double(), top, dim=-1).indices)
        assert torch.allclose(wts.cpu().double(), torch.gather(s, 1, ids.cpu().long()), atol=1e-6)
    # logits so large that the scores are all one: the larger logit still comes first
    h = torch.ones(3, 8)
    wr = torch.stack([torch.full((8,), v) for v in (10.0, 12.0, 11.0)])
    ids, wts, _ = ops.expert_route(h.cuda(), wr.cuda(), None, 1, 1, 2, sigmoid_scores=True)
    assert ids.cpu().tolist() == [[1, 2]] * 3 and torch.equal(wts.cpu(), torch.ones(3, 2))


@pytest.mark.parametrize("T, E, W, F, top", [(9, 5, 24, 12, 3), (70, 5, 24, 16, 3), (150, 7, 40, 72, 2), (33, 40, 64, 8, 1), (260, 4, 128, 136, 4), (300, 3, 72, 200, 2)])
def test_experts_that_read_weighted_rows(T, E, W, F, top):
    """sum of expert(weight * h): pair by pair for few tokens, sorted by expert into tiles for many (bfloat16); an
    identity expert, an empty place, an expert that nobody chose."""
    torch.manual_seed(4)
    w = {}
    for e in range(E):
        w.update({f"f.e{e}.gate": torch.randn(F, W) / 5, f"f.e{e}.up": torch.randn(F, W) / 5, f"f.e{e}.down": torch.randn(W, F) / 3})
    w = {k: v.bfloat16().double() for k, v in w.items()}
    h = torch.randn(T, W).bfloat16().double()
    ids = torch.randint(0, E + 1, (T, top), dtype=torch.int32)
    ids[ids == 1] = 0
    if top > 1:
        ids[0, 1] = -1
    wts = torch.rand(T, top) + 0.1
    want = torch.zeros(T, W, dtype=torch.float64)
    for t in range(T):
        for k in range(top):
            e = int(ids[t, k])
            if e >= 0:
                want[t] += pv.expert(wts[t, k].double() * h[t : t + 1], w, f"f.e{e}")[0] if e < E else wts[t, k].double() * h[t]
    gu = torch.stack([torch.cat([w[f"f.e{e}.gate"], w[f"f.e{e}.up"]]) for e in range(E)])
    dn = torch.stack([w[f"f.e{e}.down"] for e in range(E)])
    for dtype, tol in ((torch.float32, 1e-5), (torch.bfloat16, 3e-2)):
        got = ops.expert_mix(h.to(dtype).cuda(), gu.to(dtype).cuda(), dn.to(dtype).cuda(), ids.cuda(), wts.cuda(), weights_on_input=True)
        rel = (got.cpu().double() - want).norm(dim=-1) / want.norm(dim=-1).clamp_min(1e-6)
        assert float(rel.max()) < tol, f"{dtype}: rows {torch.nonzero(rel > tol).flatten().tolist()[:8]} of {T}"


# ---------------------------------------------------------------------------------- one mechanism a model


SINGLE_LAYERS = {
    "states": mamba_layer(2, 16, 16, 1, 1, 4),
    "states_one_group_a_head": mamba_layer(4, 8, 32, 4, 4, 3),
    "states_odd_sizes": mamba_layer(3, 10, 7, 3, 5, 2),
    "states_large": mamba_layer(2, 64, 128, 1, 2, 4),
    "states_one_tap": mamba_layer(2, 16, 8, 2, 1, 1),
    "states_many_taps": mamba_layer(1, 24, 40, 1, 1, 9),
    "states_of_one_row_and_column": mamba_layer(2, 1, 1, 1, 1, 4),
    "latent": latent_layer(4, 16, 16, 16, 32, 48, 0.3),
    "latent_one_head": latent_layer(1, 32, 8, 16, 16, 24, 0.3, base=100.0),
    "latent_odd_sizes": latent_layer(3, 9, 6, 7, 11, 13, 0.3),
    "latent_many_heads": latent_layer(16, 16, 4, 32, 24, 60, 0.3),
    "latent_large": latent_layer(4, 64, 64, 128, 96, 192, 0.1, base=500000.0),
    "latent_larger_than_the_tile_kernel": latent_layer(2, 16, 16, 16, 24, 256, 0.3),
    "experts": mamba_layer(1, 8, 8, 1, 1, 2, mlp=moe(24, 7, 2)),
    "experts_one_of_many": latent_layer(2, 16, 8, 16, 16, 24, 0.3, mlp=moe(10, 20, 1)),
    "experts_all": mamba_layer(1, 8, 8, 1, 1, 2, mlp=moe(33, 3, 3)),
    "one_expert": mamba_layer(1, 8, 8, 1, 1, 2, mlp=moe(16, 1, 1)),
}


@pytest.mark.parametrize("name", sorted(SINGLE_LAYERS))
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_one_layer_alone(tmp_path, name, dtype):
    """A model of one layer: whole, token by token and in portions of two and three tokens; run once, and passed twice
    with an added row each time."""
    for loop in (None, (0, 1, 2)):
        config = model(61, 64, [SINGLE_LAYERS[name]], loop=loop)
        folder = make_folder(tmp_path / f"one{bool(loop)}", config, seed=3, steady_choice=STEADY[dtype])
        reqs = {"a": random_tokens(50, 61, 1), "b": random_tokens(19, 61, 2)}
        plain = plain_rows(folder, reqs)
        limits = rounding_limits(folder, reqs) if dtype == "bfloat16" else None
        runner = runner_for(folder, dtype, tokens=128)
        for rid, toks in reqs.items():
            compare_rows(run_steps(runner, whole(rid, toks)), plain, TOL[dtype], limits)
        compare_rows(run_steps(runner, tail_one_by_one("a", reqs["a"], tail=30)), plain, TOL[dtype], limits)
        compare_rows(run_steps(runner, portions("a", reqs["a"], [2, 3])), plain, TOL[dtype], limits)
        compare_rows(run_steps(runner, mixed_trace(reqs, 1, max_live=2)), plain, TOL[dtype], limits)


def test_the_stream_after_every_layer_run(vekasun_folders):
    """The stream that every run of a layer leaves (before the row of the next pass is added) against the plain model's."""
    for name in ("mixed", "awkward"):
        folder = vekasun_folders[name, False]
        cfg, w = load_plain(folder)
        tokens = random_tokens(37, cfg["vocab"], 6)
        want: list = []
        pv.forward(tokens, w, cfg, want)
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
def test_every_cutting_gives_the_plain_rows(vekasun_folders, name, dtype):
    """Whole prompts, a tail decoded token by token (through recorded steps), portions of changing sizes down to
    two tokens and one, and unequal requests mixed in one batch on a pool so small that pages and slots are used
    again."""
    folder, vocab = vekasun_folders[name, STEADY[dtype]], CONFIGS[name]["vocab"]
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


def test_batch_rows_do_not_depend_on_their_neighbours(vekasun_folders):
    """A request's rows beside other requests are those it has alone (32-bit: up to the order of sums)."""
    folder, vocab = vekasun_folders["mixed", False], MIXED["vocab"]
    reqs = {f"r{i}": random_tokens(n, vocab, 70 + i) for i, n in enumerate((33, 5, 18))}
    runner = runner_for(folder, "float32", tokens=256)
    alone = {}
    for rid, toks in reqs.items():
        alone.update(run_steps(runner, whole(rid, toks)))
    together = run_steps(runner, [{"entries": [(rid, toks, list(range(len(toks)))) for rid, toks in reqs.items()], "end": list(reqs)}])
    for key, row in together.items():
        assert float((row - alone[key]).abs().max()) < 2e-4 * max(1.0, float(row.abs().max())), key


@pytest.mark.parametrize("name", ["mixed", "only_states", "awkward"])
def test_slots_and_pages_are_clean_for_their_next_holder(vekasun_folders, name):
    """Two slots and few pages: a request that takes a slot after another finds zero states (the matrices, the
    convolutions' last inputs) in every pass of a loop, and its own keys only."""
    folder, vocab = vekasun_folders[name, False], CONFIGS[name]["vocab"]
    reqs = {f"q{i}": random_tokens(n, vocab, 90 + i) for i, n in enumerate((40, 25, 31, 12, 37))}
    plain = plain_rows(folder, reqs)
    runner = runner_for(folder, "float32", tokens=96, slots=2)
    compare_rows(run_steps(runner, mixed_trace(reqs, 5, max_live=2)), plain, TOL["float32"])
    for rid, toks in reqs.items():
        compare_rows(run_steps(runner, tail_one_by_one(rid, toks, tail=3)), plain, TOL["float32"])


# ---------------------------------------------------------------------------------- marked tokens


def best_key_for_the_last_query(w, cfg, last_token: int, distance: int):
    """(token, others): of a one-layer latent attention, the token whose key ``distance`` back scores highest for the
    last query (over the heads' mean), and tokens whose scores lie in the lower half."""
    m, eps = cfg["layers"][0]["mixer"], cfg["norm"]["eps"]
    H, d, r, rank = m["heads"], m["dim"], m["rot_dim"], m["kv_rank"]
    h = pv.layer_norm(w["embed"], w["l0.norm1"], eps)
    q = (pv.rms(h[last_token] @ w["l0.mix.dq"].T, eps) * w["l0.mix.dq.norm"] @ w["l0.mix.uq"].T).view(H, d + r)
    down = h @ w["l0.mix.dkv"].T
    c = pv.rms(down[:, :rank], eps) * w["l0.mix.dkv.norm"]
    k = (c @ w["l0.mix.uk"].T).view(-1, H, d)
    f = torch.tensor([m["rot"]["base"] ** (-2.0 * i / r) for i in range(r // 2)], dtype=torch.float64) * distance
    u, v = q[:, d : d + r // 2], q[:, d + r // 2 :]
    turned = torch.cat([u * torch.cos(f) - v * torch.sin(f), v * torch.cos(f) + u * torch.sin(f)], -1)  # by the distance
    score = (torch.einsum("thd,hd->th", k, q[:, :d]) + down[:, rank:] @ turned.T).mean(-1) * m["scale"]
    order = torch.argsort(score, descending=True).tolist()
    return order[0], [t for t in order[len(order) // 2 :] if t != last_token]


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_a_key_that_stands_out_at_page_borders_and_far_back(tmp_path, dtype):
    """A sharp attention (a large scale) and one token whose key stands out for the last query, put at a page's borders,
    a page and two pages back, in front of a chunk of keys and hundreds of tokens back: the plain last row moves by
    it, and the engine's last rows are the plain model's, in a whole prompt, decoded at the end, in portions, and with
    the key itself decoded alone."""
    n = 300
    config = model(64, 32, [latent_layer(1, 16, 4, 32, 24, 24, 2.0, base=50.0)])
    # (the rotated parts of the keys are small beside the others, so that a token is dull wherever it stands)
    folder = make_folder(tmp_path / "sharp", config, seed=8, edits={
        ".sink": lambda t: t * 0, ".mix.o": lambda t: t * 3.0, ".dkv": lambda t: torch.cat([t[:24], t[24:] * 0.3])})
    cfg, w = load_plain(folder)
    runner = runner_for(folder, dtype, tokens=320)
    for back in (1, 11, 12, 13, 27, 28, 43, 44, 250, 299):  # position n - 1 - back: 288, 287, .., 272, 271, .. are page borders
        last = 5
        mark, dull = best_key_for_the_last_query(w, cfg, last, back)
        g = random.Random(back)
        tokens = [g.choice(dull) for _ in range(n - 1)] + [last]
        unmarked = pv.forward(tokens, w, cfg)[-1]
        tokens[n - 1 - back] = mark
        plain = pv.forward(tokens, w, cfg).float()
        assert float((plain[-1] - unmarked).norm() / unmarked.norm()) > 0.5, back
        cuts = [whole("e", tokens), tail_one_by_one("e", tokens, tail=3), portions("e", tokens, [2, 61])]
        if back < 50:
            cuts.append(tail_one_by_one("e", tokens, tail=back + 2))
        for steps in cuts:
            got = run_steps(runner, steps)
            compare_rows({k: v for k, v in got.items() if k[1] >= n - 3}, {"e": plain}, TOL[dtype])


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_sinks_of_every_size(tmp_path, dtype):
    """A sink far below every score, one that takes half and one that takes nearly all: over few keys and over so many
    that a decoded token's keys are cut among workgroups (each counts the sink once)."""
    n = 600
    config = model(64, 32, [latent_layer(3, 16, 4, 16, 24, 24, 0.3, base=50.0)])
    folder = make_folder(tmp_path / "sinks", config, seed=12, edits={".sink": lambda t: torch.tensor([-20.0, 5.0, 9.0])})
    cfg, w = load_plain(folder)
    tokens = random_tokens(n, 64, 3)
    plain = {"s": pv.forward(tokens, w, cfg).float()}
    w2 = {**w, "l0.mix.sink": w["l0.mix.sink"] + 0.6931471805599453}  # (counted twice, a sink would be this much larger)
    assert float((pv.forward(tokens, w2, cfg)[-1].float() - plain["s"][-1]).norm() / plain["s"][-1].norm()) > 3 * TOL["float32"]
    runner = runner_for(folder, dtype, tokens=640)
    for steps in (whole("s", tokens), tail_one_by_one("s", tokens, tail=20), portions("s", tokens, [2, 130, 1])):
        compare_rows(run_steps(runner, steps), plain, TOL[dtype])



@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_a_token_far_back_shows_through_the_recurrence(tmp_path, dtype):
    """Heads that hardly forget and a large step at the marked token only (dt reads one direction of the stream): its
    mark is still in the last row 300 tokens on, in a whole prompt, token by token and across portions."""
    config = model(64, 32, [mamba_layer(4, 8, 16, 2, 1, 2)])
    folder = make_folder(tmp_path / "slow", config, seed=3, edits={
        ".A_log": lambda t: t * 0 - 7.0, ".dt_bias": lambda t: t * 0 - 2.0, ".D": lambda t: t * 0 + 0.5})
    cfg, w = load_plain(folder)
    n = 300
    tokens = [t % 63 for t in random_tokens(n, 64, 9)]
    unmarked = pv.forward(tokens, w, cfg)[-1]
    tokens[0] = 63
    plain = pv.forward(tokens, w, cfg).float()
    moved = float((plain[-1] - unmarked).norm() / unmarked.norm())
    assert moved > 1e-3
    runner = runner_for(folder, dtype, tokens=448)
    for steps in (whole("e", tokens), tail_one_by_one("e", tokens, tail=250), portions("e", tokens, [2, 61, 1])):
        got = run_steps(runner, steps)
        compare_rows({k: v for k, v in got.items() if k[1] >= n - 3}, {"e": plain}, 3e-5 if dtype == "float32" else 2e-2)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_tokens_on_both_sides_of_a_chunk_s_border(tmp_path, dtype):
    """Prompts that end at, one before and one behind a border of the recurrence's 64-token chunks and 16-token tiles, and
    cuts that move the borders: every row is the plain one's, and the rows of two cuts agree."""
    config = model(64, 48, [mamba_layer(4, 16, 32, 2, 2, 4), mamba_layer(2, 24, 48, 1, 1, 3)])
    folder = make_folder(tmp_path / "chunks", config, seed=6, edits={".A_log": lambda t: t - 2.0})
    cfg, w = load_plain(folder)
    tokens = random_tokens(200, 64, 4)
    plain = {"c": pv.forward(tokens, w, cfg).float()}
    runner = runner_for(folder, dtype, tokens=256)
    for n in (15, 16, 17, 63, 64, 65, 80, 127, 128, 129, 193):
        compare_rows(run_steps(runner, whole("c", tokens[:n])), plain, TOL[dtype])
    for sizes in ([64], [63, 1], [65], [16], [17, 15], [1, 64, 128], [100, 2]):
        compare_rows(run_steps(runner, portions("c", tokens, sizes)), plain, TOL[dtype])


def test_the_convolution_reaches_across_the_cut(tmp_path):
    """A convolution of five taps: a row's logits depend on the four tokens before it, so an input that is lost at the
    start of a portion shows.  Portions of one to six tokens against the whole."""
    config = model(64, 32, [mamba_layer(1, 8, 8, 1, 1, 5)])
    folder = make_folder(tmp_path / "taps", config, seed=4, edits={".conv": lambda t: t * 2.0, ".A_log": lambda t: t * 0 + 3.0})
    cfg, w = load_plain(folder)
    tokens = random_tokens(40, 64, 5)
    plain = {"c": pv.forward(tokens, w, cfg).float()}
    other = list(tokens)
    other[30] = (other[30] + 1) % 64
    assert float((pv.forward(other, w, cfg)[34] - plain["c"][34]).abs().max()) > 1e-3
    runner = runner_for(folder, "float32", tokens=64)
    for sizes in ([1], [2], [3, 1, 2], [4, 5], [6]):
        compare_rows(run_steps(runner, portions("c", tokens, sizes)), plain, TOL["float32"])


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_first_tokens_of_a_sequence(vekasun_folders, dtype):
    """Requests of one, two and three tokens, whole and token by token: zeros in front of the convolution, a state
    that starts at zero, one key beside the sink, the first page half empty."""
    for name in sorted(CONFIGS):
        folder, vocab = vekasun_folders[name, STEADY[dtype]], CONFIGS[name]["vocab"]
        reqs = {f"s{n}": random_tokens(n, vocab, 30 + n) for n in (1, 2, 3, 6)}
        plain = plain_rows(folder, reqs)
        limits = rounding_limits(folder, reqs) if dtype == "bfloat16" else None
        runner = runner_for(folder, dtype, tokens=64)
        for rid, toks in reqs.items():
            compare_rows(run_steps(runner, whole(rid, toks)), plain, TOL[dtype], limits)
            compare_rows(run_steps(runner, portions(rid, toks, [1])), plain, TOL[dtype], limits)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_long_decoding(vekasun_folders, dtype):
    """A short prompt and 400 tokens decoded one by one through recorded steps."""
    folder, vocab = vekasun_folders["mixed", STEADY[dtype]], MIXED["vocab"]
    tokens = random_tokens(420, vocab, 77)
    plain = plain_rows(folder, {"d": tokens})
    runner = runner_for(folder, dtype, tokens=448)
    got = run_steps(runner, tail_one_by_one("d", tokens, tail=400))
    compare_rows(got, plain, TOL[dtype])
    assert all(step.captured for step in runner.recorded.values()) and runner.recorded


# ---------------------------------------------------------------------------------- the entry points


@pytest.mark.parametrize("name", ["mixed", "awkward", "only_states"])
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_greedy_generation_through_the_engine(vekasun_folders, dtype, name):
    """``Engine.generate``: the scheduler cuts prompts into portions beside decoding requests; the tokens are the
    plain model's greedy tokens (in bfloat16: each token is, for the plain logits of its own history, within
    rounding of the best)."""
    from tokasaurus_amd.config.engine_config import EngineConfig
    from tokasaurus_amd.engine.engine import Engine
    from tokasaurus_amd.sampling import SamplingParams

    folder, vocab = vekasun_folders[name, STEADY[dtype]], CONFIGS[name]["vocab"]
    prompts = [random_tokens(n, vocab, 10 + n) for n in (5, 40, 23, 1, 64)]
    engine = Engine(EngineConfig(model=str(folder), dtype=dtype, page_size=PAGE, kv_cache_num_tokens=512, max_seqs_per_forward=3,
                                 max_tokens_per_forward=24, allocator_sanity_checks=True))
    done = engine.generate(prompts, SamplingParams(temperature=0.0, max_tokens=12, ignore_eos=True))
    cfg, w = load_plain(folder)
    for prompt, c in zip(prompts, done):
        assert len(c.tokens) == 12 and c.finish_reason == "length"
        ids = list(prompt)
        for tok in c.tokens:
            logits = pv.forward(ids, w, cfg)[-1]
            if dtype == "float32":
                assert tok == int(logits.argmax()), f"token {tok}, plain {int(logits.argmax())}"
            else:
                assert float(logits.max() - logits[tok]) < 0.15 * float(logits.std()), f"{tok} lies below the best"
            ids.append(tok)
    assert engine.runner.manager.requests == {}


def test_command_line_and_trace_replay(vekasun_folders, tmp_path):
    """``bin/toka`` generates with the design and ``bin/trace_run`` replays a trace of it."""
    root = os.path.join(os.path.dirname(os.path.abspath(__file__)), "..")
    folder, vocab = vekasun_folders["mixed", False], MIXED["vocab"]
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
        mlp = rng.choice([None, moe(rng.choice([8, 20, 32, 33]), experts, rng.randint(1, experts)),
                          moe(rng.choice([16, 40]), 8, rng.choice([1, 2]))])
        if rng.random() < 0.5:
            groups = rng.choice([1, 2, 3])
            heads, vdim = groups * rng.choice([1, 2, 3]), rng.choice([4, 9, 16, 20, 48])
            parts = rng.choice([p for p in range(1, heads * vdim + 1) if heads * vdim % p == 0 and p <= 6])
            layers.append(mamba_layer(heads, vdim, rng.choice([4, 15, 16, 31, 64, 100]), groups, parts, rng.choice([1, 2, 3, 4, 6]), mlp=mlp))
        else:
            layers.append(latent_layer(rng.choice([1, 2, 3, 5, 8]), rng.choice([4, 8, 15, 16, 32]), rng.choice([2, 4, 8, 16, 32]),
                                       rng.choice([5, 8, 16, 32, 48]), rng.choice([7, 16, 24, 40]), rng.choice([12, 16, 32, 45, 64]),
                                       rng.choice([0.1, 0.3]), base=rng.choice([50.0, 10000.0]), mlp=mlp))
    n = len(layers)
    start = rng.randrange(n)
    loop = rng.choice([None, (start, rng.randint(start + 1, n), rng.choice([1, 2, 3]))])
    return model(rng.choice([40, 97, 130]), width, layers, eps=rng.choice([1e-6, 1e-5]), loop=loop, logit_scale=rng.choice([0.3, 1.0]))


@pytest.mark.parametrize("seed", range(12))
def test_random_configurations(tmp_path, seed):
    config = random_config(seed)
    reqs = {f"r{i}": random_tokens(n, config["vocab"], 20 * seed + i) for i, n in enumerate((90, 2, 37, 130))}
    for dtype in ("float32", "bfloat16"):
        folder = make_folder(tmp_path / f"drawn{dtype}", config, seed=seed, steady_choice=STEADY[dtype])
        plain = plain_rows(folder, reqs)
        limits = rounding_limits(folder, reqs) if dtype == "bfloat16" else None
        runner = runner_for(folder, dtype, tokens=320)
        for rid, toks in reqs.items():
            compare_rows(run_steps(runner, whole(rid, toks)), plain, TOL[dtype], limits)
        compare_rows(run_steps(runner, tail_one_by_one("r3", reqs["r3"], tail=70)), plain, TOL[dtype], limits)
        compare_rows(run_steps(runner, portions("r3", reqs["r3"], [2, 3, 16, 2, 1, 31, 5])), plain, TOL[dtype], limits)
        compare_rows(run_steps(runner, mixed_trace(reqs, seed, max_live=3)), plain, TOL[dtype], limits)
        assert runner.manager.requests == {}
