"""The plain Tefavik against properties that follow from its equations, the configuration reader, the
spec, and the pages that sections of keys take (no GPU)."""

from __future__ import annotations

import math

import pytest
import torch

import plain_tefavik as pt
from tefavik_models import (AWKWARD, CONFIGS, LARGE_HEADS, MIXED, ONLY_STATES, attention_branch, gla_layer, load_plain, make_folder,
                            memory_branch, model, moe, pair_layer)
from tokasaurus_amd.cache.manager import RELEASED, CacheGroup, CacheManager, plan_groups
from tokasaurus_amd.config.model_config import ConfigError
from tokasaurus_amd.config.tefavik_config import TefavikConfig
from tokasaurus_amd.models.registry import architecture_of, build_model, config_from_folder
from tokasaurus_amd.parts.base import INT_TABLE, CacheNeed, TensorSpec
from tokasaurus_amd.weights.loader import WeightError, read_tensors
from tokasaurus_amd.weights.random_init import draw_tensors


def weights_for(config, tmp_path, seed=0):
    return load_plain(make_folder(tmp_path / f"m{seed}", config, seed))[1]


def rnd(*shape):
    return torch.randn(*shape, dtype=torch.float64)


def test_decays_are_a_root_of_the_sigmoid():
    z = torch.tensor([-500.0, -3.0, 0.0, 2.0, 500.0], dtype=torch.float64)
    assert torch.allclose(pt.decays(z, 1.0), torch.sigmoid(z))
    assert torch.allclose(pt.decays(z[1:], 16.0) ** 16, torch.sigmoid(z[1:]))
    assert torch.allclose(pt.log_sigmoid(z), torch.nn.functional.logsigmoid(z))


def test_gated_linear_attention_as_a_sum_over_the_past():
    # o_t = sum_{s <= t} (sum_i q_t,i k_s,i prod_{s < r <= t} a_r,i) v_s
    torch.manual_seed(1)
    T, H, d, dv = 7, 2, 3, 5
    q, k, v, a = rnd(T, H, d), rnd(T, H, d), rnd(T, H, dv), torch.rand(T, H, d, dtype=torch.float64)
    o = pt.decayed_outer_products(q, k, v, a)
    for h in range(H):
        for t in range(T):
            want = sum((q[t, h] * k[s, h] * a[s + 1 : t + 1, h].prod(0)).sum() * v[s, h] for s in range(t + 1))
            assert torch.allclose(o[t, h], want)


def test_rotation_turns_neighbours_of_the_leading_part():
    torch.manual_seed(3)
    u, v = rnd(1, 8), rnd(1, 8)
    a, b = pt.rotate_neighbours(u.expand(20, 1, 8), 6, 50.0), pt.rotate_neighbours(v.expand(20, 1, 8), 6, 50.0)
    assert torch.allclose(a[0, 0], u[0]) and torch.allclose(a[9, 0, 6:], u[0, 6:])  # the rest of a head passes
    assert torch.allclose((a[7, 0] * b[3, 0]).sum(), (a[15, 0] * b[11, 0]).sum())  # only differences of positions count
    e = torch.zeros(2, 1, 8, dtype=torch.float64)
    e[1, 0, 0] = 1.0
    turned = pt.rotate_neighbours(e, 6, 50.0)[1, 0]
    assert abs(float(turned[0]) - math.cos(1.0)) < 1e-12 and abs(float(turned[1]) - math.sin(1.0)) < 1e-12


def test_chunks_are_counted_from_the_first_position():
    seen = pt.same_chunk(10, 4)
    for i in range(10):
        for j in range(10):
            assert bool(seen[i, j]) == (j <= i and i // 4 == j // 4)
    assert pt.same_chunk(5, 1).equal(torch.eye(5, dtype=torch.bool))


def test_one_in_the_denominator_is_a_sink_of_score_zero():
    s = rnd(4, 6) * 3
    seen = torch.ones(4, 6, dtype=torch.bool)
    p = pt.one_more_softmax(s, seen)
    with_sink = torch.softmax(torch.cat([s, torch.zeros(4, 1, dtype=torch.float64)], 1), 1)[:, :6]
    assert torch.allclose(p, with_sink)
    assert torch.allclose(pt.one_more_softmax(s * 0 - 800.0, seen), torch.zeros_like(s))
    assert torch.allclose(pt.one_more_softmax(s + 800.0, seen), torch.softmax(s, 1))
    seen[:, 3:] = False
    assert bool((pt.one_more_softmax(s, seen)[:, 3:] == 0).all())


def test_query_heads_share_key_heads_in_runs():
    torch.manual_seed(5)
    q, k, v = rnd(5, 6, 4), rnd(5, 2, 4), rnd(5, 2, 3)
    out = pt.chunk_attention(q, k, v, 0.5, 10.0, 64)
    for h in range(6):
        alone = pt.chunk_attention(q[:, h : h + 1], k[:, h // 3 : h // 3 + 1], v[:, h // 3 : h // 3 + 1], 0.5, 10.0, 64)
        assert torch.allclose(out[:, h : h + 1], alone)
    assert torch.allclose(pt.soft_cap(torch.tensor([1e-4, 1e6, -1e6], dtype=torch.float64), 7.0), torch.tensor([1e-4, 7.0, -7.0], dtype=torch.float64))


def test_matrix_memory_without_its_running_maximum():
    # the maximum only rescales: with S~ = e^m S and n~ = e^m n, o = S~^T q / (max(|n~ . q|, 1) + 1e-6 e^m)
    torch.manual_seed(6)
    T, H, d, dv = 9, 2, 4, 3
    q, k, v = rnd(T, H, d), rnd(T, H, d), rnd(T, H, dv)
    i, f = rnd(T, H) * 3, pt.log_sigmoid(rnd(T, H) + 1)
    o = pt.matrix_memory(q, k, v, i, f)
    for h in range(H):
        S, n, m = torch.zeros(d, dv, dtype=torch.float64), torch.zeros(d, dtype=torch.float64), 0.0
        for t in range(T):
            S = torch.exp(f[t, h]) * S + torch.exp(i[t, h]) * torch.outer(k[t, h], v[t, h])
            n = torch.exp(f[t, h]) * n + torch.exp(i[t, h]) * k[t, h]
            m = max(float(f[t, h]) + m, float(i[t, h]))
            want = (S.T @ q[t, h]) / (max(abs(float(n @ q[t, h])), 1.0) + 1e-6 * math.exp(m))
            assert torch.allclose(o[t, h], want)
    # the maximum starts at zero: a first token with a small input gate is read against e^0, not against itself
    small = pt.matrix_memory(q[:1], k[:1], v[:1], i[:1] * 0 - 8.0, f[:1])
    assert float(small.abs().max()) < 0.05 * float(pt.matrix_memory(q[:1], k[:1], v[:1], i[:1] * 0 + 8.0, f[:1]).abs().max())


def test_clamps():
    g, u = torch.tensor([5.0, -5.0, 0.5], dtype=torch.float64), torch.tensor([9.0, -9.0, 0.2], dtype=torch.float64)
    out = pt.clamped_gate(g, u, 1.0)
    want = [1.0 / (1 + math.exp(-1.702)) * 2.0, 0.0, 0.5 / (1 + math.exp(-0.851)) * 1.2]
    assert torch.allclose(out, torch.tensor(want, dtype=torch.float64), atol=1e-12)  # u = -limit gives u + 1 = 0; g has no lower clamp
    assert abs(float(pt.clamped_gate(torch.tensor(-5.0), torch.tensor(0.0), 1.0)) + 5.0 / (1 + math.exp(8.51))) < 1e-6


def test_a_token_s_experts_come_from_its_row_of_the_table(tmp_path):
    cfg = model(30, 16, [gla_layer(1, 4, 4, 2.0, 2, mlp=moe(8, 5, 2))])
    w = weights_for(cfg, tmp_path)
    h, tokens = rnd(3, 16), [4, 9, 4]
    mlp = cfg["layers"][0]["mlp"]
    out = pt.table_experts(h, tokens, w, "l0.mlp", mlp)
    table = w["l0.mlp.table"]
    assert table.dtype == torch.int32 and all(len(set(row.tolist())) == 2 for row in table) and int(table.max()) < 5
    for t in range(3):
        a, b = table[tokens[t]].tolist()
        want = 0.5 * (pt.expert(h[t], w, f"l0.mlp.e{a}", 1.5) + pt.expert(h[t], w, f"l0.mlp.e{b}", 1.5))
        assert torch.allclose(out[t], want)


def test_halves_of_two_normed_outputs(tmp_path):
    cfg = model(30, 16, [pair_layer(attention_branch(2, 1, 8, 4, 5), memory_branch(2, 4, 4))])
    w = weights_for(cfg, tmp_path)
    h, m = rnd(6, 16), cfg["layers"][0]["mixer"]
    out = pt.parallel_mixer(h, w, "l0.mix", m, 1e-5)
    big = {**w, "l0.mix.left.o": w["l0.mix.left.o"] * 50.0}
    assert torch.allclose(pt.parallel_mixer(h, big, "l0.mix", m, 0.0), pt.parallel_mixer(h, w, "l0.mix", m, 0.0))  # normed: no size
    none = {**w, "l0.mix.left.out": w["l0.mix.left.out"] * 0}
    right = pt.rms(pt.memory_branch(h, w, "l0.mix.right", m["right"], 1e-5), 1e-5) * w["l0.mix.right.out"]
    assert torch.allclose(pt.parallel_mixer(h, none, "l0.mix", m, 1e-5), 0.5 * right) and not torch.allclose(out, 0.5 * right)


def test_run_order_and_the_embedding_s_output_in_front_of_a_pass(tmp_path):
    assert pt.run_order(MIXED) == [(0, False), (1, False), (2, False), (1, True), (2, False), (3, False)]
    for name, cfg in CONFIGS.items():
        assert TefavikConfig.from_dict(cfg).run_order() == pt.run_order(cfg), name
    w = weights_for(AWKWARD, tmp_path)
    tokens = [1, 2, 3]
    streams: list = []
    pt.forward(tokens, w, AWKWARD, streams)
    x = x0 = w["embed"][tokens]
    for n, (i, add) in enumerate([(0, False), (1, False), (0, True), (1, False), (0, True), (1, False)]):
        x = pt.layer(x + x0 if add else x, tokens, w, i, AWKWARD)
        assert torch.equal(streams[n], x)


def test_the_model_is_causal(tmp_path):
    w = weights_for(MIXED, tmp_path)
    tokens = [5, 9, 11, 2, 7, 7, 3]
    a = pt.forward(tokens, w, MIXED)
    b = pt.forward(tokens[:4] + [8] + tokens[5:], w, MIXED)
    assert torch.allclose(a[:4], b[:4]) and not torch.allclose(a[4:], b[4:])


def test_configuration_reader():
    c = TefavikConfig.from_dict(MIXED)
    assert c.layers[0].mixer.tau == 8.0 and c.layers[0].ff.top == 2 and c.layers[2].ff is None
    left, right = c.layers[1].mixer.left, c.layers[3].mixer.right
    assert left.chunk == 24 and left.rot_dims == 16 and left.softcap == 20.0 and right.gate_cap == 5.0 and c.layers[1].ff.limit == 0.7
    assert c.loop.times == 2 and TefavikConfig.from_dict({**MIXED, "loop": None}).loop is None
    bare = attention_branch(2, 1, 8, 8, 4)
    del bare["softcap"], bare["mask"], bare["rot"]
    open_branch = TefavikConfig.from_dict(model(20, 16, [pair_layer(bare, memory_branch(1, 4, 4))])).layers[0].mixer.left
    assert open_branch.softcap is None and open_branch.chunk == 0 and open_branch.rot_base is None
    good_left, good_right, good = attention_branch(2, 1, 8, 8, 4), memory_branch(1, 4, 4), gla_layer(1, 4, 4, 2.0, 2)
    for broken in (
        model(20, 16, [{**good, "type": "lightning"}]),
        model(20, 16, [gla_layer(1, 4, 4, 0.0, 2)]),
        model(20, 16, [gla_layer(0, 4, 4, 2.0, 2)]),
        model(20, 16, [pair_layer(attention_branch(3, 2, 8, 8, 4), good_right)]),
        model(20, 16, [pair_layer(attention_branch(2, 1, 8, 8, 4, rot_dims=10), good_right)]),
        model(20, 16, [pair_layer(attention_branch(2, 1, 8, 8, 4, rot_dims=3), good_right)]),
        model(20, 16, [pair_layer(attention_branch(2, 1, 8, 8, 0), good_right)]),
        model(20, 16, [pair_layer(attention_branch(2, 1, 8, 8, 4, softcap=-1.0), good_right)]),
        model(20, 16, [pair_layer(good_left, memory_branch(1, 4, 4, cap=0.0))]),
        model(20, 16, [{**pair_layer(good_left, good_right), "mixer": {"left": good_left}}]),
        model(20, 16, [gla_layer(1, 4, 4, 2.0, 2, mlp=moe(8, 2, 3))]),
        model(20, 16, [gla_layer(1, 4, 4, 2.0, 2, mlp=moe(8, 2, 1, limit=0.0))]),
        model(20, 16, [gla_layer(1, 4, 4, 2.0, 2, mlp={"kind": "dense", "ff": 8})]),
        model(20, 16, [good], loop=(0, 2, 2)),
        model(20, 16, [good], loop=(0, 1, 0)),
        model(20, 16, []),
        {k: v for k, v in MIXED.items() if k != "norm"},
    ):
        with pytest.raises(ConfigError):
            TefavikConfig.from_dict(broken)


def test_spec_names_every_tensor_once_and_plans_caches_and_states():
    arch = architecture_of(MIXED)
    assert arch.name == "tefavik"
    m = build_model(arch, arch.config_from_dict(MIXED))
    shapes = {s.name: s.shape for s in m.tensor_specs()}
    assert len(shapes) == len(m.tensor_specs()) and "head" not in shapes
    assert shapes["l0.mix.a1"] == (12, 96) and shapes["l0.mix.a2"] == (96, 12) and shapes["l0.mix.a2.b"] == (96,)
    assert shapes["l0.mix.norm"] == (48,) and shapes["l1.mix.right.norm"] == (64,) and shapes["l1.mix.left.out"] == (96,)
    assert shapes["l1.mix.left.q.b"] == (128,) and shapes["l1.mix.left.k.norm"] == (32,) and shapes["l3.mix.right.i"] == (6, 96)
    assert shapes["l1.mlp.table"] == (150, 3) and shapes["l1.mlp.e4.down"] == (96, 24) and "l2.norm2" not in shapes
    caches, states = m.cache_needs(), m.state_needs()
    # every pass of the loop has a cache and a state of its own
    assert [c is None for c in caches] == [True, False, True, False, True, False] and all(s is not None for s in states)
    assert caches[1] == caches[3] and caches[1].section == 24 and caches[5].section == 40 and not caches[1].keeps_all
    # the matrices and the keys' sums, then two rows of running maxima; the matrices alone
    assert states[1].shape == (2 * 33 * 24 + 4,) and states[0].shape == (3 * 48 * 32,)
    groups, where = plan_groups(caches, [None] * 6)
    assert len(groups) == 2 and where[1] == (0, 0) and where[3] == (0, 1) and where[5] == (1, 0)


def test_the_rank_of_the_decays_is_the_checkpoint_s(tmp_path):
    folder = make_folder(tmp_path / "m", MIXED, 0)
    text = (folder / "config.json").read_text()
    import json

    cfg = json.loads(text)
    for layer in cfg["layers"]:
        layer["mixer"].pop("rank", None)
    (folder / "config.json").write_text(json.dumps(cfg))
    arch, c = config_from_folder(folder)
    assert c.layers[0].mixer.rank == 12 and c.layers[2].mixer.rank == 24
    m = build_model(arch, c)
    tensors = read_tensors(folder, m.tensor_specs(), m.spec.ignorable_tensors)
    assert tensors["l0.mlp.table"].dtype == torch.int32


def test_tables_name_experts_that_exist(tmp_path):
    spec = TensorSpec("t", (50, 3), INT_TABLE, below=4)
    drawn = draw_tensors([spec], 1)["t"]
    assert int(drawn.min()) >= 0 and int(drawn.max()) == 3 and all(len(set(r.tolist())) == 3 for r in drawn)
    folder = make_folder(tmp_path / "m", ONLY_STATES, 0)
    arch, c = config_from_folder(folder)
    specs = build_model(arch, c).tensor_specs()
    read_tensors(folder, specs)
    short = [TensorSpec(s.name, s.shape, s.kind, below=2 if s.kind == INT_TABLE else 0) for s in specs]
    with pytest.raises(WeightError, match="outside"):
        read_tensors(folder, short)


# ---------------------------------------------------------------------------------- pages of sections


def test_pages_go_back_when_their_section_is_over():
    need = CacheNeed(1, 8, section=24)
    m = CacheManager([CacheGroup(need, (0,))], 8, 16, 2, max_blocks_per_request=8)
    m.admit("a")
    for n in range(1, 100):
        m.reserve("a", n)
        m.advance("a", n)
        m.check()
        # the next query, at position n, reads from its section's first position on
        first = n // 24 * 24
        table = m.requests["a"].tables[0]
        assert all((p == RELEASED) == ((b + 1) * 16 <= first) for b, p in enumerate(table)), n
        assert need.first_read(n) == first
    m.release("a")
    assert m.num_free_pages() == [8]
    # a pool of fewer pages than the request's tokens serves it
    small = CacheManager([CacheGroup(need, (0,))], 3, 16, 1, max_blocks_per_request=64)
    small.admit("b")
    for n in range(1, 400):
        small.reserve("b", n)
        small.advance("b", n)
    small.check()


def test_sections_and_windows_do_not_mix():
    with pytest.raises(ValueError):
        CacheNeed(1, 8, window=4, section=4)
    whole, cut = CacheNeed(1, 8), CacheNeed(1, 8, section=16)
    plan_groups([whole, cut], [None, 0])  # a reader of less than the owner keeps
    with pytest.raises(ValueError):
        plan_groups([cut, whole], [None, 0])
    with pytest.raises(ValueError):
        plan_groups([cut, CacheNeed(1, 8, section=32)], [None, 0])
    assert LARGE_HEADS["layers"][0]["mixer"]["left"]["mask"]["size"] == 64
