"""The plain Vekasun against properties that follow from its equations, the configuration reader and
the spec (no GPU)."""

from __future__ import annotations

import math

import pytest
import torch

import plain_vekasun as pv
from tokasaurus_amd.config.model_config import ConfigError
from tokasaurus_amd.config.vekasun_config import VekasunConfig
from tokasaurus_amd.models.registry import architecture_of, build_model
from tokasaurus_amd.weights.random_init import draw_tensors
from vekasun_models import AWKWARD, CONFIGS, MIXED, ONLY_ATTENTION, ONLY_STATES, latent_layer, mamba_layer, model, moe


def weights_for(config, seed=0):
    arch = architecture_of(config)
    m = build_model(arch, arch.config_from_dict(config))
    w = {k: v.double() for k, v in draw_tensors(m.tensor_specs(), seed).items()}
    return {k: (v * (1.0 / (0.02 * v.shape[1] ** 0.5)) if (v.dim() == 2 and not k.endswith(".conv")) else v) for k, v in w.items()}


def test_layer_norm_knows_neither_a_shift_nor_a_factor():
    torch.manual_seed(0)
    x, w = torch.randn(3, 40, dtype=torch.float64), torch.rand(40, dtype=torch.float64)
    y = pv.layer_norm(x, w, 0.0)
    assert torch.allclose(y, pv.layer_norm(5.0 * x + 3.0, w, 0.0))
    assert torch.allclose((y / w).mean(-1), torch.zeros(3, dtype=torch.float64), atol=1e-12)
    assert torch.allclose((y / w).pow(2).mean(-1), torch.ones(3, dtype=torch.float64))
    assert torch.allclose(y, torch.nn.functional.layer_norm(x, (40,), w, None, 0.0))


def test_convolution_is_causal_starts_from_zeros_and_has_its_bias():
    torch.manual_seed(0)
    u, taps, b = torch.randn(6, 3, dtype=torch.float64), torch.randn(3, 4, dtype=torch.float64), torch.randn(3, dtype=torch.float64)
    out = pv.causal_convolution(u, taps, b)
    assert torch.allclose(out[0], b + taps[:, 3] * u[0])
    assert torch.allclose(out[5], b + sum(taps[:, j] * u[2 + j] for j in range(4)))
    u2 = u.clone()
    u2[4] += 1.0
    assert torch.equal(pv.causal_convolution(u2, taps, b)[:4], out[:4])


def test_state_space_as_a_sum_over_the_past():
    # y_t = sum_{s <= t} (C_t . B_s) exp(-e^A sum_{s < r <= t} dt_r) dt_s x_s + D x_t, head h with the B and C of group h // (H / G)
    torch.manual_seed(1)
    T, H, G, N, dv = 7, 4, 2, 3, 5
    x, B, C = torch.randn(T, H, dv), torch.randn(T, G, N), torch.randn(T, G, N)
    x, B, C = x.double(), B.double(), C.double()
    dt, A, D = torch.rand(T, H).double(), torch.randn(H).double(), torch.randn(H).double()
    y = pv.state_space(x, B, C, dt, A, D)
    for h in range(H):
        g = h // 2
        for t in range(T):
            want = D[h] * x[t, h]
            for s in range(t + 1):
                decay = torch.exp(-torch.exp(A[h]) * dt[s + 1 : t + 1, h].sum())
                want = want + (C[t, g] @ B[s, g]) * decay * dt[s, h] * x[s, h]
            assert torch.allclose(y[t, h], want)


def test_softplus():
    z = torch.tensor([-800.0, -3.0, 0.0, 2.0, 800.0], dtype=torch.float64)
    assert torch.allclose(pv.softplus(z), torch.tensor([0.0, math.log1p(math.exp(-3)), math.log(2), math.log(1 + math.exp(2)), 800.0], dtype=torch.float64))


def test_the_gate_comes_before_the_norm_and_the_norm_is_taken_part_by_part():
    torch.manual_seed(2)
    y, z = torch.randn(3, 12, dtype=torch.float64), torch.randn(3, 12, dtype=torch.float64)
    one = torch.ones(12, dtype=torch.float64)
    out = pv.gate_then_norm(y, z, one, 3, 0.0)
    assert torch.allclose(out.view(3, 3, 4).pow(2).mean(-1), torch.ones(3, 3, dtype=torch.float64))  # normed behind the gate
    big = y.clone()
    big[:, 4:8] *= 100.0
    assert torch.allclose(pv.gate_then_norm(big, z, one, 3, 0.0), out)  # every part by its own size
    assert not torch.allclose(pv.gate_then_norm(big, z, one, 1, 0.0), pv.gate_then_norm(y, z, one, 1, 0.0))


def test_rotation_keeps_lengths_and_knows_differences_of_positions_only():
    torch.manual_seed(3)
    u, v = torch.randn(8, dtype=torch.float64), torch.randn(8, dtype=torch.float64)
    a, b = pv.rotate_halves(u.expand(20, 8), 50.0), pv.rotate_halves(v.expand(20, 8), 50.0)
    assert torch.allclose(a[0], u) and torch.allclose(a.norm(dim=-1), u.norm().expand(20))
    assert torch.allclose(a[7] @ b[3], a[15] @ b[11]) and not torch.allclose(a[7] @ b[3], a[7] @ b[4])
    # element 0 meets element 4 (halves), at the full speed of one radian a position
    e = torch.zeros(2, 8, dtype=torch.float64)
    e[1, 0] = 1.0
    turned = pv.rotate_halves(e, 50.0)[1]
    assert abs(float(turned[0]) - math.cos(1.0)) < 1e-12 and abs(float(turned[4]) - math.sin(1.0)) < 1e-12


def test_a_sink_takes_weight_and_gives_no_value():
    torch.manual_seed(4)
    T, H = 5, 2
    q, k = torch.randn(T, H, 3, dtype=torch.float64), torch.randn(T, H, 3, dtype=torch.float64)
    v = torch.ones(T, H, 4, dtype=torch.float64)
    none = pv.sink_attention(q, k, v, 0.5, torch.full((H,), -1e9, dtype=torch.float64))
    assert torch.allclose(none, v)
    out = pv.sink_attention(q * 0, k, v, 0.5, torch.zeros(H, dtype=torch.float64))
    want = torch.tensor([(t + 1) / (t + 2) for t in range(T)], dtype=torch.float64)
    assert torch.allclose(out[:, 0, 0], want)  # it counts once, whatever the number of keys, and is not scaled
    assert float(pv.sink_attention(q, k, v, 0.5, torch.full((H,), 50.0, dtype=torch.float64)).abs().max()) < 1e-12


def test_router_and_the_weight_on_the_input():
    cfg = model(40, 16, [mamba_layer(1, 4, 4, 1, 1, 2, mlp=moe(8, 5, 2))])
    w = weights_for(cfg)
    h = torch.randn(6, 16, dtype=torch.float64)
    mlp = cfg["layers"][0]["mlp"]
    ids, wts = pv.route(h, w, "l0.mlp", mlp["router"])
    s = torch.sigmoid(h @ w["l0.mlp.router"].T)
    assert torch.allclose(wts, torch.gather(s, 1, ids)) and bool((wts[:, 0] >= wts[:, 1]).all())
    out = pv.experts_ff(h, w, "l0.mlp", mlp)
    other = torch.zeros_like(out)
    for t in range(6):
        for e, g in zip(ids[t].tolist(), wts[t]):
            gate, up, down = (w[f"l0.mlp.e{e}.{n}"] for n in ("gate", "up", "down"))
            other[t] += (pv.silu(g * (h[t] @ gate.T)) * (g * (h[t] @ up.T))) @ down.T
    assert torch.allclose(out, other)


def test_run_order_and_the_row_of_a_pass():
    assert pv.run_order(MIXED) == [(0, None), (1, 0), (2, None), (1, 1), (2, None), (3, None)]
    for name, cfg in CONFIGS.items():
        assert VekasunConfig.from_dict(cfg).run_order() == pv.run_order(cfg), name
    # a row is added in front of a pass's first layer: with equal rows of zeros nothing is added
    w = weights_for(AWKWARD)
    tokens = [1, 2, 3]
    a = pv.forward(tokens, w, AWKWARD)
    for t in range(3):
        w2 = dict(w)
        w2["loop.step"] = w["loop.step"].clone()
        w2["loop.step"][t] += torch.randn(90, dtype=torch.float64)
        assert not torch.allclose(pv.forward(tokens, w2, AWKWARD), a)
    streams: list = []
    pv.forward(tokens, w, AWKWARD, streams)
    x = w["embed"][tokens]
    for n, (i, t) in enumerate(pv.run_order(AWKWARD)):
        x = pv.layer(x + w["loop.step"][t] if t is not None else x, w, i, AWKWARD)
        assert torch.equal(streams[n], x)


def test_the_model_is_causal():
    w = weights_for(MIXED)
    tokens = [5, 9, 11, 2, 7, 7, 3]
    a = pv.forward(tokens, w, MIXED)
    b = pv.forward(tokens[:4] + [8] + tokens[5:], w, MIXED)
    assert torch.allclose(a[:4], b[:4]) and not torch.allclose(a[4:], b[4:])


def test_configuration_reader():
    c = VekasunConfig.from_dict(MIXED)
    assert c.layers[0].mixer.taps == 4 and c.layers[0].mixer.norm_groups == 2 and c.layers[2].ff is None
    assert c.layers[1].mixer.q_rank == 64 and c.layers[3].mixer.rot_base == 500.0 and c.layers[1].ff.top == 3
    assert c.logit_scale == 0.7 and c.loop.times == 2
    bare = {k: v for k, v in ONLY_ATTENTION.items() if k != "logit_scale"}
    assert VekasunConfig.from_dict({**bare, "loop": None}).logit_scale == 1.0
    good = mamba_layer(2, 4, 4, 1, 1, 2)
    odd = latent_layer(2, 8, 6, 8, 8, 8, 0.3)
    odd["mixer"]["rot"]["dims"] = 4
    for broken in (
        model(20, 16, [{**good, "type": "mamba"}]),
        model(20, 16, [mamba_layer(3, 4, 4, 2, 1, 2)]),
        model(20, 16, [mamba_layer(3, 4, 4, 1, 5, 2)]),
        model(20, 16, [mamba_layer(3, 4, 0, 1, 1, 2)]),
        model(20, 16, [odd]),
        model(20, 16, [latent_layer(2, 8, 5, 8, 8, 8, 0.3)]),
        model(20, 16, [mamba_layer(2, 4, 4, 1, 1, 2, mlp=moe(8, 2, 3))]),
        model(20, 16, [mamba_layer(2, 4, 4, 1, 1, 2, mlp={"kind": "dense", "ff": 8})]),
        model(20, 16, [good], loop=(0, 2, 2)),
        model(20, 16, [good], loop=(0, 1, 0)),
        model(20, 16, []),
        {k: v for k, v in MIXED.items() if k != "norm"},
    ):
        with pytest.raises(ConfigError):
            VekasunConfig.from_dict(broken)


def test_spec_names_every_tensor_once_and_plans_caches_and_states():
    arch = architecture_of(MIXED)
    assert arch.name == "vekasun"
    m = build_model(arch, arch.config_from_dict(MIXED))
    shapes = {s.name: s.shape for s in m.tensor_specs()}
    assert len(shapes) == len(m.tensor_specs())
    assert shapes["l0.mix.in"] == (2 * 96 + 2 * 3 * 32 + 6, 96) and shapes["l0.mix.conv"] == (96 + 192, 4) and shapes["l0.mix.conv.b"] == (288,)
    assert shapes["l1.mix.uq"] == (4 * 48, 64) and shapes["l1.mix.dkv"] == (64, 96) and shapes["l1.mix.g"] == (4 * 48, 96)
    assert shapes["l1.mix.sink"] == (4,) and shapes["loop.step"] == (2, 96) and shapes["l3.mlp.e2.down"] == (96, 56)
    assert "l2.norm2" not in shapes and "l0.mlp.correction" not in shapes
    caches, states = m.cache_needs(), m.state_needs()
    # every pass of the loop has a cache and a state of its own
    assert [c is None for c in caches] == [True, False, True, False, True, False] and [s is None for s in states] == [False, True] * 3
    assert caches[1].head_dim == 64 and caches[1].value_size == 48 and caches[5].head_dim == 40
    # the matrices, then the convolution's last inputs
    assert states[0].shape == (6 * 16 * 32 + 4 * 288,)
    arch1 = architecture_of(ONLY_STATES)
    assert build_model(arch1, arch1.config_from_dict(ONLY_STATES)).state_needs()[0].shape == (2 * 8 * 24,)  # one tap: no inputs kept
