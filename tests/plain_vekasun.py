"""A plain, slow Vekasun on whole sequences, one function per mechanism, written from the
equations alone.  It shares no code with the engine: tensors by their checkpoint names, the
configuration as the dict that config.json holds, everything in the dtype of the weights it is
given (float64 for an oracle).

Notation: T tokens, W the width, H heads, G groups of heads that share B and C, N the rows of a
head's state, dv the size of a head's value.
"""

from __future__ import annotations

from contextlib import contextmanager

import torch

_round = False


@contextmanager
def rounding():
    """Inside, what an engine with bfloat16 storage keeps in bfloat16 (rows behind norms, activations, queries, keys and
    values) is rounded to it: a measure of what rounding alone does to a row, in the place of a tolerance."""
    global _round
    _round = True
    try:
        yield
    finally:
        _round = False


def kept(x: torch.Tensor) -> torch.Tensor:
    return x.float().bfloat16().to(x.dtype) if _round else x



def rms(x: torch.Tensor, eps: float) -> torch.Tensor:
    """x / sqrt(mean(x^2) + eps) over the last axis."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def layer_norm(x: torch.Tensor, weight: torch.Tensor, eps: float) -> torch.Tensor:
    """(x - mean) / sqrt(mean((x - mean)^2) + eps) * weight over the last axis; no bias."""
    d = x - x.mean(-1, keepdim=True)
    return kept(d / torch.sqrt((d * d).mean(-1, keepdim=True) + eps) * weight)


def silu(z: torch.Tensor) -> torch.Tensor:
    return z * torch.sigmoid(z)


def softplus(z: torch.Tensor) -> torch.Tensor:
    """log(1 + e^z), without overflow."""
    return torch.clamp(z, min=0) + torch.log1p(torch.exp(-z.abs()))


# --------------------------------------------------------------------------- the state-space mixer


def causal_convolution(u: torch.Tensor, taps: torch.Tensor, bias: torch.Tensor) -> torch.Tensor:
    """bias + sum_j taps[:, j] * u_(t - n + 1 + j), zeros before the start; u [T, C], taps [C, n]."""
    T, n = u.shape[0], taps.shape[1]
    out = torch.zeros_like(u)
    for t in range(T):
        out[t] = bias
        for j in range(n):
            s = t - n + 1 + j
            if s >= 0:
                out[t] += taps[:, j] * u[s]
    return out


def state_space(x: torch.Tensor, B: torch.Tensor, C: torch.Tensor, dt: torch.Tensor, A_log: torch.Tensor, D: torch.Tensor) -> torch.Tensor:
    """x [T, H, dv], B and C [T, G, N], dt [T, H] -> y [T, H, dv]: per head, with g = h // (H / G),
    S <- exp(-exp(A_log_h) dt) S + dt B_g x^T (from zero), y = S^T C_g + D_h x."""
    T, H, dv = x.shape
    G, N = B.shape[1:]
    y = torch.zeros_like(x)
    for h in range(H):
        g = h // (H // G)
        S = torch.zeros((N, dv), dtype=x.dtype)
        for t in range(T):
            S = torch.exp(-torch.exp(A_log[h]) * dt[t, h]) * S + dt[t, h] * torch.outer(B[t, g], x[t, h])
            y[t, h] = S.T @ C[t, g] + D[h] * x[t, h]
    return y


def gate_then_norm(y: torch.Tensor, z: torch.Tensor, weight: torch.Tensor, groups: int, eps: float) -> torch.Tensor:
    """y * silu(z), then every one of ``groups`` equal parts of a row over its own root mean square, times weight."""
    v = y * silu(z)
    return kept(rms(v.reshape(v.shape[0], groups, -1), eps).reshape(v.shape) * weight)


def mamba2_mixer(h: torch.Tensor, w: dict, p: str, m: dict, eps: float) -> torch.Tensor:
    T = h.shape[0]
    H, dv, N, G = int(m["heads"]), int(m["vdim"]), int(m["state"]), int(m["groups"])
    inner = H * dv
    z, u, dt = torch.split(h @ w[f"{p}.in"].T, [inner, inner + 2 * G * N, H], dim=-1)
    u = kept(silu(causal_convolution(u, w[f"{p}.conv"], w[f"{p}.conv.b"])))
    x, B, C = torch.split(u, [inner, G * N, G * N], dim=-1)
    dt = softplus(dt + w[f"{p}.dt_bias"])
    y = state_space(x.reshape(T, H, dv), B.reshape(T, G, N), C.reshape(T, G, N), dt, w[f"{p}.A_log"], w[f"{p}.D"]).reshape(T, inner)
    return gate_then_norm(y, z, w[f"{p}.norm"], int(m["norm_groups"]), eps) @ w[f"{p}.o"].T


# --------------------------------------------------------------------------- latent attention


def rotate_halves(x: torch.Tensor, base: float) -> torch.Tensor:
    """x [T, ..., n]: element i and element i + n/2 turned by t * base^(-2i/n), t the row's place."""
    T, n = x.shape[0], x.shape[-1]
    f = torch.tensor([float(base) ** (-2.0 * i / n) for i in range(n // 2)], dtype=torch.float64)
    a = (torch.arange(T, dtype=torch.float64)[:, None] * f[None, :]).view(T, *([1] * (x.dim() - 2)), n // 2)
    c, s = torch.cos(a).to(x.dtype), torch.sin(a).to(x.dtype)
    u, v = x[..., : n // 2], x[..., n // 2 :]
    return torch.cat([u * c - v * s, v * c + u * s], dim=-1)


def sink_attention(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, scale: float, sink: torch.Tensor) -> torch.Tensor:
    """q, k [T, H, d], v [T, H, dv] -> [T, H, dv]: causal; exp(sink_h) joins the softmax's denominator once."""
    T, H, _ = q.shape
    out = torch.zeros((T, H, v.shape[2]), dtype=q.dtype)
    mask = torch.ones((T, T), dtype=torch.bool).tril()
    for h in range(H):
        s = ((q[:, h] @ k[:, h].T) * scale).masked_fill(~mask, float("-inf"))
        top = torch.maximum(s.max(-1, keepdim=True).values, sink[h])
        e = torch.exp(s - top)
        out[:, h] = (e / (e.sum(-1, keepdim=True) + torch.exp(sink[h] - top))) @ v[:, h]
    return out


def latent_attention_mixer(h: torch.Tensor, w: dict, p: str, m: dict, eps: float) -> torch.Tensor:
    T = h.shape[0]
    H, d, r, dv, rank = int(m["heads"]), int(m["dim"]), int(m["rot_dim"]), int(m["vdim"]), int(m["kv_rank"])
    base = float(m["rot"]["base"])
    cq = kept(rms(h @ w[f"{p}.dq"].T, eps) * w[f"{p}.dq.norm"])
    q = (cq @ w[f"{p}.uq"].T).view(T, H, d + r)
    down = h @ w[f"{p}.dkv"].T
    c = kept(rms(down[:, :rank], eps) * w[f"{p}.dkv.norm"])
    k_rot = rotate_halves(down[:, rank:], base)
    k = torch.cat([(c @ w[f"{p}.uk"].T).view(T, H, d), k_rot[:, None, :].expand(T, H, r)], dim=-1)
    q = torch.cat([q[..., :d], rotate_halves(q[..., d:], base)], dim=-1)
    o = sink_attention(kept(q), kept(k), (c @ w[f"{p}.uv"].T).view(T, H, dv), float(m["scale"]), w[f"{p}.sink"]).reshape(T, H * dv)
    return kept(kept(o) * torch.sigmoid(h @ w[f"{p}.g"].T)) @ w[f"{p}.o"].T


# --------------------------------------------------------------------------- feed-forward


def expert(h: torch.Tensor, w: dict, p: str) -> torch.Tensor:
    return kept(silu(h @ w[f"{p}.gate"].T) * (h @ w[f"{p}.up"].T)) @ w[f"{p}.down"].T


def route(h: torch.Tensor, w: dict, p: str, r: dict) -> tuple[torch.Tensor, torch.Tensor]:
    """The chosen experts [T, top] and their weights: sigmoid scores, the largest chosen, the scores as they are."""
    s = torch.sigmoid(h @ w[f"{p}.router"].T)
    top = torch.topk(s, int(r["top"]), dim=-1)
    return top.indices, top.values


def experts_ff(h: torch.Tensor, w: dict, p: str, mlp: dict) -> torch.Tensor:
    """A token's weight for an expert multiplies what the expert reads."""
    ids, weights = route(h, w, p, mlp["router"])
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e, g in zip(ids[t].tolist(), weights[t]):
            out[t] += expert(g * h[t : t + 1], w, f"{p}.e{e}")[0]
    return out


# --------------------------------------------------------------------------- the model


MIXERS = {"mamba2": mamba2_mixer, "latent_attention": latent_attention_mixer}


def run_order(cfg: dict) -> list[tuple[int, int | None]]:
    """(layer, number of the loop's pass that begins with it or None) in the order the layers run."""
    n, loop = len(cfg["layers"]), cfg.get("loop")
    if not loop:
        return [(i, None) for i in range(n)]
    a, b = int(loop["start"]), int(loop["stop"])
    order: list[tuple[int, int | None]] = [(i, None) for i in range(a)]
    for t in range(int(loop["times"])):
        order += [(i, t if i == a else None) for i in range(a, b)]
    return order + [(i, None) for i in range(b, n)]


def layer(x: torch.Tensor, w: dict, i: int, cfg: dict) -> torch.Tensor:
    eps, entry = float(cfg["norm"]["eps"]), cfg["layers"][i]
    x = x + MIXERS[entry["type"]](layer_norm(x, w[f"l{i}.norm1"], eps), w, f"l{i}.mix", entry["mixer"], eps)
    if entry.get("mlp") is not None:
        x = x + experts_ff(layer_norm(x, w[f"l{i}.norm2"], eps), w, f"l{i}.mlp", entry["mlp"])
    return x


def forward(tokens: list[int], w: dict, cfg: dict, streams: list | None = None) -> torch.Tensor:
    """Logits [T, vocab] of one whole sequence; ``streams`` collects the stream after every layer run."""
    x = w["embed"][tokens]
    for i, loop_pass in run_order(cfg):
        if loop_pass is not None:
            x = x + w["loop.step"][loop_pass]
        x = layer(x, w, i, cfg)
        if streams is not None:
            streams.append(x)
    return layer_norm(x, w["final.norm"], float(cfg["norm"]["eps"])) @ w["head"].T * float(cfg.get("logit_scale", 1.0))
