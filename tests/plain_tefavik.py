"""A plain, slow Tefavik on whole sequences, one function per mechanism, written from the
equations alone.  It shares no code with the engine: tensors by their checkpoint names, the
configuration as the dict that config.json holds, everything in the dtype of the weights it is
given (float64 for an oracle; tables of integers stay integers).

Notation: T tokens, W the width, H heads, G key/value heads, d the size of a head's queries and keys, dv of its values.
"""

from __future__ import annotations

from contextlib import contextmanager

import torch

_round = False


@contextmanager
def rounding():
    """Inside, what an engine with bfloat16 storage keeps in bfloat16 (rows behind norms, queries, keys, values, gated
    activations) is rounded to it: a measure of what rounding alone does to a row, in the place of a tolerance."""
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


def log_sigmoid(z: torch.Tensor) -> torch.Tensor:
    """log(1 / (1 + e^-z)), without overflow."""
    return torch.clamp(z, max=0) - torch.log1p(torch.exp(-z.abs()))


# --------------------------------------------------------------------------- gated linear attention


def decays(z: torch.Tensor, tau: float) -> torch.Tensor:
    """sigmoid(z)^(1 / tau)."""
    return torch.exp(log_sigmoid(z) / tau)


def decayed_outer_products(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, a: torch.Tensor) -> torch.Tensor:
    """q, k, a [T, H, d], v [T, H, dv] -> o [T, H, dv]: per head S <- diag(a_t) S + k_t v_t^T from zero, o_t = S^T q_t."""
    T, H, d = q.shape
    o = torch.zeros_like(v)
    for h in range(H):
        S = torch.zeros((d, v.shape[2]), dtype=v.dtype)
        for t in range(T):
            S = a[t, h][:, None] * S + torch.outer(k[t, h], v[t, h])
            o[t, h] = S.T @ q[t, h]
    return o


def gla_mixer(h: torch.Tensor, w: dict, p: str, m: dict, eps: float) -> torch.Tensor:
    T = h.shape[0]
    H, d, dv = int(m["heads"]), int(m["dim"]), int(m["vdim"])
    q = (h @ w[f"{p}.q"].T).view(T, H, d) * d ** -0.5
    k = (h @ w[f"{p}.k"].T).view(T, H, d)
    v = (h @ w[f"{p}.v"].T).view(T, H, dv)
    z = (h @ w[f"{p}.a1"].T) @ w[f"{p}.a2"].T + w[f"{p}.a2.b"]
    o = decayed_outer_products(q, k, v, decays(z, float(m["tau"])).view(T, H, d))
    o = (rms(o, eps) * w[f"{p}.norm"]).reshape(T, H * dv)
    g = h @ w[f"{p}.g"].T
    return kept(o * (g * torch.sigmoid(g))) @ w[f"{p}.o"].T


# --------------------------------------------------------------------------- attention inside chunks


def rotate_neighbours(x: torch.Tensor, dims: int, base: float) -> torch.Tensor:
    """x [T, H, d]: elements 2i and 2i + 1 of the leading ``dims`` turned by t * base^(-2i/dims), t the row's place."""
    T = x.shape[0]
    f = torch.tensor([float(base) ** (-2.0 * i / dims) for i in range(dims // 2)], dtype=torch.float64)
    a = (torch.arange(T, dtype=torch.float64)[:, None] * f[None, :]).view(T, 1, dims // 2)
    c, s = torch.cos(a).to(x.dtype), torch.sin(a).to(x.dtype)
    out = x.clone()
    u, v = x[..., 0:dims:2], x[..., 1:dims:2]
    out[..., 0:dims:2] = u * c - v * s
    out[..., 1:dims:2] = v * c + u * s
    return out


def soft_cap(s: torch.Tensor, cap: float) -> torch.Tensor:
    return cap * torch.tanh(s / cap)


def same_chunk(T: int, size: int) -> torch.Tensor:
    """[T, T]: query i sees key j <= i of its own chunk of ``size`` positions, counted from position 0."""
    i = torch.arange(T)
    return (i[:, None] >= i[None, :]) & ((i[:, None] // size) == (i[None, :] // size))


def one_more_softmax(s: torch.Tensor, seen: torch.Tensor) -> torch.Tensor:
    """exp(s_j) / (1 + sum over the seen of exp(s_j)); zero where not seen."""
    s = s.masked_fill(~seen, float("-inf"))
    top = torch.clamp(s.max(-1, keepdim=True).values, min=0)
    e = torch.exp(s - top)
    return e / (torch.exp(-top) + e.sum(-1, keepdim=True))


def chunk_attention(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, scale: float, cap: float, size: int) -> torch.Tensor:
    """q [T, H, d], k [T, G, d], v [T, G, dv] -> [T, H, dv]; query head h reads key/value head h // (H / G)."""
    T, H, _ = q.shape
    per = H // k.shape[1]
    seen = same_chunk(T, size)
    out = torch.zeros((T, H, v.shape[2]), dtype=q.dtype)
    for h in range(H):
        out[:, h] = one_more_softmax(soft_cap(q[:, h] @ k[:, h // per].T * scale, cap), seen) @ v[:, h // per]
    return out


def attention_branch(h: torch.Tensor, w: dict, p: str, m: dict, eps: float) -> torch.Tensor:
    T = h.shape[0]
    H, G, d, dv = int(m["heads"]), int(m["kv_heads"]), int(m["dim"]), int(m["vdim"])
    q = (h @ w[f"{p}.q"].T + w[f"{p}.q.b"]).view(T, H, d)
    k = (h @ w[f"{p}.k"].T + w[f"{p}.k.b"]).view(T, G, d)
    v = kept(h @ w[f"{p}.v"].T + w[f"{p}.v.b"]).view(T, G, dv)
    dims, base = int(m["rot"]["dims"]), float(m["rot"]["base"])
    q = kept(rotate_neighbours(rms(kept(q), eps) * w[f"{p}.q.norm"], dims, base))
    k = kept(rotate_neighbours(rms(kept(k), eps) * w[f"{p}.k.norm"], dims, base))
    o = chunk_attention(q, k, v, float(m["scale"]), float(m["softcap"]), int(m["mask"]["size"]))
    return kept(o.reshape(T, H * dv)) @ w[f"{p}.o"].T


# --------------------------------------------------------------------------- matrix memory (mLSTM)


def matrix_memory(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, i: torch.Tensor, f: torch.Tensor) -> torch.Tensor:
    """q, k [T, H, d], v [T, H, dv], log gates i, f [T, H] -> o [T, H, dv].  Per head, with m, S and n from zero:
    m' = max(f + m, i);  S <- e^(f + m - m') S + e^(i - m') k v^T;  n likewise with k alone;
    o = S^T q / (max(|n . q|, e^-m') + 1e-6)."""
    T, H, d = q.shape
    o = torch.zeros_like(v)
    for h in range(H):
        S = torch.zeros((d, v.shape[2]), dtype=v.dtype)
        n = torch.zeros((d,), dtype=v.dtype)
        m = torch.zeros((), dtype=v.dtype)
        for t in range(T):
            top = torch.maximum(f[t, h] + m, i[t, h])
            keep, write = torch.exp(f[t, h] + m - top), torch.exp(i[t, h] - top)
            S = keep * S + write * torch.outer(k[t, h], v[t, h])
            n = keep * n + write * k[t, h]
            m = top
            o[t, h] = (S.T @ q[t, h]) / (torch.maximum((n @ q[t, h]).abs(), torch.exp(-m)) + 1e-6)
    return o


def memory_branch(h: torch.Tensor, w: dict, p: str, m: dict, eps: float) -> torch.Tensor:
    T = h.shape[0]
    H, d, dv, cap = int(m["heads"]), int(m["dim"]), int(m["vdim"]), float(m["gate_cap"])
    q = (h @ w[f"{p}.q"].T).view(T, H, d) * d ** -0.5
    k = (h @ w[f"{p}.k"].T).view(T, H, d)
    v = (h @ w[f"{p}.v"].T).view(T, H, dv)
    i = soft_cap(h @ w[f"{p}.i"].T + w[f"{p}.i.b"], cap)
    f = log_sigmoid(soft_cap(h @ w[f"{p}.f"].T + w[f"{p}.f.b"], cap))
    o = rms(matrix_memory(q, k, v, i, f), eps).reshape(T, H * dv)
    return kept(o * w[f"{p}.norm"] * torch.sigmoid(h @ w[f"{p}.g"].T)) @ w[f"{p}.o"].T


def parallel_mixer(h: torch.Tensor, w: dict, p: str, m: dict, eps: float) -> torch.Tensor:
    left = rms(attention_branch(h, w, f"{p}.left", m["left"], eps), eps) * w[f"{p}.left.out"]
    right = rms(memory_branch(h, w, f"{p}.right", m["right"], eps), eps) * w[f"{p}.right.out"]
    return 0.5 * (left + right)


# --------------------------------------------------------------------------- feed-forward


def clamped_gate(g: torch.Tensor, u: torch.Tensor, limit: float) -> torch.Tensor:
    """g sigmoid(1.702 g) (u + 1) with g held below ``limit`` and u between -limit and limit."""
    g, u = torch.clamp(g, max=limit), torch.clamp(u, min=-limit, max=limit)
    return g * torch.sigmoid(1.702 * g) * (u + 1)


def expert(h: torch.Tensor, w: dict, p: str, limit: float) -> torch.Tensor:
    return kept(clamped_gate(kept(h @ w[f"{p}.gate"].T), kept(h @ w[f"{p}.up"].T), limit)) @ w[f"{p}.down"].T


def table_experts(h: torch.Tensor, tokens: list[int], w: dict, p: str, mlp: dict) -> torch.Tensor:
    """A token's experts are its id's row of the table, in equal parts."""
    top, limit = int(mlp["router"]["top"]), float(mlp["expert"]["limit"])
    out = torch.zeros_like(h)
    for t, token in enumerate(tokens):
        for e in w[f"{p}.table"][token].tolist():
            out[t] += expert(h[t : t + 1], w, f"{p}.e{e}", limit)[0] / top
    return out


# --------------------------------------------------------------------------- the model


MIXERS = {"gla": gla_mixer, "parallel": parallel_mixer}


def run_order(cfg: dict) -> list[tuple[int, bool]]:
    """(layer, whether the embedding's output is added in front of it) in the order the layers run."""
    n, loop = len(cfg["layers"]), cfg.get("loop")
    if not loop:
        return [(i, False) for i in range(n)]
    a, b = int(loop["start"]), int(loop["stop"])
    order = [(i, False) for i in range(a)]
    for t in range(int(loop["times"])):
        order += [(i, t > 0 and i == a) for i in range(a, b)]
    return order + [(i, False) for i in range(b, n)]


def layer(x: torch.Tensor, tokens: list[int], w: dict, i: int, cfg: dict) -> torch.Tensor:
    eps, entry = float(cfg["norm"]["eps"]), cfg["layers"][i]
    x = x + MIXERS[entry["type"]](kept(rms(x, eps) * w[f"l{i}.norm1"]), w, f"l{i}.mix", entry["mixer"], eps)
    if entry.get("mlp") is not None:
        x = x + table_experts(kept(rms(x, eps) * w[f"l{i}.norm2"]), tokens, w, f"l{i}.mlp", entry["mlp"])
    return x


def forward(tokens: list[int], w: dict, cfg: dict, streams: list | None = None) -> torch.Tensor:
    """Logits [T, vocab] of one whole sequence; ``streams`` collects the stream after every layer run."""
    x0 = w["embed"][tokens]
    x = x0
    for i, add in run_order(cfg):
        if add:
            x = x + x0
        x = layer(x, tokens, w, i, cfg)
        if streams is not None:
            streams.append(x)
    return kept(rms(x, float(cfg["norm"]["eps"])) * w["final.norm"]) @ w["embed"].T
