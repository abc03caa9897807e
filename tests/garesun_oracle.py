"""Slow float64 implementation of the Garesun design, one function per
mechanism, written from the design's equations.  It imports nothing from the
package: the tests compare the engine against it.

Weights are a dict name -> float64 tensor; `cfg` is the parsed config.json
(a dict).  Sequences are processed whole, one at a time, with explicit
loops where the loop is the definition.
"""

from __future__ import annotations

import math
from typing import Dict, List, Optional

import torch

F64 = torch.float64


def unit_rms(x: torch.Tensor, eps: float) -> torch.Tensor:
    """x / sqrt(mean(x^2) + eps) over the last axis."""
    return x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps)


def layer_norm(x, w, eps):
    """Centred, divided by the root of the mean squared deviation + eps, weighted."""
    d = x - x.mean(dim=-1, keepdim=True)
    return d / torch.sqrt((d * d).mean(dim=-1, keepdim=True) + eps) * w


def silu(z):
    return z * torch.sigmoid(z)


def gelu_tanh(z):
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def log_sigmoid(z: float) -> float:
    return min(z, 0.0) - math.log1p(math.exp(-abs(z)))


def rotate_halves(v: torch.Tensor, pos: torch.Tensor, base: float, dims: int) -> torch.Tensor:
    """Pairs (i, i + dims/2) of the last axis turn by pos * base^(-2i/dims)."""
    out = v.clone()
    half = dims // 2
    for i in range(half):
        a = pos.to(F64) * base ** (-2.0 * i / dims)
        shape = [-1] + [1] * (v.dim() - 2)
        c, s = torch.cos(a).view(shape), torch.sin(a).view(shape)
        u, w = v[..., i], v[..., i + half]
        out[..., i] = u * c - w * s
        out[..., i + half] = w * c + u * s
    return out


def rotate_neighbours(v: torch.Tensor, pos: torch.Tensor, base: float, dims: int) -> torch.Tensor:
    """Pairs (2i, 2i + 1) of the last axis turn by pos * base^(-2i/dims)."""
    out = v.clone()
    for i in range(dims // 2):
        a = pos.to(F64) * base ** (-2.0 * i / dims)
        shape = [-1] + [1] * (v.dim() - 2)
        c, s = torch.cos(a).view(shape), torch.sin(a).view(shape)
        u, w = v[..., 2 * i], v[..., 2 * i + 1]
        out[..., 2 * i] = u * c - w * s
        out[..., 2 * i + 1] = w * c + u * s
    return out


def retention_recurrence(q, k, v, decay: List[float], state=None):
    """q, k [T, H, D], v [T, H, Dv]: S <- d S + k v^T, o = S^T q per head.
    Returns (o [T, H, Dv], final S [H, D, Dv])."""
    T, H, D = q.shape
    S = torch.zeros(H, D, v.shape[-1], dtype=F64) if state is None else state.clone()
    d = torch.tensor([float(x) for x in decay], dtype=F64).view(H, 1, 1)
    out = []
    for t in range(T):
        S = d * S + k[t][:, :, None] * v[t][:, None, :]
        out.append((q[t][:, None, :] @ S)[:, 0])
    return torch.stack(out), S


def mlstm_recurrence(q, k, v, i_gate, f_gate, state=None):
    """q, k [T, H, D], v [T, H, Dv]; i_gate, f_gate [T, H] are the log gates.
    Matrix S, vector n and running maximum m (all start at zero).  Returns
    (o [T, H, Dv], (S, n, m))."""
    T, H, D = q.shape
    Dv = v.shape[-1]
    if state is None:
        S, n, m = torch.zeros(H, D, Dv, dtype=F64), torch.zeros(H, D, dtype=F64), torch.zeros(H, dtype=F64)
    else:
        S, n, m = (t.clone() for t in state)
    out = torch.zeros(T, H, Dv, dtype=F64)
    for t in range(T):
        m_new = torch.maximum(f_gate[t] + m, i_gate[t])
        a, b = torch.exp(f_gate[t] + m - m_new), torch.exp(i_gate[t] - m_new)
        m = m_new
        S = a[:, None, None] * S + b[:, None, None] * k[t][:, :, None] * v[t][:, None, :]
        n = a[:, None] * n + b[:, None] * k[t]
        den = torch.maximum((n * q[t]).sum(-1).abs(), torch.exp(-m)) + 1e-6
        out[t] = (q[t][:, None, :] @ S)[:, 0] / den[:, None]
    return out, (S, n, m)


def retention(h, W: Dict[str, torch.Tensor], p: str, m: dict, eps: float) -> torch.Tensor:
    T = h.shape[0]
    H, D, Dv = m["heads"], m["dim"], m["vdim"]
    pos = torch.arange(T)
    base, dims = m["rot"]["base"], m["rot"]["dims"]
    q = rotate_halves((h @ W[p + "q"].T).view(T, H, D), pos, base, dims)
    k = rotate_halves((h @ W[p + "k"].T).view(T, H, D), pos, base, dims) * D ** -0.5
    v = (h @ W[p + "v"].T).view(T, H, Dv)
    o, _ = retention_recurrence(q, k, v, m["decay"])
    o = unit_rms(o, eps).reshape(T, H * Dv) * silu(h @ W[p + "g"].T)
    return o @ W[p + "o"].T


def mlstm_gates(h, W, p: str, cap: float):
    """(log input gate, log forget gate), each [T, heads]."""
    i = cap * torch.tanh((h @ W[p + "i"].T + W[p + "i.b"]) / cap)
    f = cap * torch.tanh((h @ W[p + "f"].T + W[p + "f.b"]) / cap)
    return i, torch.nn.functional.logsigmoid(f)


def mlstm(h, W: Dict[str, torch.Tensor], p: str, m: dict, eps: float) -> torch.Tensor:
    T = h.shape[0]
    H, D, Dv = m["heads"], m["dim"], m["vdim"]
    q = (h @ W[p + "q"].T).view(T, H, D) * D ** -0.5
    k = (h @ W[p + "k"].T).view(T, H, D)
    v = (h @ W[p + "v"].T).view(T, H, Dv)
    i, f = mlstm_gates(h, W, p, m["gate_cap"])
    o, _ = mlstm_recurrence(q, k, v, i, f)
    o = unit_rms(o, eps).reshape(T, H * Dv) * W[p + "norm"] * torch.sigmoid(h @ W[p + "g"].T)
    return o @ W[p + "o"].T


def softmax_attention(q, k, v, scale: float) -> torch.Tensor:
    """Causal attention of one sequence.  q, k [T, H, D]; v [T, H, Dv]."""
    T, H, _ = q.shape
    out = torch.zeros(T, H, v.shape[-1], dtype=F64)
    for h in range(H):
        for i in range(T):
            s = (k[: i + 1, h] @ q[i, h]) * scale
            out[i, h] = torch.softmax(s, dim=0) @ v[: i + 1, h]
    return out


def latent_rows(h, W, p: str, m: dict, eps: float):
    """(latent c [T, kv_rank], rotated shared key part [T, rot_dim]): what a
    layer with a down-projection of its own caches."""
    Rk = m["kv_rank"]
    low = h @ W[p + "dkv"].T
    c = unit_rms(low[:, :Rk], eps) * W[p + "dkv.norm"]
    kr = rotate_neighbours(low[:, Rk:], torch.arange(h.shape[0]), m["rot"]["base"], m["rot"]["dims"])
    return c, kr


def latent_attention(h, rows, W, p: str, m: dict) -> torch.Tensor:
    """`rows` = (c, rotated key part) of this layer or of the one it shares with."""
    T = h.shape[0]
    H, D, R, Dv = m["heads"], m["dim"], m["rot_dim"], m["vdim"]
    c, kr = rows
    q = (h @ W[p + "q"].T).view(T, H, D + R)
    qr = rotate_neighbours(q[..., D:], torch.arange(T), m["rot"]["base"], m["rot"]["dims"])
    k_un = (c @ W[p + "uk"].T).view(T, H, D)
    val = (c @ W[p + "uv"].T).view(T, H, Dv)
    qf = torch.cat([q[..., :D], qr], dim=-1)
    kf = torch.cat([k_un, kr[:, None, :].expand(T, H, R)], dim=-1)
    o = softmax_attention(qf, kf, val, m["scale"])
    o = o * torch.sigmoid(h @ W[p + "g"].T)[:, :, None]
    return o.reshape(T, H * Dv) @ W[p + "o"].T


def relu2_ff(h, W, p: str) -> torch.Tensor:
    return torch.relu(h @ W[p + "up"].T).pow(2) @ W[p + "down"].T


def route(z: torch.Tensor, top: int):
    """The `top` largest logits of one token and the softmax over them."""
    val, idx = torch.topk(z, top)
    return idx.tolist(), torch.softmax(val, dim=0).tolist()


def moe_ff(h, W, p: str, mlp: dict) -> torch.Tensor:
    z = h @ W[p + "router"].T
    out = torch.zeros(h.shape[0], W[p + "e0.down"].shape[0], dtype=F64)
    for t in range(h.shape[0]):
        for e, w in zip(*route(z[t], mlp["router"]["top"])):
            out[t] += w * relu2_ff(h[t], W, f"{p}e{e}.")
    if mlp.get("shared"):
        out = out + relu2_ff(h, W, p + "shared.")
    return out


def token_side(x, tokens, W, i: int, dim: int, eps: float) -> torch.Tensor:
    """What the per-layer token table adds to the residual after layer i."""
    p = f"l{i}.side."
    e = W["side.embed"][tokens][:, i * dim : (i + 1) * dim]
    y = (gelu_tanh(x @ W[p + "gate"].T) * e) @ W[p + "proj"].T
    return unit_rms(y, eps) * W[p + "norm"]


def forward(cfg: dict, W: Dict[str, torch.Tensor], tokens: List[int], residuals: Optional[list] = None):
    """Logits [T, vocab] of one whole sequence (float64)."""
    W = {k: v.to(F64) for k, v in W.items()}
    eps = cfg["norm"]["eps"]
    tok = torch.tensor(tokens)
    x = W["embed"][tok] * cfg["embedding"]["scale"]
    rows = {}  # layer -> its latent rows, for the layers that share them
    for i, spec in enumerate(cfg["layers"]):
        p, m = f"l{i}.", spec["mixer"]
        h = layer_norm(x, W[p + "norm1"], eps)
        if spec["type"] == "retention":
            y = retention(h, W, p + "mix.", m, eps)
        elif spec["type"] == "mlstm":
            y = mlstm(h, W, p + "mix.", m, eps)
        else:
            src = m.get("kv_from")
            rows[i] = rows[src] if src is not None else latent_rows(h, W, p + "mix.", m, eps)
            y = latent_attention(h, rows[i], W, p + "mix.", m)
        if spec.get("mlp") is not None:
            y = y + moe_ff(h, W, p + "mlp.", spec["mlp"])
        x = x + y
        x = x + token_side(x, tok, W, i, cfg["token_side"]["dim"], eps)
        if residuals is not None:
            residuals.append(x.clone())
    return layer_norm(x, W["final.norm"], eps) @ W["head"].T
