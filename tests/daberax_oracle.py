"""Slow float64 implementation of the Daberax design, one function per
mechanism, written from the design's equations.  It imports nothing from the
package: the tests compare the engine against it.

Weights are a dict name -> float64 tensor; `cfg` is the parsed config.json
(a dict).  Sequences are processed whole, one at a time, with explicit loops
where the loop is the definition.
"""

from __future__ import annotations

import math
from typing import Dict, List, Optional

import torch

F64 = torch.float64


def unit_rms(x: torch.Tensor, eps: float) -> torch.Tensor:
    """x / sqrt(mean(x^2) + eps) over the last axis."""
    return x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps)


def unit_length(x: torch.Tensor) -> torch.Tensor:
    """x / sqrt(sum(x^2) + 1e-6) over the last axis."""
    return x / torch.sqrt((x * x).sum(dim=-1, keepdim=True) + 1e-6)


def silu(z):
    return z * torch.sigmoid(z)


def gelu_tanh(z):
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def softplus(z):
    return torch.clamp(z, min=0.0) + torch.log1p(torch.exp(-z.abs()))


def frequencies(rot: dict) -> List[float]:
    """Angular frequency of every rotated pair, banded scaling included: long
    wavelengths are slowed down by `factor`, short ones kept, a linear ramp
    in original / wavelength between."""
    out = []
    sc = rot.get("scaling")
    for i in range(rot["dims"] // 2):
        f = rot["base"] ** (-2.0 * i / rot["dims"])
        if sc:
            wave = 2.0 * math.pi / f
            if wave > sc["original"] / sc["low"]:
                f = f / sc["factor"]
            elif wave >= sc["original"] / sc["high"]:
                s = (sc["original"] / wave - sc["low"]) / (sc["high"] - sc["low"])
                f = (1.0 - s) * f / sc["factor"] + s * f
        out.append(f)
    return out


def rotate_neighbours(v: torch.Tensor, pos: torch.Tensor, freqs: List[float]) -> torch.Tensor:
    """Pairs (2i, 2i + 1) of the last axis turn by pos * freqs[i]; v [T, ...]."""
    out = v.clone()
    for i, f in enumerate(freqs):
        a = pos.to(F64) * f
        shape = [-1] + [1] * (v.dim() - 2)
        c, s = torch.cos(a).view(shape), torch.sin(a).view(shape)
        u, w = v[..., 2 * i], v[..., 2 * i + 1]
        out[..., 2 * i] = u * c - w * s
        out[..., 2 * i + 1] = w * c + u * s
    return out


def causal_conv(x: torch.Tensor, w: torch.Tensor) -> torch.Tensor:
    """x [T, C], w [C, taps]: y[t, c] = sum_j w[c, j] x[t - (taps - 1) + j, c],
    zeros ahead of the sequence."""
    T, taps = x.shape[0], w.shape[1]
    out = torch.zeros_like(x)
    for t in range(T):
        for j in range(taps):
            at = t - (taps - 1) + j
            if at >= 0:
                out[t] += w[:, j] * x[at]
    return out


def delta_recurrence(q, k, v, g, beta, state=None):
    """q, k [T, H, D], v [T, H, Dv], g, beta [T, H]: decay, then the write
    corrects what the state holds under k, then the read-out.  Returns
    (o [T, H, Dv], final S [H, D, Dv])."""
    T, H, D = q.shape
    S = torch.zeros(H, D, v.shape[-1], dtype=F64) if state is None else state.clone()
    out = []
    for t in range(T):
        S = g[t].view(H, 1, 1) * S
        held = (k[t][:, None, :] @ S)[:, 0]
        u = beta[t].view(H, 1) * (v[t] - held)
        S = S + k[t][:, :, None] * u[:, None, :]
        out.append((q[t][:, None, :] @ S)[:, 0])
    return torch.stack(out), S


def delta_gates(h, W, p: str):
    """(decay g, write strength beta), each [T, heads]."""
    beta = torch.sigmoid(h @ W[p + "b"].T)
    g = torch.exp(-torch.exp(W[p + "A_log"]) * softplus(h @ W[p + "a"].T + W[p + "dt_bias"]))
    return g, beta


def delta(h, W: Dict[str, torch.Tensor], p: str, m: dict, eps: float) -> torch.Tensor:
    T = h.shape[0]
    H, G, D, Dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q, k, v = (silu(causal_conv(h @ W[p + n].T, W[p + n + ".conv"])) for n in "qkv")
    q = unit_length(q.view(T, G, D)) * D ** -0.5
    k = unit_length(k.view(T, G, D))
    q, k = (t.repeat_interleave(H // G, dim=1) for t in (q, k))
    g, beta = delta_gates(h, W, p)
    o, _ = delta_recurrence(q, k, v.view(T, H, Dv), g, beta)
    o = unit_rms(o, eps) * W[p + "norm"]
    o = o.reshape(T, H * Dv) * silu(h @ W[p + "g"].T)
    return o @ W[p + "o"].T


def window_attention(q, k, v, scale: float, window: int = 0, cap: float = 0.0) -> torch.Tensor:
    """Causal softmax attention of one sequence, one query at a time.  q
    [T, H, D]; k [T, G, D], v [T, G, Dv].  Position i sees j <= i with
    i - j < window (0: all); scores may be bent by cap * tanh(score / cap)."""
    T, H, _ = q.shape
    per = H // k.shape[1]
    out = torch.zeros(T, H, v.shape[-1], dtype=F64)
    for h in range(H):
        for i in range(T):
            lo = max(0, i - window + 1) if window > 0 else 0
            s = (k[lo : i + 1, h // per] @ q[i, h]) * scale
            if cap > 0:
                s = cap * torch.tanh(s / cap)
            out[i, h] = torch.softmax(s, dim=0) @ v[lo : i + 1, h // per]
    return out


def window_of(m: dict) -> int:
    return int((m.get("mask") or {}).get("size", 0))


def attention(h, W, p: str, m: dict, eps: float) -> torch.Tensor:
    T = h.shape[0]
    H, G, D, Dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    pos = torch.arange(T)
    q, k, v = (h @ W[p + n].T + W[p + n + ".b"] for n in "qkv")
    q = (unit_rms(q, eps) * W[p + "q.norm"]).view(T, H, D)
    k = (unit_rms(k, eps) * W[p + "k.norm"]).view(T, G, D)
    freqs = frequencies(m["rot"])
    q, k = rotate_neighbours(q, pos, freqs), rotate_neighbours(k, pos, freqs)
    o = window_attention(q, k, v.view(T, G, Dv), m["scale"], window_of(m), m["softcap"])
    o = o * torch.sigmoid(h @ W[p + "g"].T)[:, :, None]
    return o.reshape(T, H * Dv) @ W[p + "o"].T + W[p + "o.b"]


def latent_attention(h, W, p: str, m: dict, eps: float) -> torch.Tensor:
    """Per-head keys and values written out, nothing absorbed."""
    T = h.shape[0]
    H, D, R, Dv, Rk = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    pos, freqs = torch.arange(T), frequencies(m["rot"])
    q = (h @ W[p + "q"].T).view(T, H, D + R)
    q = torch.cat([q[..., :D], rotate_neighbours(q[..., D:], pos, freqs)], dim=-1)
    low = h @ W[p + "dkv"].T
    c = unit_rms(low[:, :Rk], eps) * W[p + "dkv.norm"]
    kr = rotate_neighbours(low[:, Rk:], pos, freqs)
    k = torch.cat([(c @ W[p + "uk"].T).view(T, H, D), kr[:, None, :].expand(T, H, R)], dim=-1)
    v = (c @ W[p + "uv"].T).view(T, H, Dv)
    o = window_attention(q, k, v, m["scale"], window_of(m))
    return o.reshape(T, H * Dv) @ W[p + "o"].T


MIXERS = {"delta": delta, "attention": attention, "latent_attention": latent_attention}


def gated_ff(x, W, p: str) -> torch.Tensor:
    return (gelu_tanh(x @ W[p + "gate"].T) * (x @ W[p + "up"].T)) @ W[p + "down"].T


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
    x = W["embed"][tok]
    for i, spec in enumerate(cfg["layers"]):
        p = f"l{i}."
        y = MIXERS[spec["type"]](x, W, p + "mix.", spec["mixer"], eps)
        x = x + unit_rms(y, eps) * W[p + "norm1"]
        if spec.get("mlp") is not None:
            x = x + unit_rms(gated_ff(x, W, p + "mlp."), eps) * W[p + "norm2"]
        if cfg.get("token_side"):
            x = x + token_side(x, tok, W, i, cfg["token_side"]["dim"], eps)
        if residuals is not None:
            residuals.append(x.clone())
    return (unit_rms(x, eps) * W["final.norm"]) @ W["head"].T * cfg["logit_scale"]
