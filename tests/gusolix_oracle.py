"""A plain float64 formulation of the Gusolix design, one function per mechanism, written from the design's equations.
It shares no code with the product path: whole sequences, explicit loops over tokens where a recurrence runs, dense
score matrices with explicit masks. Weights arrive as a dict of float64 tensors under the checkpoint's names.

Notation: W width, H heads, G key/value heads, D key size, V value size, n tokens.
"""
import math
from typing import Any, Dict, List, Optional, Tuple

import torch

F64 = torch.float64


def layer_norm(x: torch.Tensor, w: torch.Tensor, b: torch.Tensor, eps: float) -> torch.Tensor:
    d = x - x.mean(-1, keepdim=True)
    return d / torch.sqrt((d * d).mean(-1, keepdim=True) + eps) * w + b


def rms_norm(x: torch.Tensor, w: torch.Tensor, eps: float) -> torch.Tensor:
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps) * w


def silu(z: torch.Tensor) -> torch.Tensor:
    return z * torch.sigmoid(z)


def softplus(z: torch.Tensor) -> torch.Tensor:
    return torch.clamp(z, min=0) + torch.log1p(torch.exp(-torch.abs(z)))


def causal_conv(h: torch.Tensor, w: torch.Tensor) -> torch.Tensor:
    """Per channel, the last column of w [channels, taps] on the current token, zeros ahead of the sequence."""
    n, taps = h.shape[0], w.shape[1]
    out = torch.zeros_like(h)
    for t in range(n):
        for j in range(taps):
            s = t - taps + 1 + j
            if s >= 0:
                out[t] += w[:, j] * h[s]
    return out


def with_history(h: torch.Tensor, w: torch.Tensor) -> torch.Tensor:
    """What a sublayer reads: its input plus the convolution of it."""
    return h + causal_conv(h, w)


def frequencies(base: float, dims: int, scaling: Optional[Dict[str, Any]]) -> List[float]:
    """Turns per position of every rotated pair; long wavelengths are slowed down by `factor`, with a linear blend
    between the two wavelength limits."""
    out = []
    for i in range(dims // 2):
        f = float(base) ** (-2.0 * i / dims)
        if scaling:
            factor, low, high, orig = (float(scaling[k]) for k in ("factor", "low", "high", "original"))
            wl = 2.0 * math.pi / f
            if wl > orig / low:
                f = f / factor
            elif wl >= orig / high:
                s = (orig / wl - low) / (high - low)
                f = (1.0 - s) * f / factor + s * f
        out.append(f)
    return out


def rotate_half(x: torch.Tensor, pos: torch.Tensor, rot: Dict[str, Any]) -> torch.Tensor:
    """x [n, heads, d]: coordinate i with i + dims/2 turned by pos * f_i; coordinates from dims on stay."""
    dims = int(rot["dims"])
    out = x.clone()
    for i, f in enumerate(frequencies(rot["base"], dims, rot.get("scaling"))):
        a = (pos.to(F64) * f).unsqueeze(1)
        u, v = x[:, :, i], x[:, :, i + dims // 2]
        out[:, :, i] = u * torch.cos(a) - v * torch.sin(a)
        out[:, :, i + dims // 2] = v * torch.cos(a) + u * torch.sin(a)
    return out


def attention_weights(q: torch.Tensor, k: torch.Tensor, scale: float, chunk: int) -> torch.Tensor:
    """q [n, H, D], k [n, G, D] -> softmax weights [H, n, n]; with chunk > 0 a query sees its own chunk only."""
    n, H, G = q.shape[0], q.shape[1], k.shape[1]
    out = torch.zeros(H, n, n, dtype=F64)
    i, j = torch.arange(n).unsqueeze(1), torch.arange(n).unsqueeze(0)
    seen = j <= i
    if chunk > 0:
        seen = seen & (i // chunk == j // chunk)
    for h in range(H):
        s = (q[:, h] @ k[:, h // (H // G)].T) * scale
        out[h] = torch.softmax(s.masked_fill(~seen, float("-inf")), -1)
    return out


def chunked_attention(h: torch.Tensor, w: Dict[str, torch.Tensor], p: str, m: Dict[str, Any], eps: float) -> torch.Tensor:
    """Rotated grouped-query attention inside chunks of positions; the keys as projected are the values."""
    n, H, G, D = h.shape[0], m["heads"], m["kv_heads"], m["dim"]
    pos = torch.arange(n)
    kraw = h @ w[p + "k"].T
    q = rms_norm(h @ w[p + "q"].T, w[p + "q.norm"], eps).view(n, H, D)
    k = rms_norm(kraw, w[p + "k.norm"], eps).view(n, G, D)
    if m.get("rot"):
        q, k = rotate_half(q, pos, m["rot"]), rotate_half(k, pos, m["rot"])
    pr = attention_weights(q, k, m["scale"], int((m.get("mask") or {}).get("size") or 0))
    v = kraw.view(n, G, D)
    o = torch.stack([pr[hd] @ v[:, hd // (H // G)] for hd in range(H)], 1)
    return o.reshape(n, H * D) @ w[p + "o"].T


def mixed_attention(h: torch.Tensor, w: Dict[str, torch.Tensor], p: str, m: Dict[str, Any], eps: float) -> torch.Tensor:
    """Causal grouped-query attention without rotation whose softmax weights are mixed over the heads."""
    n, H, G, D, V = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = rms_norm(h @ w[p + "q"].T, w[p + "q.norm"], eps).view(n, H, D)
    k = rms_norm(h @ w[p + "k"].T, w[p + "k.norm"], eps).view(n, G, D)
    v = (h @ w[p + "v"].T).view(n, G, V)
    pr = attention_weights(q, k, m["scale"], 0)
    mixed = torch.einsum("hg,gij->hij", w[p + "talk"], pr)
    o = torch.stack([mixed[hd] @ v[:, hd // (H // G)] for hd in range(H)], 1)
    return o.reshape(n, H * V) @ w[p + "o"].T


def gla(h: torch.Tensor, w: Dict[str, torch.Tensor], p: str, m: Dict[str, Any], eps: float) -> torch.Tensor:
    """Gated linear attention, token by token."""
    n, H, D, V, tau = h.shape[0], m["heads"], m["dim"], m["vdim"], float(m["tau"])
    q = (h @ w[p + "q"].T).view(n, H, D) * D ** -0.5
    k = (h @ w[p + "k"].T).view(n, H, D)
    v = (h @ w[p + "v"].T).view(n, H, V)
    z = (h @ w[p + "a1"].T) @ w[p + "a2"].T + w[p + "a2.b"]
    alpha = torch.sigmoid(z).pow(1.0 / tau).view(n, H, D)
    S = torch.zeros(H, D, V, dtype=F64)
    o = torch.zeros(n, H, V, dtype=F64)
    for t in range(n):
        for hd in range(H):
            S[hd] = alpha[t, hd].unsqueeze(1) * S[hd] + torch.outer(k[t, hd], v[t, hd])
            o[t, hd] = S[hd].T @ q[t, hd]
    y = rms_norm(o, w[p + "norm"], eps).reshape(n, H * V) * silu(h @ w[p + "g"].T)
    return y @ w[p + "o"].T


def selective_scan(x: torch.Tensor, dt: torch.Tensor, A: torch.Tensor, B: torch.Tensor, C: torch.Tensor,
                   D: torch.Tensor) -> torch.Tensor:
    """x, dt [n, channels], A [channels, N], B, C [n, N], D [channels] -> y [n, channels]."""
    S = torch.zeros_like(A)
    y = torch.zeros_like(x)
    for t in range(x.shape[0]):
        S = torch.exp(dt[t].unsqueeze(1) * A) * S + (dt[t] * x[t]).unsqueeze(1) * B[t].unsqueeze(0)
        y[t] = S @ C[t] + D * x[t]
    return y


def mamba(h: torch.Tensor, w: Dict[str, torch.Tensor], p: str, m: Dict[str, Any]) -> torch.Tensor:
    I, R, N = m["inner"], m["dt_rank"], m["state"]
    xz = h @ w[p + "in"].T
    x = silu(causal_conv(xz[:, :I], w[p + "conv"]) + w[p + "conv.b"])
    z = xz[:, I:]
    low = x @ w[p + "x"].T
    dt = softplus(low[:, :R] @ w[p + "dt"].T + w[p + "dt.b"])
    y = selective_scan(x, dt, -torch.exp(w[p + "A_log"]), low[:, R:R + N], low[:, R + N:], w[p + "D"])
    return (y * silu(z)) @ w[p + "o"].T


def parallel_mixer(h: torch.Tensor, w: Dict[str, torch.Tensor], p: str, m: Dict[str, Any], eps: float) -> torch.Tensor:
    return (m["left_scale"] * mixed_attention(h, w, p + "left.", m["left"], eps)
            + m["right_scale"] * gla(h, w, p + "right.", m["right"], eps))


def gated_unit(h: torch.Tensor, w: Dict[str, torch.Tensor], p: str) -> torch.Tensor:
    return (silu(h @ w[p + "gate"].T) * (h @ w[p + "up"].T)) @ w[p + "down"].T


def forward(cfg: Dict[str, Any], w: Dict[str, torch.Tensor], tokens: List[int]) -> Tuple[torch.Tensor, torch.Tensor]:
    """Logits [n, vocab] and the stream after every layer [L, n, W] for one whole sequence."""
    eps = float(cfg["norm"]["eps"])
    x = w["embed"][torch.tensor(tokens)] * float(cfg["embedding"]["scale"])
    after = []
    for i, l in enumerate(cfg["layers"]):
        p = f"l{i}."
        h = with_history(x, w[p + "canon1"])
        if l["type"] == "attention":
            y = chunked_attention(h, w, p + "mix.", l["mixer"], eps)
        elif l["type"] == "mamba1":
            y = mamba(h, w, p + "mix.", l["mixer"])
        else:
            y = parallel_mixer(h, w, p + "mix.", l["mixer"], eps)
        x = x + layer_norm(y, w[p + "norm1"], w[p + "norm1.b"], eps)
        if l.get("mlp"):
            y = gated_unit(with_history(x, w[p + "canon2"]), w, p + "mlp.")
            x = x + layer_norm(y, w[p + "norm2"], w[p + "norm2.b"], eps)
        after.append(x)
    return layer_norm(x, w["final.norm"], w["final.norm.b"], eps) @ w["head"].T, torch.stack(after)


def greedy(cfg: Dict[str, Any], w: Dict[str, torch.Tensor], prompt: List[int], n_new: int) -> List[int]:
    """Greedy continuation, recomputing the whole sequence for every new token."""
    toks, out = list(prompt), []
    for _ in range(n_new):
        logits, _ = forward(cfg, w, toks)
        out.append(int(torch.argmax(logits[-1])))
        toks.append(out[-1])
    return out
