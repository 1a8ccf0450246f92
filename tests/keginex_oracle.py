"""A plain float64 formulation of the Keginex design, one function per mechanism, written from the design's equations.
It shares no code with the product path: whole sequences, explicit loops over tokens where a recurrence runs, dense
score matrices with explicit masks, expanded keys and values. Weights arrive as a dict of float64 tensors under the
checkpoint's names.

Notation: W width, H heads, G query/key heads of the delta rule, D key size, V value size, R latent size, n tokens.
"""
import math
from typing import Any, Dict, List, Optional, Tuple

import torch

F64 = torch.float64


def rms_norm(x: torch.Tensor, w: torch.Tensor, eps: float) -> torch.Tensor:
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps) * w


def dyt(x: torch.Tensor, alpha: torch.Tensor, w: torch.Tensor, b: torch.Tensor) -> torch.Tensor:
    return torch.tanh(alpha * x) * w + b


def norm(x: torch.Tensor, weights: Dict[str, torch.Tensor], name: str) -> torch.Tensor:
    return dyt(x, weights[name + ".alpha"].reshape(()), weights[name], weights[name + ".b"])


def silu(z: torch.Tensor) -> torch.Tensor:
    return z * torch.sigmoid(z)


def softplus(z: torch.Tensor) -> torch.Tensor:
    return torch.clamp(z, min=0) + torch.log1p(torch.exp(-torch.abs(z)))


def position_vector(p: int, width: int) -> torch.Tensor:
    out = torch.zeros(width, dtype=F64)
    for c in range(width):
        a = p * 10000.0 ** (-2.0 * (c // 2) / width)
        out[c] = math.cos(a) if c % 2 else math.sin(a)
    return out


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


def unit(x: torch.Tensor) -> torch.Tensor:
    return x / torch.sqrt((x * x).sum(-1, keepdim=True) + 1e-6)


def delta_rule(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, g: torch.Tensor, beta: torch.Tensor,
               state: Optional[torch.Tensor] = None) -> Tuple[torch.Tensor, torch.Tensor]:
    """q, k [n, G, D] (as they enter the recurrence), v [n, H, V], g [n, H, D] factors, beta [n, H] -> read-outs
    [n, H, V] and the last state [H, D, V]."""
    n, H, V = v.shape
    G, D = q.shape[1], q.shape[2]
    S = torch.zeros(H, D, V, dtype=F64) if state is None else state.clone()
    out = torch.zeros(n, H, V, dtype=F64)
    for t in range(n):
        for h in range(H):
            kk, qq = k[t, h // (H // G)], q[t, h // (H // G)]
            A = g[t, h].unsqueeze(1) * S[h]
            u = beta[t, h] * (v[t, h] - A.T @ kk)
            S[h] = A + torch.outer(kk, u)
            out[t, h] = S[h].T @ qq
    return out, S


def channel_delta(h: torch.Tensor, w: Dict[str, torch.Tensor], p: str, m: Dict[str, Any], eps: float) -> torch.Tensor:
    n, H, G, D, V = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q, k, v = (silu(causal_conv(h @ w[p + c].T, w[p + c + ".conv"])) for c in "qkv")
    q, k, v = unit(q.view(n, G, D)) * D ** -0.5, unit(k.view(n, G, D)), v.view(n, H, V)
    beta = torch.sigmoid(h @ w[p + "b"].T)
    z = (h @ w[p + "a1"].T @ w[p + "a2"].T + w[p + "dt_bias"]).view(n, H, D)
    g = torch.exp(-torch.exp(w[p + "A_log"]).view(1, H, 1) * softplus(z))
    o, _ = delta_rule(q, k, v, g, beta)
    o = rms_norm(o, w[p + "norm"], eps).reshape(n, H * V)
    return (o * torch.sigmoid(h @ w[p + "g1"].T @ w[p + "g2"].T)) @ w[p + "o"].T


def latent_attention(h: torch.Tensor, w: Dict[str, torch.Tensor], p: str, m: Dict[str, Any], eps: float) -> torch.Tensor:
    n, H, D, V = h.shape[0], m["heads"], m["dim"], m["vdim"]
    q = (rms_norm(h @ w[p + "dq"].T, w[p + "dq.norm"], eps) @ w[p + "uq"].T).view(n, H, D)
    c = rms_norm(h @ w[p + "dkv"].T, w[p + "dkv.norm"], eps)
    k, v = (c @ w[p + "uk"].T).view(n, H, D), (c @ w[p + "uv"].T).view(n, H, V)
    out = torch.zeros(n, H, V, dtype=F64)
    for i in range(n):
        for hd in range(H):
            s = (k[:i + 1, hd] @ q[i, hd]) * m["scale"]
            top = max(float(s.max()), float(w[p + "sink"][hd]))
            e = torch.exp(s - top)
            out[i, hd] = (e.unsqueeze(1) * v[:i + 1, hd]).sum(0) / (e.sum() + torch.exp(w[p + "sink"][hd] - top))
    return out.reshape(n, H * V) @ w[p + "o"].T


def route(z: torch.Tensor, correction: torch.Tensor, router: Dict[str, Any]) -> List[Tuple[List[int], torch.Tensor]]:
    """Logits z [n, E] -> per token the chosen experts and their weights."""
    E, top = router["experts"], router["top"]
    groups = router.get("groups") or {"count": 1, "keep": 1}
    size = E // groups["count"]
    out = []
    for row in z:
        s = torch.exp(row - row.max())
        s = s / s.sum()
        c = s + correction
        best = sorted(range(groups["count"]), key=lambda a: -float(c[a * size:(a + 1) * size].max()))[:groups["keep"]]
        able = [e for e in range(E) if e // size in best]
        chosen = sorted(able, key=lambda e: -float(c[e]))[:top]
        out.append((chosen, s[chosen] / (s[chosen].sum() + 1e-20) * router["scale"]))
    return out


def gated(h: torch.Tensor, w: Dict[str, torch.Tensor], p: str) -> torch.Tensor:
    return (silu(h @ w[p + "gate"].T) * (h @ w[p + "up"].T)) @ w[p + "down"].T


def mixture(h: torch.Tensor, w: Dict[str, torch.Tensor], p: str, e: Dict[str, Any]) -> torch.Tensor:
    out = torch.zeros_like(h)
    for t, (chosen, weights) in enumerate(route(h @ w[p + "router"].T, w[p + "correction"], e["router"])):
        for x, a in zip(chosen, weights):
            out[t] += a * gated(h[t:t + 1], w, p + f"e{x}.")[0]
    if e.get("shared"):
        out = out + torch.sigmoid(h @ w[p + "shared.sg"].T) * gated(h, w, p + "shared.")
    return out


def relu_squared(h: torch.Tensor, w: Dict[str, torch.Tensor], p: str) -> torch.Tensor:
    return torch.clamp(h @ w[p + "up"].T, min=0).pow(2) @ w[p + "down"].T


def runs(cfg: Dict[str, Any]) -> List[Tuple[int, Optional[int]]]:
    """(layer, number of the pass that begins with it or None), in order."""
    n, loop = len(cfg["layers"]), cfg.get("loop")
    if not loop:
        return [(i, None) for i in range(n)]
    a, b = loop["start"], loop["stop"]
    out = [(i, None) for i in range(a)]
    for t in range(loop["times"]):
        out += [(i, t if i == a else None) for i in range(a, b)]
    return out + [(i, None) for i in range(b, n)]


def forward(cfg: Dict[str, Any], w: Dict[str, torch.Tensor], tokens: List[int]) -> Tuple[torch.Tensor, List[torch.Tensor]]:
    """Logits [n, vocab] and the stream after every layer run."""
    eps = cfg["norm"]["eps"]
    x = w["embed"][tokens] + torch.stack([position_vector(p, cfg["width"]) for p in range(len(tokens))])
    x0, layers = x, []
    for i, begins in runs(cfg):
        if begins is not None:
            x = torch.cat([x, x0], 1) @ w["loop.in"].T + w["loop.step"][begins]
        p, spec = f"l{i}.", cfg["layers"][i]
        mixer = channel_delta if spec["type"] == "channel_delta" else latent_attention
        x = x + norm(mixer(norm(x, w, p + "norm1"), w, p + "mix.", spec["mixer"], eps), w, p + "norm1b")
        e = spec.get("mlp")
        if e:
            h = norm(x, w, p + "norm2")
            y = relu_squared(h, w, p + "mlp.") if e["kind"] == "dense" else mixture(h, w, p + "mlp.", e)
            x = x + norm(y, w, p + "norm2b")
        layers.append(x)
    z = norm(x, w, "final.norm") @ w["head"].T
    cap = cfg.get("logit_softcap")
    return (cap * torch.tanh(z / cap) if cap else z), layers


def greedy(cfg: Dict[str, Any], w: Dict[str, torch.Tensor], prompt: List[int], n: int) -> List[int]:
    toks = list(prompt)
    for _ in range(n):
        toks.append(int(forward(cfg, w, toks)[0][-1].argmax()))
    return toks[len(prompt):]
