"""Element-wise norm ("dynamic tanh") on an fp32 residual stream, and what stands around it:

    N(z) = tanh(alpha z) * w + b                   alpha one number, w and b vectors over the channels; no statistics
    x   <- x + N_b(y)                              closing a sublayer; the next norm N(x) comes out of the same launch
    x   <- p + c + s                               entering a pass over a span of layers: p, c fp32 products, s a vector
    x_0  = E[token] + P(position)                  P[2i] = sin(p base^(-2i/W)), P[2i+1] = cos of the same

GPU: ``csrc/hip/tanh_norm.hip``. CPU: PyTorch formulations of the same arithmetic (fp32).
"""
from typing import Optional, Tuple

import torch

from . import _lib as L

Norm = Tuple[torch.Tensor, torch.Tensor, torch.Tensor]  # (alpha [1], w [W], b [W]) in the compute dtype


class Routed:
    """A sublayer's output that is still in pieces: expert rows ys [T k, W] in expert order, `inv` their places, fp32
    weights wt [T, k]; optionally the shared expert's rows with one gate logit per token (sg [T] fp32, any stride)."""

    def __init__(self, ys, inv, wt, y_shared=None, sg=None):
        self.ys, self.inv, self.wt, self.y_shared, self.sg = ys, inv, wt, y_shared, sg

    def total(self) -> torch.Tensor:
        T, k = self.wt.shape
        y = (self.ys[self.inv].view(T, k, -1).float() * self.wt.view(T, k, 1)).sum(1)
        if self.y_shared is not None:
            y = y + (torch.sigmoid(self.sg).view(T, 1) if self.sg is not None else 1.0) * self.y_shared.float()
        return y


def _norm(z: torch.Tensor, n: Norm) -> torch.Tensor:
    return torch.tanh(n[0].float() * z) * n[1].float() + n[2].float()


def sinusoid_frequencies(width: int, base: float, device) -> torch.Tensor:
    """fp64 [(width + 1) / 2]: angle per position of every (sine, cosine) pair of channels."""
    i = torch.arange((width + 1) // 2, dtype=torch.float64)
    return torch.pow(torch.tensor(float(base), dtype=torch.float64), -2.0 * i / width).to(device)


def embed_sinusoid(tokens: torch.Tensor, positions: torch.Tensor, embed: torch.Tensor, freq: torch.Tensor,
                   want_copy: bool = False) -> Tuple[torch.Tensor, Optional[torch.Tensor]]:
    """tokens int64 [T], positions int32 [T] -> (fp32 stream [T, W], with `want_copy` the same in embed's dtype)."""
    T, W = tokens.numel(), embed.shape[1]
    f32 = embed.dtype == torch.float32
    if L.use_hip(embed):
        assert tokens.dtype == torch.int64 and positions.dtype == torch.int32 and embed.is_contiguous()
        assert positions.numel() == T and freq.dtype == torch.float64 and freq.numel() == (W + 1) // 2
        x = torch.empty(T, W, dtype=torch.float32, device=embed.device)
        xc = torch.empty(T, W, dtype=embed.dtype, device=embed.device) if want_copy and not f32 else None
        L.check(L.lib().areal_embed_sinusoid(L.ptr(tokens), L.ptr(positions), L.ptr(embed), L.ptr(freq),
                                             L.c_int(embed.shape[0]), L.ptr(x), L.ptr(xc), L.c_int(T), L.c_int(W),
                                             L.c_int(L.dtype_flag(embed)), L.stream_ptr()), "embed_sinusoid")
        return x, ((x if f32 else xc) if want_copy else None)
    a = positions.double().view(T, 1) * freq
    x = embed[tokens].float() + torch.stack([a.sin(), a.cos()], -1).view(T, -1)[:, :W].float()
    return x, (x.to(embed.dtype) if want_copy else None)


def _launch(x, y, b: Optional[Norm], enter, nxt: Optional[Norm], want32, want_copy, dtype, out, store=True):
    T, W = out.shape
    f32 = dtype == torch.float32
    routed, slabs = isinstance(y, Routed), 0
    for n in (b, nxt):
        assert n is None or (all(t.dtype == dtype for t in n) and n[0].numel() == 1 and n[1].numel() == W and n[2].numel() == W)
    if routed:
        k = y.wt.shape[1]
        assert y.ys.dtype == dtype and y.ys.is_contiguous() and y.ys.shape[1] == W and y.inv.dtype == torch.int64
        assert y.inv.numel() == T * k and y.wt.dtype == torch.float32 and y.wt.is_contiguous() and y.wt.shape[0] == T
        if y.y_shared is not None:
            assert y.y_shared.dtype == dtype and y.y_shared.is_contiguous() and y.y_shared.shape == (T, W)
            assert y.sg.dtype == torch.float32 and y.sg.dim() == 1 and y.sg.numel() == T
    elif y is not None:
        slabs = y.shape[0] if y.dim() == 3 else 0
        assert y.is_contiguous() and y.shape[-2:] == (T, W) and y.dtype == (torch.float32 if slabs else dtype)
    o32 = oc = None
    if nxt is not None:
        o32 = torch.empty(T, W, dtype=torch.float32, device=out.device) if want32 or f32 else None
    if (nxt is not None or want_copy) and not f32:
        oc = torch.empty(T, W, dtype=dtype, device=out.device)
    p, c, s = enter if enter is not None else (None, None, None)
    for t in (p, c):
        assert t is None or (t.dtype == torch.float32 and t.is_contiguous() and t.shape == (T, W))
    assert s is None or (s.dtype == dtype and s.numel() == W and s.is_contiguous())
    r = y if routed else None
    L.check(L.lib().areal_tanh_norm_step(
        L.ptr(x), L.ptr(r.ys if routed else y), L.c_int(slabs), L.ptr(r.inv) if routed else None,
        L.ptr(r.wt) if routed else None, L.c_int(r.wt.shape[1] if routed else 0),
        L.ptr(r.y_shared) if routed else None, L.ptr(r.sg) if routed and r.y_shared is not None else None,
        L.c_int64(r.sg.stride(0) if routed and r.sg is not None else 0), *(L.ptr(t) for t in (b or (None,) * 3)), L.ptr(p),
        L.ptr(c), L.ptr(s), *(L.ptr(t) for t in (nxt or (None,) * 3)), L.ptr(out) if store else None, L.ptr(o32), L.ptr(oc), L.c_int(T),
        L.c_int(W), L.c_int(L.dtype_flag(torch.empty(0, dtype=dtype))), L.stream_ptr()), "tanh_norm_step")
    if nxt is not None:
        return out, o32, (o32 if f32 else oc)
    return out, None, ((out if f32 else oc) if want_copy else None)


def _handed_on(x, nxt, want_copy, dtype):
    if nxt is not None:
        h = _norm(x, nxt)
        return x, h, h.to(dtype)
    return x, None, (x.to(dtype) if want_copy else None)


def norm_add(x: torch.Tensor, y, b: Optional[Norm], nxt: Optional[Norm], dtype: torch.dtype, want32: bool = False,
             want_copy: bool = False) -> Tuple[torch.Tensor, Optional[torch.Tensor], Optional[torch.Tensor]]:
    """x + N_b(y) on the fp32 stream x [T, W], in place (y None: x as it is). y: [T, W] in the compute dtype, fp32 [S, T, W]
    (the sum of S slabs), or `Routed`. Returns (x, N_nxt(x) in fp32 or None unless `want32` / the compute dtype is fp32,
    N_nxt(x) in the compute dtype); without `nxt` the last one is x itself in the compute dtype (`want_copy`) or None."""
    assert x.dtype == torch.float32 and x.dim() == 2 and x.is_contiguous()
    if L.use_hip(x):
        return _launch(x, y, b, None, nxt, want32, want_copy, dtype, x, store=y is not None)
    if y is not None:
        z = y.total() if isinstance(y, Routed) else (y.sum(0) if y.dim() == 3 else y.float())
        x = x.add_(_norm(z, b))
    return _handed_on(x, nxt, want_copy, dtype)


def enter_pass(p: torch.Tensor, c: torch.Tensor, step: torch.Tensor, out: torch.Tensor, nxt: Norm, dtype: torch.dtype):
    """out fp32 [T, W] <- p + c + step (p, c fp32 [T, W]; step [W] in the compute dtype); returns as `norm_add`."""
    if L.use_hip(out):
        return _launch(None, None, None, (p, c, step), nxt, False, False, dtype, out)
    out.copy_(p + c + step.float())
    return _handed_on(out, nxt, False, dtype)


def softcap_(z: torch.Tensor, cap: float) -> torch.Tensor:
    """z <- cap tanh(z / cap), in place (z contiguous, fp32 or bf16; the arithmetic is fp32)."""
    if L.use_hip(z):
        assert z.is_contiguous()
        L.check(L.lib().areal_softcap(L.ptr(z), L.c_int64(z.numel()), L.c_float(cap), L.c_int(L.dtype_flag(z)), L.stream_ptr()),
                "softcap")
        return z
    return z.copy_(cap * torch.tanh(z.float() / cap))
