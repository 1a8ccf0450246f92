"""Sublayers between two norms on an fp32 residual stream, and what feeds them.

    h        = LN(x)                                   layer norm with weight and bias, fp32 statistics
    x       <- x + s * LN'(y * sigmoid(r))             y: the sublayer's output, r: gate logits (a projection of h),
                                                       s: one scale per channel ("layer scale")
    conv(h)_t = sum_j w[:, j] * h_(t - taps + 1 + j)   causal per-channel convolution over time; the last taps - 1
                                                       inputs of every sequence live in a state slot (`conv_silu`: the
                                                       convolution with a bias and SiLU instead of the sum with h)
    x_0      = LN(E[tok] + B[(prev * a + tok * b) mod n])   token plus hashed-bigram embedding (row n of B for a
                                                       sequence's first token); the previous token lives in a slot

GPU: ``csrc/hip/sandwich.hip``. CPU: PyTorch formulations of the same arithmetic (fp32).

Rows of a packed batch are described as everywhere in the serving path: row b owns tokens cu_q[b]:cu_q[b+1], its
first token has position first_pos[b] and its state lives in slot state_slots[b] (negative: the row is padding and
touches nothing).
"""
from typing import Optional, Tuple

import torch

from . import _lib as L


def layer_norm(x: torch.Tensor, weight: torch.Tensor, bias: torch.Tensor, eps: float, dtype: torch.dtype,
               want32: bool = True) -> Tuple[Optional[torch.Tensor], torch.Tensor]:
    """x fp32 [T, W] -> (LN(x) in fp32 or None when `want32` is False, LN(x) in `dtype`; one tensor when `dtype` is
    fp32)."""
    assert x.dtype == torch.float32 and x.dim() == 2 and x.is_contiguous()
    T, W = x.shape
    if L.use_hip(x):
        assert weight.dtype == dtype and bias.dtype == dtype and weight.numel() == W and bias.numel() == W
        f32 = dtype == torch.float32
        o32 = torch.empty_like(x) if (want32 or f32) else None
        oc = o32 if f32 else torch.empty(T, W, dtype=dtype, device=x.device)
        L.check(L.lib().areal_layer_norm32(L.ptr(x), L.ptr(weight), L.ptr(bias), L.ptr(o32),
                                           None if f32 else L.ptr(oc), L.c_int(T), L.c_int(W), L.c_float(eps),
                                           L.c_int(L.dtype_flag(weight)), L.stream_ptr()), "layer_norm32")
        return o32, oc
    m = x.mean(-1, keepdim=True)
    d = x - m
    h = d * torch.rsqrt(d.pow(2).mean(-1, keepdim=True) + eps) * weight.float() + bias.float()
    return h, (h if dtype == torch.float32 else h.to(dtype))


def gated_norm_add(x: torch.Tensor, y: torch.Tensor, gate: Optional[torch.Tensor], weight: torch.Tensor,
                   bias: torch.Tensor, scale: Optional[torch.Tensor], eps: float,
                   next_norm: Optional[Tuple[torch.Tensor, torch.Tensor]] = None, want32: bool = True):
    """x <- x + scale * LN(y * sigmoid(gate); weight, bias) in place on the fp32 stream x [T, W]; y and gate [T, W] in
    the compute dtype (gate / scale None: left out). With `next_norm` = (weight, bias) the norm of the new x that the
    next sublayer reads is produced by the same launch: returns (x, h32 or None, h in the compute dtype)."""
    assert x.dtype == torch.float32 and x.is_contiguous() and y.shape == x.shape
    T, W = x.shape
    dtype = y.dtype
    if L.use_hip(x):
        assert y.is_contiguous() and (gate is None or (gate.is_contiguous() and gate.dtype == dtype))
        assert weight.dtype == dtype and bias.dtype == dtype and (scale is None or scale.dtype == dtype)
        f32 = dtype == torch.float32
        h32 = hc = None
        if next_norm is not None:
            h32 = torch.empty_like(x) if (want32 or f32) else None
            hc = h32 if f32 else torch.empty(T, W, dtype=dtype, device=x.device)
        L.check(L.lib().areal_gated_norm_add(
            L.ptr(x), L.ptr(y), L.ptr(gate), L.ptr(weight), L.ptr(bias), L.ptr(scale),
            L.ptr(next_norm[0]) if next_norm else None, L.ptr(next_norm[1]) if next_norm else None, L.ptr(h32),
            None if (f32 or hc is None) else L.ptr(hc), L.c_int(T), L.c_int(W), L.c_float(eps),
            L.c_int(L.dtype_flag(y)), L.stream_ptr()), "gated_norm_add")
        return x, h32, hc
    z = y.float()
    if gate is not None:
        z = z * torch.sigmoid(gate.float())
    m = z.mean(-1, keepdim=True)
    d = z - m
    z = d * torch.rsqrt(d.pow(2).mean(-1, keepdim=True) + eps) * weight.float() + bias.float()
    if scale is not None:
        z = z * scale.float()
    x.add_(z)
    if next_norm is None:
        return x, None, None
    h32, hc = layer_norm(x, next_norm[0], next_norm[1], eps, dtype)
    return x, h32, hc


def canon_conv(h: torch.Tensor, weight: torch.Tensor, state: Optional[torch.Tensor], cu_q: torch.Tensor,
               first_pos: torch.Tensor, state_slots: torch.Tensor, dtype: torch.dtype) -> torch.Tensor:
    """h fp32 [T, W] -> h + conv(h) in `dtype`, with weight [W, taps] and state fp32 [slots, taps - 1, W] (entry k of a
    slot: the input taps - 1 - k tokens before the row's first token; None when taps == 1). Positions before a
    sequence's start count as zeros, so a slot's old contents do not matter to a row that starts at position 0.
    Afterwards every row's slot holds its last taps - 1 inputs."""
    assert h.dtype == torch.float32 and h.is_contiguous()
    T, W = h.shape
    taps = weight.shape[1]
    assert weight.shape[0] == W and weight.is_contiguous()
    assert taps == 1 or (state is not None and state.shape[1:] == (taps - 1, W) and state.dtype == torch.float32)
    B = cu_q.numel() - 1
    if L.use_hip(h):
        assert weight.dtype == dtype and cu_q.dtype == torch.int32 and first_pos.dtype == torch.int32
        assert state_slots.dtype == torch.int32
        out = torch.empty(T, W, dtype=dtype, device=h.device)
        L.check(L.lib().areal_canon_conv(L.ptr(h), L.ptr(weight), L.ptr(state), L.ptr(cu_q), L.ptr(first_pos),
                                         L.ptr(state_slots), L.ptr(out), L.c_int(B), L.c_int(T), L.c_int(W),
                                         L.c_int(taps), L.c_int(L.dtype_flag(weight)), L.stream_ptr()), "canon_conv")
        return out
    conv = _causal_conv_cpu(h, weight, state, cu_q, first_pos, state_slots)
    out = h + conv
    return out if dtype == torch.float32 else out.to(dtype)


def stream_conv(x: torch.Tensor, weight: Optional[torch.Tensor], state: Optional[torch.Tensor], cu_q: torch.Tensor,
                first_pos: torch.Tensor, state_slots: torch.Tensor, dtype: torch.dtype) -> torch.Tensor:
    """`canon_conv` of the stream itself; without a weight the stream in `dtype`."""
    if weight is None:
        return x if dtype == torch.float32 else x.to(dtype)
    return canon_conv(x, weight, state, cu_q, first_pos, state_slots, dtype)


def norm_add_conv(x: torch.Tensor, y: torch.Tensor, weight: torch.Tensor, bias: torch.Tensor, eps: float,
                  conv: Optional[Tuple[Optional[torch.Tensor], Optional[torch.Tensor]]], cu_q: torch.Tensor,
                  first_pos: torch.Tensor, state_slots: torch.Tensor, max_q: int = 0
                  ) -> Tuple[torch.Tensor, Optional[torch.Tensor]]:
    """x + LN(y; weight, bias) on the fp32 stream x [T, W] (x itself may be overwritten) and, with `conv` = (weight, state),
    `stream_conv` of the sum in the weights' dtype: one launch for up to four taps and 8192 channels. y [T, W] in the compute
    dtype, or fp32 [S, T, W]: the sum of S slabs (a split GEMM's partial products). `max_q`: longest row when it is known.
    Returns (new stream, convolved stream or None)."""
    T, W = x.shape
    dtype = weight.dtype
    slabs = y.shape[0] if y.dim() == 3 else 0
    assert y.shape[-2:] == x.shape and y.dtype == (torch.float32 if slabs else dtype)
    cw, state = conv if conv is not None else (None, None)
    taps = cw.shape[1] if cw is not None else 0
    if L.use_hip(x) and L.lib().areal_norm_add_conv_serves(L.c_int(W), L.c_int(taps)):
        assert x.is_contiguous() and y.is_contiguous() and bias.dtype == dtype
        assert weight.numel() == W and bias.numel() == W
        assert taps == 0 or (cw.is_contiguous() and cw.shape[0] == W and cw.dtype == dtype)
        assert taps <= 1 or (state.shape[1:] == (taps - 1, W) and state.dtype == torch.float32 and state.is_contiguous())
        assert cu_q.dtype == torch.int32 and first_pos.dtype == torch.int32 and state_slots.dtype == torch.int32
        if all(t.data_ptr() % 16 == 0 for t in (x, y, weight, bias, *([cw] if taps else []))):
            xo = torch.empty_like(x)
            hc = torch.empty(T, W, dtype=dtype, device=x.device) if taps else None
            L.check(L.lib().areal_norm_add_conv(
                L.ptr(x), L.ptr(y), L.c_int(slabs), L.ptr(weight), L.ptr(bias), L.ptr(cw), L.ptr(state), L.ptr(cu_q),
                L.ptr(first_pos), L.ptr(state_slots), L.ptr(xo), L.ptr(hc), L.c_int(cu_q.numel() - 1), L.c_int(T),
                L.c_int(W), L.c_int(taps), L.c_int(int(max_q)), L.c_float(eps), L.c_int(L.dtype_flag(weight)),
                L.stream_ptr()), "norm_add_conv")
            if conv is not None and cw is None:
                hc = stream_conv(xo, None, None, cu_q, first_pos, state_slots, dtype)
            return xo, hc
    if slabs:
        y = y.sum(0).to(dtype)
    x, _, _ = gated_norm_add(x, y, None, weight, bias, None, eps)
    return x, (None if conv is None else stream_conv(x, cw, state, cu_q, first_pos, state_slots, dtype))


def conv_silu(h: torch.Tensor, weight: torch.Tensor, bias: Optional[torch.Tensor], state: Optional[torch.Tensor],
              cu_q: torch.Tensor, first_pos: torch.Tensor, state_slots: torch.Tensor, max_q: int = 0) -> torch.Tensor:
    """silu(conv(h) + bias) of h [T, W] in the compute dtype (a view with unit column stride), contiguous; weight, state
    and history as in `canon_conv` (the state is fp32 and holds the inputs h exactly)."""
    T, W = h.shape
    taps = weight.shape[1]
    assert weight.shape[0] == W and weight.is_contiguous() and h.stride(1) == 1
    assert taps == 1 or (state is not None and state.shape[1:] == (taps - 1, W) and state.dtype == torch.float32)
    if L.use_hip(h):
        assert weight.dtype == h.dtype and (bias is None or (bias.dtype == h.dtype and bias.numel() == W))
        assert cu_q.dtype == torch.int32 and first_pos.dtype == torch.int32 and state_slots.dtype == torch.int32
        out = torch.empty(T, W, dtype=h.dtype, device=h.device)
        L.check(L.lib().areal_conv_silu(L.ptr(h), L.c_int64(h.stride(0)), L.ptr(weight), L.ptr(bias), L.ptr(state),
                                        L.ptr(cu_q), L.ptr(first_pos), L.ptr(state_slots), L.ptr(out),
                                        L.c_int(cu_q.numel() - 1), L.c_int(T), L.c_int(W), L.c_int(taps),
                                        L.c_int(int(max_q)), L.c_int(L.dtype_flag(h)), L.stream_ptr()), "conv_silu")
        return out
    a = _causal_conv_cpu(h.float(), weight, state, cu_q, first_pos, state_slots)
    if bias is not None:
        a = a + bias.float()
    return (a * torch.sigmoid(a)).to(h.dtype)


def _causal_conv_cpu(h, weight, state, cu_q, first_pos, state_slots):
    """The convolution alone, fp32 (zero for padding rows); rewrites the rows' state slots."""
    out = torch.zeros_like(h)
    w = weight.float()
    taps = w.shape[1]
    K = taps - 1
    cq, fp, ss = cu_q.tolist(), first_pos.tolist(), state_slots.tolist()
    for b in range(len(cq) - 1):
        lo, hi = cq[b], cq[b + 1]
        if hi <= lo or ss[b] < 0:
            continue
        if K == 0:
            out[lo:hi] = h[lo:hi] * w[:, 0]
            continue
        hist = state[ss[b]].clone()  # [K, W], oldest first
        if fp[b] < K:  # before the sequence's start there is nothing
            hist[:K - fp[b]] = 0
        ext = torch.cat([hist, h[lo:hi]], 0)
        n = hi - lo
        for j in range(taps):
            out[lo:hi] += w[:, j] * ext[j:j + n]
        state[ss[b]] = ext[n:n + K]
    return out


def embed_bigram_norm(tokens: torch.Tensor, embed: torch.Tensor, bigram: Optional[torch.Tensor], mul_prev: int,
                      mul_cur: int, weight: torch.Tensor, bias: torch.Tensor, eps: float, cu_q: torch.Tensor,
                      first_pos: torch.Tensor, state_slots: torch.Tensor, prev_state: Optional[torch.Tensor]
                      ) -> torch.Tensor:
    """tokens int64 [T] -> fp32 stream [T, W] = LN(embed[tok] + bigram[row]); row = (prev * mul_prev + tok * mul_cur)
    mod buckets with buckets = bigram rows - 1, the last row for a token at position 0. `prev_state` int32 [slots]:
    the last token every sequence has seen (read by a row's first token, then replaced by the row's last token).
    `bigram` None: the token embedding alone."""
    T = tokens.numel()
    W = embed.shape[1]
    B = cu_q.numel() - 1
    if L.use_hip(embed):
        assert tokens.dtype == torch.int64 and embed.is_contiguous() and (bigram is None or bigram.is_contiguous())
        assert bigram is None or (bigram.dtype == embed.dtype and prev_state is not None
                                  and prev_state.dtype == torch.int32)
        out = torch.empty(T, W, dtype=torch.float32, device=embed.device)
        L.check(L.lib().areal_embed_bigram_norm(
            L.ptr(tokens), L.ptr(embed), L.ptr(bigram), L.c_int(bigram.shape[0] - 1 if bigram is not None else 0),
            L.c_int64(mul_prev), L.c_int64(mul_cur), L.ptr(weight), L.ptr(bias), L.c_float(eps), L.ptr(cu_q),
            L.ptr(first_pos), L.ptr(state_slots), L.ptr(prev_state), L.ptr(out), L.c_int(B), L.c_int(T), L.c_int(W),
            L.c_int(embed.shape[0]), L.c_int(L.dtype_flag(embed)), L.stream_ptr()), "embed_bigram_norm")
        return out
    x = embed[tokens].float()
    if bigram is not None:
        n = bigram.shape[0] - 1
        cq, fp, ss = cu_q.tolist(), first_pos.tolist(), state_slots.tolist()
        rows = torch.zeros(T, dtype=torch.long)
        live = torch.zeros(T, dtype=torch.bool)
        for b in range(B):
            lo, hi = cq[b], cq[b + 1]
            if hi <= lo or ss[b] < 0:
                continue
            tk = tokens[lo:hi].cpu().long()
            prev = torch.cat([prev_state[ss[b]:ss[b] + 1].cpu().long(), tk[:-1]])
            r = (prev * mul_prev + tk * mul_cur) % n
            if fp[b] == 0:
                r[0] = n
            rows[lo:hi] = r
            live[lo:hi] = True
            prev_state[ss[b]] = int(tk[-1])
        add = bigram[rows.to(bigram.device)].float()
        x = x + add * live.to(add.device).unsqueeze(-1)
    m = x.mean(-1, keepdim=True)
    d = x - m
    return d * torch.rsqrt(d.pow(2).mean(-1, keepdim=True) + eps) * weight.float() + bias.float()
