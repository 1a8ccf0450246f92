"""Selective scan (Gu and Dao, "Mamba: Linear-Time Sequence Modeling with Selective State Spaces"): a diagonal recurrence
per channel, carried as fp32 state per request slot:

    dt_t = softplus(r_t + bias)                                           r_t [channels]: fp32
    S_t[n, c] = exp(dt_t[c] A[c, n]) S_(t-1)[n, c] + dt_t[c] x_t[c] B_t[n],   A = -exp(A_log)
    out_t[c]  = (sum_n S_t[n, c] C_t[n] + D[c] x_t[c]) * silu(z_t[c])

GPU: ``csrc/hip/mamba.hip``. CPU: the same recurrence in PyTorch, token by token (fp32). The short convolution ahead of it
is ``ops/sandwich.py::conv_silu``.
"""
import torch
import torch.nn.functional as F

from . import _lib as L


def alloc_state(n_slots: int, channels: int, n_state: int, device) -> torch.Tensor:
    """State slots [slots, N, channels] fp32. A row that starts at position 0 ignores what its slot held, so slots are
    handed on without clearing."""
    return torch.zeros(n_slots, n_state, channels, dtype=torch.float32, device=device)


def selective_scan(x: torch.Tensor, r: torch.Tensor, dt_bias: torch.Tensor, a_log: torch.Tensor, bc: torch.Tensor,
                   d_skip: torch.Tensor, z: torch.Tensor, cu_q: torch.Tensor, first_pos: torch.Tensor,
                   state_slots: torch.Tensor, state: torch.Tensor, max_q: int = 1) -> torch.Tensor:
    """Advance the state of every row's slot over the row's tokens. x [T, I] and z [T, I] in the compute dtype (views with
    unit column stride), r fp32 [T, I], bc [T, 2 N]: read-in | read-out weights (a view), a_log [I, N]. first_pos [B] int32:
    position of each row's first token (0: fresh state); state_slots [B] int32 (negative: the row is skipped). Returns the
    gated read-out [T, I] in the compute dtype."""
    T, I = x.shape
    N = state.shape[1]
    B = cu_q.numel() - 1
    assert state.shape[2] == I and bc.shape == (T, 2 * N) and a_log.shape == (I, N) and z.shape == (T, I)
    assert r.dtype == torch.float32 and r.shape == (T, I)
    if L.use_hip(x):
        for t in (x, z, bc, r):
            assert t.stride(1) == 1
        for t in (z, bc, dt_bias, a_log, d_skip):
            assert t.dtype == x.dtype
        assert a_log.is_contiguous() and dt_bias.numel() == I and d_skip.numel() == I
        assert cu_q.dtype == torch.int32 and first_pos.dtype == torch.int32 and state_slots.dtype == torch.int32
        assert state.dtype == torch.float32 and state.is_contiguous()
        if N > 256:
            raise RuntimeError("selective scan: more than 256 state numbers per channel are not built")
        out = torch.empty(T, I, dtype=x.dtype, device=x.device)
        L.check(L.lib().areal_selective_scan(
            L.ptr(x), L.c_int64(x.stride(0)), L.ptr(r), L.c_int64(r.stride(0)), L.ptr(dt_bias), L.ptr(a_log), L.ptr(bc),
            L.c_int64(bc.stride(0)), L.ptr(d_skip), L.ptr(z), L.c_int64(z.stride(0)), L.ptr(cu_q), L.ptr(first_pos),
            L.ptr(state_slots), L.ptr(state), L.ptr(out), L.c_int(B), L.c_int(I), L.c_int(N), L.c_int(int(max_q)),
            L.c_int(L.dtype_flag(x)), L.stream_ptr()), "selective_scan")
        return out
    y = torch.zeros(T, I)
    cq, fp, sl = cu_q.tolist(), first_pos.tolist(), state_slots.tolist()
    dt = F.softplus(r + dt_bias.float(), threshold=60.0)
    A = -torch.exp(a_log.float()).t()  # [N, I]
    xf, bf = x.float(), bc.float()
    for b in range(B):
        if sl[b] < 0 or cq[b + 1] <= cq[b]:
            continue
        S = torch.zeros(N, I) if fp[b] == 0 else state[sl[b]].clone()
        for t in range(cq[b], cq[b + 1]):
            S = torch.exp(dt[t] * A) * S + (dt[t] * xf[t]) * bf[t, :N].unsqueeze(1)
            y[t] = (S * bf[t, N:].unsqueeze(1)).sum(0) + d_skip.float() * xf[t]
        state[sl[b]] = S
    return (y * F.silu(z.float())).to(x.dtype)
