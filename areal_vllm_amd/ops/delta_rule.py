"""Gated delta rule with one decay per head and key channel: a matrix state per head, carried as fp32 state per request
slot. Queries and keys are unit vectors, the queries times q_scale; heads / kv_heads heads share a query / key head:

    g_t = exp(-exp(A_h) softplus(z_t + bias))       one factor per head and key channel;   beta_t = sigmoid(b_t)
    S'  = diag(g_t) S_(t-1);   u_t = beta_t (v_t - S'^T k_t);   S_t = S' + k_t u_t^T;   o_t = S_t^T q_t

GPU: ``csrc/hip/delta_rule.hip`` (token by token for decoding and short portions; chunks of 16 tokens for prompt
portions: one launch forms what does not depend on the state for all chunks at once, the next walks the chunks with
matrix products only). CPU: the same recurrence in PyTorch, token by token (fp32).
"""
import torch
import torch.nn.functional as F

from . import _lib as L


CHUNK = 16  # tokens per chunk of the chunked form
MAX_KEY = 256  # largest key size the kernels are built for


def alloc_state(n_slots: int, heads: int, k_dim: int, v_dim: int, device) -> torch.Tensor:
    """State slots [slots, heads, V, D] fp32 (the state transposed: a value column's numbers are neighbours). A row that
    starts at position 0 ignores what its slot held, so slots are handed on without clearing."""
    return torch.zeros(n_slots, heads, v_dim, k_dim, dtype=torch.float32, device=device)


def delta_scan(qkv: torch.Tensor, q_off: int, k_off: int, v_off: int, kv_heads: int, z: torch.Tensor,
               z_bias: torch.Tensor, a_log: torch.Tensor, beta: torch.Tensor, q_scale: float, cu_q: torch.Tensor,
               first_pos: torch.Tensor, state_slots: torch.Tensor, state: torch.Tensor, max_q: int = 1,
               unit_eps: float = 1e-6, chunked: bool = True) -> torch.Tensor:
    """Advance the state of every row's slot over the row's tokens. qkv [T, *] holds kv_heads x D queries at column q_off,
    kv_heads x D keys at k_off, heads x V values at v_off; z fp32 [T, heads D]; beta [T, heads] logits (a view with unit
    column stride); z_bias [heads D], a_log [heads], all three in qkv's dtype. first_pos [B] int32: position of each row's
    first token (0: fresh state); state_slots [B] int32 (negative: the row is skipped). Returns [T, heads, V] fp32."""
    T = qkv.shape[0]
    H, V, D = state.shape[1:]
    B, G = cu_q.numel() - 1, int(kv_heads)
    assert H % G == 0 and z.dtype == torch.float32 and z.shape == (T, H * D) and z.stride(1) == 1
    assert beta.shape == (T, H) and beta.stride(1) == 1 and z_bias.numel() == H * D and a_log.numel() == H
    if L.use_hip(qkv):
        assert qkv.stride(1) == 1 and cu_q.dtype == torch.int32 and first_pos.dtype == torch.int32
        assert state_slots.dtype == torch.int32 and state.dtype == torch.float32 and state.is_contiguous()
        assert min(q_off, k_off, v_off) >= 0 and max(q_off + G * D, k_off + G * D, v_off + H * V) <= qkv.shape[1]
        assert beta.dtype == qkv.dtype and z_bias.dtype == qkv.dtype and a_log.dtype == qkv.dtype
        if D > MAX_KEY:
            raise RuntimeError(f"delta rule: key size above {MAX_KEY} is not built")
        obuf = torch.empty(T, H, V, dtype=torch.float32, device=qkv.device)
        scratch = None
        if chunked and max_q >= CHUNK and D <= 128:  # the chunked form's state-independent operands
            fn = L.lib().areal_delta_scratch
            fn.restype = L.c_int64
            scratch = torch.empty(int(fn(L.c_int(T), L.c_int(B), L.c_int(H), L.c_int(D))), dtype=torch.float32,
                                  device=qkv.device)
        L.check(L.lib().areal_delta_scan(
            L.ptr(qkv), L.c_int64(qkv.stride(0)), L.c_int(q_off), L.c_int(k_off), L.c_int(v_off), L.ptr(z),
            L.c_int64(z.stride(0)), L.ptr(z_bias), L.ptr(a_log), L.ptr(beta), L.c_int64(beta.stride(0)), L.c_float(q_scale),
            L.c_float(unit_eps), L.ptr(cu_q), L.ptr(first_pos), L.ptr(state_slots), L.ptr(state), L.ptr(obuf),
            L.ptr(scratch), L.c_int(T), L.c_int(B), L.c_int(H), L.c_int(G), L.c_int(D), L.c_int(V), L.c_int(int(max_q)),
            L.c_int(L.dtype_flag(qkv)), L.stream_ptr()), "delta_scan")
        return obuf
    obuf = torch.zeros(T, H, V, dtype=torch.float32, device=qkv.device)
    cq, fp, sl = cu_q.tolist(), first_pos.tolist(), state_slots.tolist()

    def unit(x):
        x = x.float().reshape(T, G, D)
        x = x * torch.rsqrt(x.pow(2).sum(-1, keepdim=True) + unit_eps)
        return x.repeat_interleave(H // G, 1)

    q, k = unit(qkv[:, q_off:q_off + G * D]) * float(q_scale), unit(qkv[:, k_off:k_off + G * D])
    v = qkv[:, v_off:v_off + H * V].float().reshape(T, H, V)
    g = torch.exp(-torch.exp(a_log.float()).view(1, H, 1) * F.softplus((z + z_bias.float()).view(T, H, D)))
    bt = torch.sigmoid(beta.float())
    for b in range(B):
        if sl[b] < 0 or cq[b + 1] <= cq[b]:
            continue
        S = torch.zeros(H, V, D) if fp[b] == 0 else state[sl[b]].clone()
        for t in range(cq[b], cq[b + 1]):
            S = S * g[t].unsqueeze(1)
            u = bt[t].unsqueeze(1) * (v[t] - torch.einsum("hvd,hd->hv", S, k[t]))
            S = S + u.unsqueeze(2) * k[t].unsqueeze(1)
            obuf[t] = torch.einsum("hvd,hd->hv", S, q[t])
        state[sl[b]] = S
    return obuf
