"""Causal attention over the paged cache whose softmax weights are mixed over the heads before they meet the values:

    p_g(i, j) = softmax_j(q_g(i) . k_c(g)(j) * scale),    w_h = sum_g M[h, g] p_g,    o_h(i) = sum_j w_h(i, j) v_c(h)(j)

with c(g) = g // (H / G). Mixing after the normalisation needs every head's denominator first: two passes over the keys.

GPU: ``csrc/hip/mixed_attn.hip``. CPU: a PyTorch formulation used by the unit tests and CPU runs.

Cache layout: K [pages, G, 32, D], V [pages, G, Dv, 32] (a channel's 32 tokens side by side), any key and value size.
"""
from typing import Optional, Tuple

import torch

from . import _lib as L
from .attention import PAGE_SIZE, decode_num_splits


def alloc_mixed_cache(num_pages: int, n_kv_heads: int, k_dim: int, v_dim: int, dtype, device
                      ) -> Tuple[torch.Tensor, torch.Tensor]:
    return (torch.zeros(num_pages, n_kv_heads, PAGE_SIZE, k_dim, dtype=dtype, device=device),
            torch.zeros(num_pages, n_kv_heads, v_dim, PAGE_SIZE, dtype=dtype, device=device))


def matrix_cores_serve(heads: int, kv_heads: int, k_dim: int, v_dim: int, dtype, device) -> Tuple[bool, bool]:
    """Whether (prompt portions, decoding) of these sizes run the matrix-core kernels: bf16, key and value sizes 64 / 128;
    4, 8, 16 or 32 heads for prompts; at most 64 heads and 16 per key/value head for decoding."""
    if dtype != torch.bfloat16 or torch.device(device).type != "cuda":
        return False, False
    m = int(L.lib().areal_mixed_attn_matrix_cores(L.c_int(heads), L.c_int(kv_heads), L.c_int(k_dim), L.c_int(v_dim)))
    return bool(m & 1), bool(m & 2)


def decode_splits(batch: int, max_context: int, kv_heads: int = 1, matrix_cores: bool = False) -> int:
    """Key-range splits of a decode launch: about two workgroups per compute unit, down to one page each; the matrix-core
    kernels have a workgroup per key/value head and share a split's pages among four waves."""
    if matrix_cores:
        return decode_num_splits(batch, kv_heads, max_context)
    pages = max(1, (max_context + PAGE_SIZE - 1) // PAGE_SIZE)
    return int(max(1, min(512 // max(1, batch), pages, 32)))


def workspace_floats(rows: int, nsplit: int, heads: int, vdim: int, score_keys: int = 0) -> Tuple[int, int]:
    """Floats of the two workspace buffers of a launch over `rows` tokens: partial sums and (`score_keys` per row and head)
    scores, partial softmax statistics."""
    return (rows * nsplit * heads * vdim if nsplit > 1 else 0) + rows * heads * score_keys, rows * nsplit * heads * 2


def mixed_attention(q: torch.Tensor, kcache: torch.Tensor, vcache_t: torch.Tensor, block_tables: torch.Tensor,
                    cu_q: torch.Tensor, ctx_len: torch.Tensor, max_q: int, scale: float, mix: torch.Tensor,
                    out: Optional[torch.Tensor] = None, out_scale: float = 1.0, nsplit: int = 1,
                    workspace: Optional[Tuple[torch.Tensor, torch.Tensor]] = None,
                    matrix_cores: bool = True) -> torch.Tensor:
    """q [T, H, D] (row b owns tokens cu_q[b]:cu_q[b+1], the LAST positions of its context of ctx_len[b] tokens, whose
    keys / values are in the cache already), mix [H, H]. Writes out_scale * o into `out` ([T, H Dv], a view with unit
    stride along the columns; None: a new tensor) and returns it. nsplit > 1 (single-query rows): the keys of a row are
    shared out over that many workgroups. `matrix_cores` False: always the any-size kernel."""
    T, H, D = q.shape
    G, V = kcache.shape[1], vcache_t.shape[2]
    B = cu_q.numel() - 1
    if out is None:
        out = torch.empty(T, H * V, dtype=q.dtype, device=q.device)
    assert out.shape == (T, H * V) and out.stride(1) == 1 and out.dtype == q.dtype and mix.shape == (H, H)
    if L.use_hip(q):
        assert q.is_contiguous() and kcache.dtype == q.dtype and vcache_t.dtype == q.dtype and mix.dtype == q.dtype
        assert block_tables.dtype == torch.int32 and block_tables.is_contiguous() and mix.is_contiguous()
        assert cu_q.dtype == torch.int32 and ctx_len.dtype == torch.int32 and (nsplit == 1 or max_q == 1)
        prompt_mc, decode_mc = matrix_cores_serve(H, G, D, V, q.dtype, q.device) if matrix_cores else (False, False)
        aligned = out.stride(0) % 4 == 0 and out.data_ptr() % 8 == 0
        decode_mc = decode_mc and max_q == 1
        prompt_mc = prompt_mc and max_q > 1 and nsplit == 1 and aligned
        max_pages = block_tables.shape[1]
        na, nm = workspace_floats(T, nsplit, H, V, max_pages * PAGE_SIZE if decode_mc else 0)
        if workspace is None or workspace[0].numel() < na or workspace[1].numel() < nm:
            workspace = (torch.empty(na, dtype=torch.float32, device=q.device),
                         torch.empty(nm, dtype=torch.float32, device=q.device))
        acc, stats = workspace
        if decode_mc:
            assert T == B
            ns = T * H * max_pages * PAGE_SIZE  # scores first, then the partial sums
            L.check(L.lib().areal_mixed_attn_decode(
                L.ptr(q), L.ptr(kcache), L.ptr(vcache_t), L.ptr(block_tables), L.c_int(max_pages), L.ptr(ctx_len), L.ptr(mix),
                L.ptr(acc), L.ptr(stats), L.ptr(out), L.c_int64(out.stride(0)), L.ptr(acc[ns:]) if nsplit > 1 else None,
                L.c_int(B), L.c_int(H), L.c_int(G), L.c_int(D), L.c_int(V), L.c_float(scale), L.c_float(out_scale),
                L.c_int(int(nsplit)), L.stream_ptr()), "mixed_attn_decode")
            return out
        if prompt_mc:
            L.check(L.lib().areal_mixed_attn_prompt(
                L.ptr(q), L.ptr(kcache), L.ptr(vcache_t), L.ptr(block_tables), L.c_int(max_pages), L.ptr(cu_q),
                L.ptr(ctx_len), L.ptr(mix), L.ptr(stats), L.ptr(out), L.c_int64(out.stride(0)), L.c_int(B),
                L.c_int(int(max_q)), L.c_int(T), L.c_int(H), L.c_int(G), L.c_int(D), L.c_int(V), L.c_float(scale),
                L.c_float(out_scale), L.stream_ptr()), "mixed_attn_prompt")
            return out
        want = 1 if max_q == 1 else 16
        while want > 1 and want // 2 >= max_q:
            want //= 2
        bq = int(L.lib().areal_mixed_attn_tile(L.c_int(H), L.c_int(G), L.c_int(D), L.c_int(V), L.c_int(want)))
        if bq <= 0:
            raise RuntimeError(f"mixed attention: {H} heads of size {D} / {V} do not fit the kernel's tile memory")
        L.check(L.lib().areal_mixed_attn(
            L.ptr(q), L.ptr(kcache), L.ptr(vcache_t), L.ptr(block_tables), L.c_int(max_pages), L.ptr(cu_q),
            L.ptr(ctx_len), L.ptr(mix), L.ptr(stats), L.ptr(out), L.c_int64(out.stride(0)),
            L.ptr(acc) if nsplit > 1 else None, L.c_int(B), L.c_int(int(max_q)), L.c_int(T), L.c_int(H),
            L.c_int(G), L.c_int(D), L.c_int(V), L.c_int(bq), L.c_float(scale), L.c_float(out_scale), L.c_int(int(nsplit)),
            L.c_int(L.dtype_flag(q)), L.stream_ptr()), "mixed_attn")
        return out
    cq, cl = cu_q.tolist(), ctx_len.tolist()
    rep = H // G
    for b in range(B):
        n, ctx = cq[b + 1] - cq[b], cl[b]
        if n == 0:
            continue
        pages = block_tables[b, :(ctx + PAGE_SIZE - 1) // PAGE_SIZE].long()
        kk = kcache[pages].permute(1, 0, 2, 3).reshape(G, -1, D)[:, :ctx].float().repeat_interleave(rep, 0)
        vv = vcache_t[pages].permute(1, 0, 3, 2).reshape(G, -1, V)[:, :ctx].float().repeat_interleave(rep, 0)
        s = torch.matmul(q[cq[b]:cq[b + 1]].float().transpose(0, 1), kk.transpose(1, 2)) * scale
        i = torch.arange(ctx - n, ctx).view(n, 1)
        p = torch.softmax(s.masked_fill(torch.arange(ctx).view(1, -1) > i, float("-inf")), -1)
        w = torch.einsum("hg,gij->hij", mix.float(), p)
        o = torch.matmul(w, vv).transpose(0, 1).reshape(n, H * V) * out_scale
        out[cq[b]:cq[b + 1]] = o.to(out.dtype)
    return out
