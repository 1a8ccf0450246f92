"""Gusolix (layer-list decoder with a layer norm on every sublayer's output and a short convolution ahead of every
sublayer: attention inside chunks of positions with keys as values, selective scan, attention with mixed weights beside
gated linear attention) against the plain float64 formulation in ``gusolix_oracle.py``: every mechanism alone, then the
serving engine - scheduler, paged caches, state slots, prefill and decode plans - on small random models of several
shapes. Every test runs on the CPU formulations of the ops and, marked `gpu`, on the HIP kernels."""
import json
import math
import os
import random
import sys

import pytest
import torch

sys.path.insert(0, os.path.dirname(os.path.abspath(__file__)))
import gusolix_oracle as O  # noqa: E402
from serving_helpers import (F64, PAGE, cut, i32, is32, make_engine, portions_of, rel_err, replay, rows_agree,  # noqa: E402
                             rows_of, seen, slots_of, tokens_of, tol, weights_of)

from areal_vllm_amd.api.cli_args import InferenceServerConfig  # noqa: E402
from areal_vllm_amd.inference.engine import NativeInferenceEngine  # noqa: E402
from areal_vllm_amd.models.config import ModelConfig  # noqa: E402
from areal_vllm_amd.ops import gla as gla_ops  # noqa: E402
from areal_vllm_amd.ops import mamba as mamba_ops  # noqa: E402
from areal_vllm_amd.ops import mixed_attention as xattn  # noqa: E402
from areal_vllm_amd.ops import sandwich as sw  # noqa: E402
from areal_vllm_amd.ops import window_attention as wattn  # noqa: E402

DEVICES = ["cpu", pytest.param("cuda", marks=pytest.mark.gpu)]
CASES = [("cpu", "float32"), pytest.param("cuda", "float32", marks=pytest.mark.gpu),
         pytest.param("cuda", "bfloat16", marks=pytest.mark.gpu)]
OP_CASES = [("cpu", torch.float32), ("cpu", torch.bfloat16),
            pytest.param("cuda", torch.float32, marks=pytest.mark.gpu),
            pytest.param("cuda", torch.bfloat16, marks=pytest.mark.gpu)]


# ------------------------------------------------------------------------------------ mechanisms
def _batch(lengths, device):
    """Packed rows of the given lengths as (cu_q, total)."""
    cu = [0]
    for n in lengths:
        cu.append(cu[-1] + n)
    return i32(cu, device), cu


@pytest.mark.parametrize("device,dtype", OP_CASES)
@pytest.mark.parametrize("W,taps", [(48, 3), (257, 2), (8, 5), (1032, 4), (2048, 3), (20, 1), (4100, 2), (64, 0)])
def test_closing_norm_sum_and_convolved_stream_in_portions(device, dtype, W, taps):
    """x + LN(y) and the convolution of it, three sequences of unequal length cut differently, slots left dirty by others,
    a padding row between them."""
    g = torch.Generator().manual_seed(W)
    lens, eps = [41, 7, 19], 1e-5
    w, b = (1 + 0.2 * torch.randn(W, generator=g)).to(dtype), (0.3 * torch.randn(W, generator=g)).to(dtype)
    cw = (0.5 * torch.randn(W, taps, generator=g)).to(dtype) if taps else None
    xs = [2 * torch.randn(n, W, generator=g) for n in lens]
    ys = [(3 * torch.randn(n, W, generator=g) + 1).to(dtype) for n in lens]
    want_x = [x.to(F64) + O.layer_norm(y.to(F64), w.to(F64), b.to(F64), eps) for x, y in zip(xs, ys)]
    want_h = [O.with_history(x, cw.to(F64)) if taps else x for x in want_x]
    state = torch.full((5, taps - 1, W), 37.0, device=device) if taps > 1 else None
    slot = [4, 0, 2]
    plans = [[41], [1], [2, 1, 3, 17, 1, 9, 2], [5, 6, 1]], [[7], [1], [3, 1, 3], [6, 1]], [[19], [1], [1, 2], [18, 1]]
    for k in range(4):
        cuts = [portions_of(n, p[k]) for n, p in zip(lens, plans)]
        at, got_x, got_h = [0, 0, 0], [[], [], []], [[], [], []]
        while any(a < n for a, n in zip(at, lens)):
            rows, parts_x, parts_y, size = [], [], [], []
            for i in range(3):
                if cuts[i]:
                    c = cuts[i].pop(0)
                    rows.append(i)
                    parts_x.append(xs[i][at[i]:at[i] + c])
                    parts_y.append(ys[i][at[i]:at[i] + c])
                    size.append(c)
            # a padding row of one token at the end
            cu_q, cu = _batch(size + [1], device)
            x = torch.cat(parts_x + [torch.ones(1, W)]).to(device)
            y = torch.cat(parts_y + [torch.ones(1, W).to(dtype)]).to(device)
            first = i32([at[i] for i in rows] + [0], device)
            ss = i32([slot[i] for i in rows] + [-1], device)
            nx, hc = sw.norm_add_conv(x, y, w.to(device), b.to(device), eps, (cw.to(device) if taps else None, state),
                                      cu_q, first, ss)
            assert nx.dtype == torch.float32 and hc.dtype == dtype and torch.isfinite(hc.float()).all()
            for j, i in enumerate(rows):
                got_x[i].append(nx[cu[j]:cu[j + 1]].cpu())
                got_h[i].append(hc[cu[j]:cu[j + 1]].float().cpu())
                at[i] += size[j]
        for i in range(3):
            assert rel_err(torch.cat(got_x[i]), want_x[i]) < 2e-6
            assert rel_err(torch.cat(got_h[i]), want_h[i]) < (3e-6 if is32(dtype) else 1e-2)
    # a decode step: one token a row, the sublayer's output as three fp32 slabs (partial products of a split GEMM)
    if state is not None:
        state[:3] = torch.randn(3, taps - 1, W, generator=g).to(device)
    hist = state[:3].cpu().to(F64) if state is not None else torch.zeros(3, 0, W, dtype=F64)
    x3, sl = torch.randn(3, W, generator=g), torch.randn(3, 3, W, generator=g)
    want3 = x3.to(F64) + O.layer_norm(sl.to(F64).sum(0), w.to(F64), b.to(F64), eps)
    nx, hc = sw.norm_add_conv(x3.clone().to(device), sl.to(device), w.to(device), b.to(device), eps, (cw.to(device) if taps else None, state),
                              i32([0, 1, 2, 3], device), i32([9, 5, 20], device), i32([2, 0, 1], device), 1)
    assert rel_err(nx.cpu(), want3) < (2e-6 if is32(dtype) else 1e-2)
    for j, s in enumerate((2, 0, 1)):
        seq = torch.cat([hist[s], want3[j:j + 1]])
        want = O.with_history(seq, cw.to(F64))[-1:] if taps else want3[j:j + 1]
        assert rel_err(hc[j:j + 1].float().cpu(), want) < (3e-6 if is32(dtype) else 2e-2)
        if taps > 1:
            assert rel_err(state[s].cpu(), seq[1:]) < (3e-6 if is32(dtype) else 2e-2)
    nx, hc = sw.norm_add_conv(x3.clone().to(device), sl.to(device), w.to(device), b.to(device), eps, None, i32([0, 1, 2, 3], device),
                              i32([9, 5, 20], device), i32([2, 0, 1], device), 1)
    assert hc is None and rel_err(nx.cpu(), want3) < (2e-6 if is32(dtype) else 1e-2)
    # without a following sublayer only the sum is formed
    nx, hc = sw.norm_add_conv(xs[0].to(device), ys[0].to(device), w.to(device), b.to(device), eps, None,
                              i32([0, 41], device), i32([0], device), i32([1], device))
    assert hc is None and rel_err(nx.cpu(), want_x[0]) < 2e-6
    if taps > 1:
        assert float(state[3].min()) == 37.0 and float(state[3].max()) == 37.0  # nobody's slot stays as it was


ROTS = [None, {"base": 10000.0, "dims": 8}, {"base": 500.0, "dims": 16},
        {"base": 1000.0, "dims": 16, "scaling": {"factor": 8.0, "low": 1.0, "high": 4.0, "original": 256}},
        {"base": 300.0, "dims": 16, "scaling": {"factor": 2.0, "low": 2.0, "high": 3.0, "original": 64}}]


def test_stretched_frequencies():
    for base, dims, sc in ((500000.0, 64, {"factor": 8.0, "low": 1.0, "high": 4.0, "original": 8192}),
                           (10000.0, 32, {"factor": 3.0, "low": 1.5, "high": 6.0, "original": 512}),
                           (77.0, 6, {"factor": 1.0, "low": 1.0, "high": 4.0, "original": 64}), (100.0, 2, None)):
        f, m = wattn.rotation_frequencies(base, dims, sc)
        want = torch.tensor(O.frequencies(base, dims, sc), dtype=F64)
        assert m == 1.0 and torch.allclose(f, want, rtol=1e-12, atol=0)
        if sc and sc["original"] == 8192:  # all three ranges of wavelengths occur
            plain = torch.tensor(O.frequencies(base, dims, None), dtype=F64)
            r = want / plain
            assert (r == 1).any() and (r == 1 / 8.0).any() and ((r > 0.126) & (r < 0.999)).any()


@pytest.mark.parametrize("device,dtype", OP_CASES)
@pytest.mark.parametrize("H,G,D,V,keyv", [(4, 2, 16, 16, True), (4, 2, 16, 8, False), (3, 1, 18, 18, True), (2, 2, 20, 5, False),
                                          (5, 1, 80, 80, True), (8, 2, 128, 128, True), (1, 1, 16, 16, True)])
@pytest.mark.parametrize("transposed", [False, True])
def test_norm_over_all_heads_rotated_halves_and_cache_write(device, dtype, H, G, D, V, keyv, transposed):
    g = torch.Generator().manual_seed(H + D)
    T, lead, eps = 6, 8, 1e-5
    v_off = H * D if keyv else (H + G) * D
    wide = (2 * torch.randn(T, lead + max((H + G) * D, v_off + G * V) + 16, generator=g)).to(dtype)
    wide[:, lead:lead + D] *= 5  # one head outweighs the others: a norm per head would show
    qw, kw = (1 + 0.3 * torch.randn(H * D, generator=g)).to(dtype), (1 + 0.3 * torch.randn(G * D, generator=g)).to(dtype)
    pos = torch.tensor([0, 1, 5, 63, 200, 299], dtype=torch.int32)
    slots = torch.tensor([33, 34, -1, 64, 2, 95], dtype=torch.int64)
    src = wide[:, lead:].to(F64)
    for rot in ROTS:
        if rot and rot["dims"] > D:
            continue
        kc = torch.full((4, G, PAGE, D), 9.0, dtype=dtype, device=device)
        vc = torch.full((4, G, V, PAGE) if transposed else (4, G, PAGE, V), -9.0, dtype=dtype, device=device)
        table = wattn.rotation_table(rot["base"], rot["dims"], 300, device, rot.get("scaling")) if rot else None
        q = wattn.qk_rows_norm_cache_write(wide.to(device)[:, lead:], v_off, qw.to(device), kw.to(device),
                                           pos.to(device) if rot else None, table, slots.to(device), kc, vc, H, eps,
                                           v_transposed=transposed)
        wq = O.rms_norm(src[:, :H * D], qw.to(F64), eps).view(T, H, D)
        wk = O.rms_norm(src[:, H * D:(H + G) * D], kw.to(F64), eps).view(T, G, D)
        if rot:
            wq, wk = O.rotate_half(wq, pos, rot), O.rotate_half(wk, pos, rot)
        assert rel_err(q.float().cpu().reshape(T, -1), wq.reshape(T, -1)) < (1e-5 if is32(dtype) else 1e-2)
        for t, s in enumerate(slots.tolist()):
            if s < 0:
                continue
            pg, off = s // PAGE, s % PAGE
            assert rel_err(kc[pg, :, off].float().cpu().reshape(1, -1), wk[t].reshape(1, -1)) < (1e-5 if is32(dtype) else 1e-2)
            v = vc[pg, :, :, off] if transposed else vc[pg, :, off]
            assert torch.equal(v.cpu().to(F64).reshape(-1), src[t, v_off:v_off + G * V])  # as projected, untouched
        assert float(kc[3].float().min()) == 9.0
        other = vc[1, :, :, 3:] if transposed else vc[1, :, 3:]
        assert float(other.float().max()) == -9.0  # nothing else is touched


def _chunk_case(H, G, D, scale, chunk, n, probe, seed):
    """Queries and raw keys of one sequence as the columns of an identity-like projection. `probe` = (query position, key
    position): that key's score for that query stands out, so a key on the wrong side of a chunk's edge shows."""
    g = torch.Generator().manual_seed(seed)
    width = (H + G) * D
    h = torch.randn(n, width, generator=g)
    if probe is not None:
        qi, kj = probe
        for c in range(G):
            h[kj, H * D + c * D:H * D + (c + 1) * D] = 3.0 * h[qi, c * (H // G) * D:c * (H // G) * D + D]
    eye = torch.eye(width, dtype=F64)
    w = {"q": eye[:H * D], "k": eye[H * D:], "o": torch.eye(H * D, dtype=F64), "q.norm": torch.ones(H * D, dtype=F64),
         "k.norm": 1 + 0.1 * torch.randn(G * D, generator=g, dtype=F64)}
    m = {"heads": H, "kv_heads": G, "dim": D, "scale": scale, "mask": {"size": chunk}, "rot": None}
    return h, w, m


def _run_chunked(h, w, m, dtype, device, portions, pages, nsplit=1, matrix_cores=True, standard=False):
    from areal_vllm_amd.ops.attention import alloc_kv_cache

    H, G, D = m["heads"], m["kv_heads"], m["dim"]
    n = h.shape[0]
    alloc = alloc_kv_cache if standard else lambda p, c, d, t, dev: wattn.alloc_window_cache(p, c, d, d, t, dev)
    kc, vc = alloc(max(pages) + 2, G, D, dtype, device)
    kc.fill_(50.0)  # what an earlier request left behind
    vc.fill_(-50.0)
    shape = wattn.ScoreShape(scale=m["scale"], chunk=m["mask"]["size"])
    bt = torch.tensor([pages], dtype=torch.int32, device=device)
    qw, kw = w["q.norm"].to(dtype).to(device), w["k.norm"].to(dtype).to(device)
    outs, at, hd = [], 0, h.to(dtype).to(device)
    for c in portions_of(n, portions):
        q = wattn.qk_rows_norm_cache_write(hd[at:at + c], H * D, qw, kw, None, None, slots_of(pages, at, at + c, device), kc,
                                           vc, H, 1e-6, v_transposed=standard)
        args = (q, kc, vc, bt, i32([0, c], device))
        if standard:
            o = wattn.window_attention_standard(*args, i32([0, at + c], device), i32([at + c], device), c, shape,
                                                nsplit=nsplit if c == 1 else 1)
        else:
            o = wattn.window_attention(*args, i32([at + c], device), c, shape, None, nsplit=nsplit if c == 1 else 1,
                                       matrix_cores=matrix_cores)
        outs.append(o.reshape(c, H * D).float().cpu())
        at += c
    return torch.cat(outs)


def _check_chunks(H, G, D, chunk, device, dtype, standard=False, n=150):
    pages = [3, 1, 4, 9, 2, 7][:(n + PAGE - 1) // PAGE]
    probes = set()
    for qi in (n - 1, 100, 97, 64, 63, 33, 32, 31, chunk, 2 * chunk, 2 * chunk - 1):
        if qi >= n:
            continue
        start = qi // chunk * chunk
        # the chunk's first key and the one before it, the key itself, page borders, the sequence's first key
        probes |= {(qi, k) for k in (start, start - 1, qi, qi - 1, qi - 32, qi // 32 * 32, qi // 32 * 32 - 1, 0) if 0 <= k <= qi}
    for k, (qi, kj) in enumerate(sorted(probes)):
        h, w, m = _chunk_case(H, G, D, 12.0 / math.sqrt(D), chunk, n, (qi, kj), 7 + k % 3)
        ws = dict(w, **{"k.norm": seen(w["k.norm"], dtype)})
        want = O.chunked_attention(seen(h, dtype)[:qi + 1], ws, "", m, 1e-6)[qi:qi + 1]
        for portions, nsplit in (([n], 1), ([qi or 1, 1, n], 1 + 2 * (k % 2)), ([max(qi - 1, 1), 2, n], 1)):
            got = _run_chunked(h, w, m, dtype, device, portions, pages, nsplit, standard=standard)
            assert rel_err(got[qi:qi + 1], want) < tol(dtype), (qi, kj, portions, nsplit)
    h, w, m = _chunk_case(H, G, D, 1.0 / math.sqrt(D), chunk, n, None, 1)
    ws = dict(w, **{"k.norm": seen(w["k.norm"], dtype)})
    want = O.chunked_attention(seen(h, dtype), ws, "", m, 1e-6)
    for portions, mc in (([n], True), ([n], False), ([1], True), ([2], True), ([3, 17, 1, 1, 64, 31, 2, 33], True),
                         ([70, 1], True)):
        if standard and not mc:
            continue
        got = _run_chunked(h, w, m, dtype, device, portions, pages, 2, mc, standard)
        assert rel_err(got, want) < tol(dtype), (portions, mc)


@pytest.mark.parametrize("device,dtype", OP_CASES)
@pytest.mark.parametrize("H,G,D,chunk", [(4, 2, 16, 37), (2, 1, 8, 32), (3, 3, 12, 5), (1, 1, 16, 64), (2, 2, 8, 1),
                                         (4, 1, 64, 48), (6, 2, 128, 41), (2, 1, 10, 1000)])
def test_chunk_edges_pages_portions_and_splits(device, dtype, H, G, D, chunk):
    _check_chunks(H, G, D, chunk, device, dtype)


@pytest.mark.gpu
@pytest.mark.parametrize("H,G,chunk", [(4, 2, 70), (2, 1, 64), (4, 4, 33), (16, 1, 128), (3, 1, 1), (2, 2, 1000)])
def test_chunks_in_the_standard_cache_layout(H, G, chunk):
    """bf16 heads of 128 live in the engine's standard cache and run its paged flash and paged decode kernels."""
    _check_chunks(H, G, 128, chunk, "cuda", torch.bfloat16, standard=True, n=190)


def _mixed_case(H, G, D, V, scale, n, probes, seed):
    """`probes`: (head, query position, key position): the key answers that head's query so that its score stands out; what
    the mixing does with it shows in every head's output."""
    g = torch.Generator().manual_seed(seed)
    width = (H + G) * D + G * V
    h = torch.randn(n, width, generator=g)
    for hd, qi, kj in probes:
        c = hd // (H // G)
        h[kj, H * D + c * D:H * D + (c + 1) * D] = 3.0 * h[qi, hd * D:(hd + 1) * D]
    eye = torch.eye(width, dtype=F64)
    a, b = H * D, (H + G) * D
    w = {"q": eye[:a], "k": eye[a:b], "v": eye[b:], "o": torch.eye(H * V, dtype=F64), "q.norm": torch.ones(a, dtype=F64),
         "k.norm": torch.ones(G * D, dtype=F64),
         "talk": torch.eye(H, dtype=F64) + 0.7 * torch.randn(H, H, generator=g, dtype=F64)}
    return h, w, {"heads": H, "kv_heads": G, "dim": D, "vdim": V, "scale": scale}


def _run_mixed(h, w, m, dtype, device, portions, pages, nsplit=1, matrix_cores=True):
    H, G, D, V = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    n = h.shape[0]
    kc, vc = xattn.alloc_mixed_cache(max(pages) + 2, G, D, V, dtype, device)
    kc.fill_(50.0)
    vc.fill_(-50.0)
    bt = torch.tensor([pages], dtype=torch.int32, device=device)
    ones = [torch.ones(k * D, dtype=dtype, device=device) for k in (H, G)]
    mix = w["talk"].to(dtype).to(device)
    outs, at, hd = [], 0, h.to(dtype).to(device)
    for c in portions_of(n, portions):
        q = wattn.qk_rows_norm_cache_write(hd[at:at + c], (H + G) * D, *ones, None, None, slots_of(pages, at, at + c, device),
                                           kc, vc, H, 1e-6, v_transposed=True)
        wide = torch.full((c, H * V + 24), 3.0, dtype=dtype, device=device)  # the outputs are columns of wider rows
        o = xattn.mixed_attention(q, kc, vc, bt, i32([0, c], device), i32([at + c], device), c, m["scale"], mix,
                                  wide[:, 16:16 + H * V], 0.5, nsplit if c == 1 else 1, matrix_cores=matrix_cores)
        assert float(wide[:, :16].float().min()) == 3.0 and float(wide[:, 16 + H * V:].float().max()) == 3.0
        outs.append(2.0 * o.float().cpu())
        at += c
    return torch.cat(outs)


@pytest.mark.parametrize("device,dtype", OP_CASES)
@pytest.mark.parametrize("H,G,D,V", [(4, 2, 16, 8), (3, 3, 12, 20), (1, 1, 16, 4), (6, 2, 20, 12), (8, 2, 64, 64), (4, 4, 128, 128),
                                     (16, 4, 128, 128), (4, 2, 64, 128), (5, 1, 64, 64), (8, 8, 32, 32), (12, 3, 96, 64)])
def test_mixed_weights_far_keys_page_borders_portions_and_splits(device, dtype, H, G, D, V):
    n, pages = 140, [3, 1, 4, 9, 2]
    probes = [(hd % H, qi, kj) for hd, qi, kj in ((0, 139, 0), (1, 139, 1), (2, 138, 31), (3, 131, 32), (0, 100, 63), (1, 97, 64),
                                                  (2, 96, 95), (0, 64, 64), (3, 63, 2), (1, 33, 0), (0, 32, 31), (0, 1, 0))]
    for k, (hd, qi, kj) in enumerate(probes):
        h, w, m = _mixed_case(H, G, D, V, 12.0 / math.sqrt(D), n, [(hd, qi, kj)], 5 + k % 3)
        ws = dict(w, talk=seen(w["talk"], dtype))
        want = O.mixed_attention(seen(h, dtype)[:qi + 1], ws, "", m, 1e-6)[qi:qi + 1]
        for portions, nsplit in (([n], 1), ([qi, 1, n], 1 + 2 * (k % 2)), ([max(qi - 1, 1), 2, n], 1)):
            got = _run_mixed(h, w, m, dtype, device, portions, pages, nsplit)
            assert rel_err(got[qi:qi + 1], want) < tol(dtype), (hd, qi, kj, portions, nsplit)
    h, w, m = _mixed_case(H, G, D, V, 2.0 / math.sqrt(D), n, [], 1)
    ws = dict(w, talk=seen(w["talk"], dtype))
    want = O.mixed_attention(seen(h, dtype), ws, "", m, 1e-6)
    for portions, nsplit, mc in (([n], 1, True), ([n], 1, False), ([1], 2, True), ([1], 1, False), ([2], 1, True),
                                 ([3, 17, 1, 1, 64, 31, 2, 33], 5, True), ([70, 1], 3, True)):
        got = _run_mixed(h, w, m, dtype, device, portions, pages, nsplit, mc)
        assert rel_err(got, want) < tol(dtype), (portions, nsplit, mc)
    if H > 1:  # mixing scores instead of weights, or not at all, is something else by far
        plain = dict(ws, talk=torch.eye(H, dtype=F64))
        assert rel_err(O.mixed_attention(seen(h, dtype), plain, "", m, 1e-6), want) > 0.3


@pytest.mark.parametrize("device,dtype", OP_CASES)
@pytest.mark.parametrize("H,G,D,V", [(4, 2, 16, 8), (16, 4, 128, 128), (8, 2, 64, 64)])
def test_mixed_weights_of_unequal_rows_in_one_batch(device, dtype, H, G, D, V):
    """Rows of a prefill batch and of a decode batch with very different contexts, pages in any order, a retired row."""
    cases = [_mixed_case(H, G, D, V, 2.0 / math.sqrt(D), n, [], 20 + n) for n in (1, 130, 33, 64)]
    mixw, m = cases[0][1], cases[0][2]
    pages = [[11], [3, 1, 4, 9, 2], [7, 5], [6, 8]]
    kc, vc = xattn.alloc_mixed_cache(13, G, D, V, dtype, device)
    bt = torch.zeros(5, 5, dtype=torch.int32)
    for i, p in enumerate(pages):
        bt[i, :len(p)] = torch.tensor(p)
    bt = bt.to(device)
    ones = [torch.ones(k * D, dtype=dtype, device=device) for k in (H, G)]
    mix = mixw["talk"].to(dtype).to(device)
    ws = dict(mixw, talk=seen(mixw["talk"], dtype))
    want = [O.mixed_attention(seen(h, dtype), dict(w, talk=ws["talk"]), "", m, 1e-6) for h, w, _ in cases]
    qs = []
    for (h, _, _), p in zip(cases, pages):
        qs.append(wattn.qk_rows_norm_cache_write(h.to(dtype).to(device), (H + G) * D, *ones, None, None,
                                                 slots_of(p, 0, h.shape[0], device), kc, vc, H, 1e-6, v_transposed=True))
    tails = [1, 40, 2, 64]  # the last tokens of every row as one prefill batch
    q = torch.cat([x[-t:] for x, t in zip(qs, tails)])
    cu_q, cu = _batch(tails, device)
    ctx = i32([x.shape[0] for x in qs], device)
    o = xattn.mixed_attention(q, kc, vc, bt[:4].contiguous(), cu_q, ctx, 64, m["scale"], mix)
    for i, t in enumerate(tails):
        assert rel_err(o[cu[i]:cu[i + 1]].float().cpu(), want[i][-t:]) < tol(dtype)
    q = torch.cat([x[-1:] for x in qs] + [qs[0][-1:]])  # and one token each, with a retired row
    cu_q, _ = _batch([1] * 5, device)
    for ns in (1, 4):
        o = xattn.mixed_attention(q, kc, vc, bt, cu_q, i32([x.shape[0] for x in qs] + [1], device), 1, m["scale"], mix, nsplit=ns)
        for i in range(4):
            assert rel_err(o[i:i + 1].float().cpu(), want[i][-1:]) < tol(dtype)
        assert torch.isfinite(o.float()).all()


@pytest.mark.parametrize("device,dtype", OP_CASES)
@pytest.mark.parametrize("I,N,R,taps", [(24, 5, 3, 4), (64, 16, 8, 2), (130, 1, 1, 1), (88, 22, 7, 4), (70, 33, 2, 5), (32, 130, 4, 3)])
def test_short_convolution_and_selective_scan(device, dtype, I, N, R, taps):
    """Three sequences in one batch, cut in several ways, dirty slots, a padding row."""
    g = torch.Generator().manual_seed(I + N)
    lens, slot = [57, 3, 20], [3, 1, 0]
    cw, cb = torch.randn(I, taps, generator=g).to(dtype), (0.3 * torch.randn(I, generator=g)).to(dtype)
    dtw, dtb = (torch.randn(I, R, generator=g) / R ** 0.5).to(dtype), (-2 + torch.randn(I, generator=g)).to(dtype)
    al, dsk = torch.log(0.2 + 3 * torch.rand(I, N, generator=g)).to(dtype), torch.randn(I, generator=g).to(dtype)
    xzs = [(1.5 * torch.randn(n, 2 * I + 3, generator=g)).to(dtype) for n in lens]
    lows = [(torch.randn(n, R + 2 * N, generator=g)).to(dtype) for n in lens]
    wx, wy = [], []
    for xz, low in zip(xzs, lows):
        x = O.silu(O.causal_conv(xz[:, :I].to(F64), cw.to(F64)) + cb.to(F64))
        wx.append(x)
        xs, lo = seen(x.float(), dtype), low.to(F64)
        y = O.selective_scan(xs, O.softplus(lo[:, :R] @ dtw.to(F64).T + dtb.to(F64)), -torch.exp(al.to(F64)), lo[:, R:R + N],
                             lo[:, R + N:], dsk.to(F64))
        wy.append(y * O.silu(xz[:, I:2 * I].to(F64)))
    S = mamba_ops.alloc_state(5, I, N, device).fill_(11.0)
    hist = torch.full((5, taps - 1, I), -7.0, device=device) if taps > 1 else None
    dev = [t.to(device) for t in (cw, cb, dtw, dtb, al, dsk)]
    for plan in ([[57], [3], [20]], [[1], [1], [1]], [[2, 1, 30, 7, 1, 1, 15], [2, 1], [17, 3]], [[40, 16, 1], [1, 2], [4]]):
        cuts = [portions_of(n, p) for n, p in zip(lens, plan)]
        at, gx, gy = [0, 0, 0], [[], [], []], [[], [], []]
        while any(cuts):
            rows = [i for i in range(3) if cuts[i]]
            size = [cuts[i].pop(0) for i in rows]
            cu_q, cu = _batch(size + [1], device)
            xz = torch.cat([xzs[i][at[i]:at[i] + c] for i, c in zip(rows, size)] + [xzs[0][:1]]).to(device)
            low = torch.cat([lows[i][at[i]:at[i] + c] for i, c in zip(rows, size)] + [lows[0][:1]]).to(device)
            first, ss = i32([at[i] for i in rows] + [0], device), i32([slot[i] for i in rows] + [-1], device)
            x = sw.conv_silu(xz[:, :I], dev[0], dev[1], hist, cu_q, first, ss)
            r = torch.nn.functional.linear(low[:, :R].float(), dev[2].float())
            y = mamba_ops.selective_scan(x, r, dev[3], dev[4], low[:, R:], dev[5], xz[:, I:2 * I], cu_q, first, ss, S,
                                         max_q=max(size))
            for j, i in enumerate(rows):
                gx[i].append(x[cu[j]:cu[j + 1]].float().cpu())
                gy[i].append(y[cu[j]:cu[j + 1]].float().cpu())
                at[i] += size[j]
        for i in range(3):
            assert rel_err(torch.cat(gx[i]), wx[i]) < (1e-5 if is32(dtype) else 1e-2), plan
            assert rel_err(torch.cat(gy[i]), wy[i]) < (tol(dtype) if is32(dtype) else 2e-2), plan
    assert float(S[2].min()) == 11.0 and float(S[4].max()) == 11.0


@pytest.mark.parametrize("device,dtype", OP_CASES)
def test_gated_linear_readout_into_columns_with_a_factor(device, dtype):
    g = torch.Generator().manual_seed(8)
    T, H, V = 5, 3, 20
    o, gate, w = torch.randn(T, H, V, generator=g), torch.randn(T, H * V, generator=g).to(dtype), torch.randn(V, generator=g).to(dtype)
    wide = torch.full((T, H * V + 9), 2.0, dtype=dtype, device=device)
    y = gla_ops.gla_out(o.to(device), gate.to(device), w.to(device), 1e-5, wide[:, 4:4 + H * V], 0.37)
    want = 0.37 * O.rms_norm(o.to(F64), w.to(F64), 1e-5).reshape(T, -1) * O.silu(gate.to(F64))
    assert y.data_ptr() == wide[:, 4:].data_ptr() and rel_err(y.float().cpu(), want) < (1e-5 if is32(dtype) else 1e-2)
    assert float(wide[:, :4].float().min()) == 2.0 and float(wide[:, 4 + H * V:].float().max()) == 2.0


# ------------------------------------------------------------------------------------ the model in the engine
def attn(heads=4, kv=2, dim=16, chunk=37, rdims=None, base=1000.0, scaling=None, scale=0.4, mlp=40):
    return {"type": "attention", "mlp": {"kind": "dense", "ff": mlp} if mlp else None,
            "mixer": {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": dim, "scale": scale, "mask": {"size": chunk},
                      "rot": {"base": base, "dims": rdims or dim, "scaling": scaling or
                              {"factor": 4.0, "low": 1.0, "high": 4.0, "original": 128}}}}


def mamba(inner=40, state=6, rank=3, conv=4, mlp=None):
    return {"type": "mamba1", "mlp": {"kind": "dense", "ff": mlp} if mlp else None,
            "mixer": {"conv": conv, "dt_rank": rank, "inner": inner, "state": state}}


def side(heads=4, kv=2, dim=12, vdim=20, scale=0.5, gh=3, gd=16, gv=24, tau=8.0, rank=5, ls=0.7, rs=1.2, mlp=None):
    return {"type": "parallel", "mlp": {"kind": "dense", "ff": mlp} if mlp else None,
            "mixer": {"left": {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim, "scale": scale},
                      "right": {"heads": gh, "dim": gd, "vdim": gv, "tau": tau, "decay_rank": rank},
                      "left_scale": ls, "right_scale": rs}}


def config(layers, width=48, vocab=101, eps=1e-5, taps=3, scale=5.0):
    return {"architecture": "Gusolix", "canon": {"taps": taps}, "embedding": {"scale": scale}, "layers": layers,
            "norm": {"eps": eps}, "vocab": vocab, "width": width}


MIXED = config([attn(), side(mlp=56), mamba(mlp=24), attn(heads=2, kv=2, dim=10, chunk=5, rdims=6, mlp=None),
                side(heads=3, kv=3, gh=1, rank=1), mamba(inner=20, state=17, rank=7, conv=2)], taps=4)
_WANT = {}


def check(got, tokens, weights, cfg, dtype, rid, key=None):
    if key is None or key not in _WANT:
        want, _ = O.forward(cfg, weights, tokens)
        if key is not None:
            _WANT[key] = want
    else:
        want = _WANT[key]
    rows = rows_of(got, rid, len(tokens))
    assert rows_agree(rows, want, dtype), rel_err(rows, want)


@pytest.mark.parametrize("device,dtype", CASES)
def test_whole_prompt_and_every_layer(device, dtype):
    eng, w = make_engine(MIXED, device, dtype)
    try:
        toks = tokens_of(75, MIXED["vocab"], 1)
        eng.runner.layer_trace = []
        got = replay(eng, cut("a", toks, [len(toks)]))
        trace, eng.runner.layer_trace = eng.runner.layer_trace, None
        want, layers = O.forward(MIXED, w, toks)
        assert len(trace) == len(layers) == 6
        for a, b in zip(trace, layers):
            assert rows_agree(a.cpu(), b, dtype)
        assert rows_agree(rows_of(got, "a", len(toks)), want, dtype)
    finally:
        eng.destroy()


@pytest.mark.parametrize("device,dtype", CASES)
def test_prefill_against_token_by_token_and_portions(device, dtype):
    eng, w = make_engine(MIXED, device, dtype)
    try:
        toks = tokens_of(140, MIXED["vocab"], 2)
        for k, sizes in enumerate(([1], [60, 1], [2], [3, 64, 2, 31, 33, 1, 1, 5], [1, 32, 32, 32, 1], [17, 16])):
            got = replay(eng, cut(f"r{k}", toks, list(sizes)))
            check(got, toks, w, MIXED, dtype, f"r{k}", key=("portions", device, dtype))
        assert eng.sched.num_free_state_slots() == 4 and eng.sched.num_free_pages() == eng.sched.num_total_pages()
    finally:
        eng.destroy()


@pytest.mark.parametrize("device,dtype", CASES)
def test_unequal_requests_in_one_batch_with_pages_and_slots_used_again(device, dtype):
    """Seven requests of very different lengths through three slots and a pool that cannot hold them all at once:
    portions of some beside single tokens of others; each must equal the request computed alone."""
    eng, w = make_engine(MIXED, device, dtype, num_pages=15, max_running=3)
    try:
        V = MIXED["vocab"]
        reqs = {f"q{i}": tokens_of(n, V, 10 + i) for i, n in enumerate((1, 70, 23, 130, 2, 97, 40))}
        plan = {"q0": [1], "q1": [5, 1, 1, 33, 2, 1], "q2": [23], "q3": [64, 2, 1, 1, 40, 1], "q4": [1, 1], "q5": [31, 33, 1],
                "q6": [2, 1]}
        left = {r: portions_of(len(reqs[r]), plan[r]) for r in reqs}
        waiting, live, at, steps = list(reqs), [], {r: 0 for r in reqs}, []
        while waiting or live:
            while waiting and len(live) < 3 and sum((len(reqs[r]) + 31) // 32 for r in live + waiting[:1]) <= 13:
                live.append(waiting.pop(0))
            step = []
            for r in list(live):
                c = left[r].pop(0)
                step.append((r, reqs[r][at[r]:at[r] + c], list(range(c)), not left[r]))
                at[r] += c
                if not left[r]:
                    live.remove(r)
            steps.append(step)
        assert max(len(s) for s in steps) == 3 and any(len(t) == 1 for s in steps if len(s) > 1 for _, t, _, _ in s)
        got = replay(eng, steps)
        for r, toks in reqs.items():
            check(got, toks, w, MIXED, dtype, r)
        assert eng.sched.num_free_state_slots() == 3 and eng.sched.num_free_pages() == eng.sched.num_total_pages()
    finally:
        eng.destroy()


SHAPES = [
    # one head everywhere, equal sizes everywhere, factors and a temperature of 1: values that hide mix-ups
    config([attn(1, 1, 16, 33, mlp=16), side(1, 1, 16, 16, 0.25, 1, 16, 16, 1.0, 16, 1.0, 1.0, mlp=16), mamba(16, 16, 16, 2)],
           width=16, taps=2, scale=1.0),
    # sizes that are no multiples of 8 or of each other, a chunk of one token and one beyond the sequence
    config([side(6, 3, 10, 20, 0.9, 5, 12, 20, 3.0, 3, 0.3, 2.0, mlp=30), attn(6, 3, 12, 1, 4, 50.0, scale=0.11),
            attn(6, 2, 20, 500, 10, 1e6, {"factor": 32.0, "low": 2.0, "high": 8.0, "original": 64}, 0.9, None),
            mamba(30, 11, 2, 3, mlp=20)], width=40, vocab=67, eps=1e-3, taps=5),
    config([mamba(24, 4, 1, 1)], width=24, taps=1),  # one layer, no paged cache at all, taps of one token
    config([side(2, 1, 8, 8, 1.0, 2, 8, 8, 16.0, 2)], width=24, taps=6),
    # nothing a multiple of 4: width, head sizes, feed-forward widths, vocabulary
    config([attn(3, 1, 10, 13, 6, mlp=9), side(3, 1, 6, 14, 0.6, 7, 6, 5, 5.0, 3, mlp=11), mamba(25, 3, 5, 3), attn(3, 1, 6, 3)],
           width=50, vocab=59),
    # sizes the matrix-core paths take
    config([attn(4, 2, 64, 40, mlp=64), side(4, 2, 64, 64, 0.2, 2, 64, 64, 16.0, 16, mlp=128), attn(8, 2, 128, 70, 64, scale=0.1),
            side(8, 2, 128, 128, 0.1, 1, 128, 128, 4.0, 8), mamba(128, 16, 8, 4, mlp=64),
            side(16, 4, 128, 128, 0.1, 2, 128, 64, 4.0, 8)], width=64),
]


@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("which", range(len(SHAPES)))
def test_other_sizes_chunks_constants_and_orders(device, dtype, which):
    cfg = SHAPES[which]
    eng, w = make_engine(cfg, device, dtype)
    try:
        toks = tokens_of(90, cfg["vocab"], 20 + which)
        key = ("shapes", which, device, dtype)
        check(replay(eng, cut("w", toks, [len(toks)])), toks, w, cfg, dtype, "w", key=key)
        check(replay(eng, cut("c", toks, [7, 2, 33, 1, 1, 20, 1])), toks, w, cfg, dtype, "c", key=key)
    finally:
        eng.destroy()


@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("seed", [1, 2, 3])
def test_random_shapes_orders_and_schedules(device, dtype, seed):
    """Random layer lists (mixer kinds and sizes, chunks, constants, with and without feed-forward) fed through random
    schedules of up to three live requests: portions of 1 .. 100 tokens, requests that skip steps."""
    rng = random.Random(seed)
    for case in range(2):
        width, vocab, layers = rng.choice([32, 48, 72]), rng.choice([37, 101]), []
        for _ in range(rng.randint(1, 4)):
            ff, kv = rng.choice([8, 20, 64, None]), rng.choice([1, 2, 3])
            kind, dim = rng.choice(["attention", "mamba1", "parallel"]), rng.choice([8, 12, 64, 128])
            if kind == "attention":
                layers.append(attn(kv * rng.choice([1, 2, 4]), kv, dim, rng.choice([1, 2, 31, 32, 33, 100, 400]), rng.choice([4, dim]),
                                   rng.choice([100.0, 1e6]), None, rng.choice([0.1, 0.3]), ff))
            elif kind == "mamba1":
                layers.append(mamba(rng.choice([16, 72, 130]), rng.choice([1, 8, 16, 40]), rng.choice([1, 4, 9]), rng.choice([1, 2, 4]), ff))
            else:
                layers.append(side(kv * rng.choice([1, 2, 4]), kv, dim, rng.choice([8, 20, 64, 128]), rng.choice([0.1, 0.3]),
                                   rng.choice([1, 2, 3]), rng.choice([8, 24, 64]), rng.choice([8, 40, 72]), rng.choice([1.0, 16.0]),
                                   rng.choice([1, 4, 16]), rng.choice([1.0, 0.2]), rng.choice([1.0, 0.6]), ff))
        cfg = config(layers, width, vocab, rng.choice([1e-5, 1e-6]), rng.choice([1, 2, 4]), rng.choice([1.0, 8.0]))
        reqs = {f"q{i}": tokens_of(rng.choice([1, 2, 17, 97, 150]), vocab, 7 + 100 * case + i) for i in range(rng.randint(1, 3))}
        at, steps = {r: 0 for r in reqs}, []
        while any(at[r] < len(t) for r, t in reqs.items()):
            step = []
            for r, t in reqs.items():
                if at[r] < len(t) and rng.random() > 0.2:
                    c = min(rng.choice([1, 1, 1, 2, 3, 16, 31, 33, 64, 100]), len(t) - at[r])
                    step.append((r, t[at[r]:at[r] + c], list(range(c)), at[r] + c == len(t)))
                    at[r] += c
            if step:
                steps.append(step)
        eng, w = make_engine(cfg, device, dtype, num_pages=24, max_running=3)
        try:
            got = replay(eng, steps)
            for r, t in reqs.items():
                check(got, t, w, cfg, dtype, r)
        finally:
            eng.destroy()


@pytest.mark.parametrize("device,dtype", CASES)
def test_first_tokens_and_long_decoding(device, dtype):
    cfg = config([attn(chunk=40), side(), mamba(mlp=24), attn(heads=2, kv=2, chunk=9, mlp=None)])
    eng, w = make_engine(cfg, device, dtype)
    try:
        for n in (1, 2, 3, 5):
            toks = tokens_of(n, cfg["vocab"], 40 + n)
            check(replay(eng, cut(f"s{n}", toks, [1])), toks, w, cfg, dtype, f"s{n}")
            check(replay(eng, cut(f"w{n}", toks, [n])), toks, w, cfg, dtype, f"w{n}")
        toks = tokens_of(230, cfg["vocab"], 44)  # chunk edges pass over decoded tokens several times
        check(replay(eng, cut("long", toks, [20, 1])), toks, w, cfg, dtype, "long")
    finally:
        eng.destroy()


@pytest.mark.parametrize("device,dtype", CASES)
def test_greedy_generation_through_the_engine(device, dtype):
    """The engine's own entry point: prompts of unequal length generated together, prefill plans, then decode plans
    (captured graphs on the GPU), more requests than request slots."""
    cfg = config([attn(chunk=21), side(mlp=24), mamba(), attn(heads=2, kv=1, chunk=70, mlp=None)], vocab=61)
    eng, w = make_engine(cfg, device, dtype, max_running=3, score=False)
    try:
        prompts = [tokens_of(n, cfg["vocab"], 50 + n) for n in (3, 41, 18, 1, 66)]
        res = eng.generate_blocking(prompts, max_new_tokens=12, greedy=True)
        agree = 0
        for p, r in zip(prompts, res):
            assert r.finish_reason == "length" and len(r.output_tokens) == 12
            want = O.greedy(cfg, w, p, 12 if is32(dtype) else 1)
            if is32(dtype):
                assert r.output_tokens == want
            else:  # a near-tie of two tokens may flip under bf16
                agree += r.output_tokens[0] == want[0]
        assert is32(dtype) or agree >= 4
        assert eng.sched.num_free_state_slots() == 3
    finally:
        eng.destroy()


def saved_model(cfg_dict, path, dtype, seed):
    from areal_vllm_amd.models import build_model

    m = build_model(ModelConfig.from_hf_dict(cfg_dict), dtype=dtype)
    m.flatten()
    m.init_weights(seed=seed)
    m.save_checkpoint(str(path))
    return m


@pytest.mark.parametrize("device", DEVICES)
def test_served_from_a_checkpoint_directory(device, tmp_path):
    """The framework's own path from a directory with config.json and model.safetensors: the model class is chosen by the
    configuration, the rank of the decay projection by a tensor's shape, the weights come through the engine's loader;
    several decode steps per plan."""
    cfg_dict = config([attn(2, 1, 8, 9, mlp=12), side(2, 1, 8, 8, 0.5, 2, 8, 8, 4.0, 3, mlp=20), mamba(24, 4, 2, 3)], width=32, vocab=53)
    w = weights_of(saved_model(cfg_dict, tmp_path, torch.bfloat16, 9))
    with open(tmp_path / "config.json") as f:
        saved = json.load(f)
    for l in saved["layers"]:  # a checkpoint whose configuration does not name the rank
        l["mixer"].get("right", {}).pop("decay_rank", None)
    with open(tmp_path / "config.json", "w") as f:
        json.dump(saved, f)
    srv = InferenceServerConfig(model_path=str(tmp_path), dtype="float32", context_length=128, max_running_requests=2,
                                num_continuous_decode_steps=2)
    eng = NativeInferenceEngine(srv, device=torch.device(device), num_pages=12)
    eng.initialize()
    try:
        prompts = [tokens_of(n, 53, 70 + n) for n in (5, 33, 17)]
        res = eng.generate_blocking(prompts, max_new_tokens=7, greedy=True)
        for p, r in zip(prompts, res):
            assert r.output_tokens == O.greedy(cfg_dict, w, p, 7)
    finally:
        eng.destroy()


def test_trace_runner_replays_steps(tmp_path):
    """The command-line runner: steps from standard input, logits of the wanted places per step, pages and slots given back."""
    import subprocess

    import numpy as np

    cfg_dict = config([attn(2, 1, 8, 9, mlp=12), side(2, 1, 8, 8), mamba(24, 4, 2, 3)], width=32, vocab=53)
    w = weights_of(saved_model(cfg_dict, tmp_path / "m", torch.bfloat16, 5))
    toks = {"a": tokens_of(40, 53, 1), "b": tokens_of(9, 53, 2)}
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": toks["a"][:33], "want": [0, 32]}], "end": []},
             {"step": 1, "entries": [{"id": "a", "tokens": toks["a"][33:34], "want": []}, {"id": "b", "tokens": toks["b"], "want": [8]}],
              "end": ["b"]},
             {"step": 2, "entries": [{"id": "a", "tokens": toks["a"][34:], "want": [5]}], "end": ["a"]}]
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    r = subprocess.run([sys.executable, os.path.join(root, "bin", "trace_run"), "--model", str(tmp_path / "m"), "--dtype", "float32",
                        "--out", str(tmp_path / "out"), "--max-tokens", "128", "--device", "cpu"],
                       input="".join(json.dumps(s) + "\n" for s in steps), capture_output=True, text=True, timeout=240)
    assert r.returncode == 0, r.stderr[-2000:]
    assert [l for l in r.stdout.splitlines() if l.startswith("done")] == ["done 0", "done 1", "done 2"]
    la, lb = O.forward(cfg_dict, w, toks["a"])[0], O.forward(cfg_dict, w, toks["b"])[0]
    for n, want in ((0, la[[0, 32]]), (1, lb[[8]]), (2, la[[39]])):
        got = torch.from_numpy(np.fromfile(tmp_path / "out" / f"{n}.f32", "<f4")).view(-1, 53)
        assert rows_agree(got, want, "float32")


def test_config_reader_and_checkpoint_save_then_load(tmp_path):
    cfg = ModelConfig.from_hf_dict(SHAPES[1])
    assert cfg.family == "gusolix" and cfg.n_layers == 4 and cfg.has_recurrent_state and not cfg.tie_word_embeddings
    assert cfg.canon_taps == 5 and cfg.rms_norm_eps == 1e-3 and cfg.embed_scale == 5.0
    from areal_vllm_amd.models import build_model

    m = saved_model(SHAPES[1], tmp_path, torch.float32, 4)
    assert sum(p.numel() for p in m.parameters()) == cfg.n_params()
    cfg2 = ModelConfig.from_pretrained(str(tmp_path))
    assert cfg2.layers == cfg.layers and cfg2.canon_taps == cfg.canon_taps
    m2 = build_model(cfg2, dtype=torch.float32)
    m2.flatten()
    m2.load_checkpoint(str(tmp_path))
    for (n1, a), (n2, b) in zip(m.checkpoint_tensors().items(), m2.checkpoint_tensors().items()):
        assert n1 == n2 and torch.equal(a, b)
    extra = dict(m2.checkpoint_tensors(), **{"l0.norm3": torch.zeros(40)})
    with pytest.raises(KeyError):
        m2.assign_named_tensors(extra)
    no_ff = [i for i, l in enumerate(cfg.layers) if l["mlp"] is None][0]  # what a missing feed-forward would own is not read
    m2.assign_named_tensors({f"l{no_ff}.norm2": torch.zeros(40), f"l{no_ff}.canon2": torch.zeros(40, 5)})
    bad = side()
    del bad["mixer"]["right"]["decay_rank"]
    for l in (dict(attn(), type="conv"), attn(rdims=3), attn(heads=3, kv=2), bad, dict(mamba(), mlp={"kind": "moe"})):
        with pytest.raises(ValueError):
            ModelConfig.from_hf_dict(config([l]))
