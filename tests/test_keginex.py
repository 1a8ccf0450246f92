"""Keginex (layer-list decoder with an element-wise tanh norm before and after every sublayer: gated delta rule with a decay
per head and key channel, latent attention without positions and with a sink, routed experts whose choice a learned
correction moves, a span of layers run several times) against the plain float64 formulation in ``keginex_oracle.py``:
every mechanism alone, then the serving engine - scheduler, paged caches, state slots, prefill and decode plans - on small
random models of several shapes. Every test runs on the CPU formulations of the ops and, marked `gpu`, on the HIP kernels."""
import json
import math
import os
import random
import sys

import pytest
import torch

sys.path.insert(0, os.path.dirname(os.path.abspath(__file__)))
import keginex_oracle as O  # noqa: E402
from serving_helpers import (F64, PAGE, cut, i32, is32, make_engine, portions_of, rel_err, replay, rows_agree,  # noqa: E402
                             rows_of, seen, slots_of, tokens_of, tol, weights_of)

from areal_vllm_amd.api.cli_args import InferenceServerConfig  # noqa: E402
from areal_vllm_amd.inference.engine import NativeInferenceEngine  # noqa: E402
from areal_vllm_amd.models.config import ModelConfig  # noqa: E402
from areal_vllm_amd.ops import delta_rule  # noqa: E402
from areal_vllm_amd.ops import gla as gla_ops  # noqa: E402
from areal_vllm_amd.ops import latent_attention as lattn  # noqa: E402
from areal_vllm_amd.ops import moe as moe_ops  # noqa: E402
from areal_vllm_amd.ops import sandwich as sw  # noqa: E402
from areal_vllm_amd.ops import tanh_norm as tn  # noqa: E402

DEVICES = ["cpu", pytest.param("cuda", marks=pytest.mark.gpu)]
CASES = [("cpu", "float32"), pytest.param("cuda", "float32", marks=pytest.mark.gpu),
         pytest.param("cuda", "bfloat16", marks=pytest.mark.gpu)]
OP_CASES = [("cpu", torch.float32), ("cpu", torch.bfloat16),
            pytest.param("cuda", torch.float32, marks=pytest.mark.gpu),
            pytest.param("cuda", torch.bfloat16, marks=pytest.mark.gpu)]


# ------------------------------------------------------------------------------------ mechanisms
@pytest.mark.parametrize("device,dtype", OP_CASES)
@pytest.mark.parametrize("W", [8, 50, 257, 1032, 7])
def test_embedding_with_sinusoidal_positions(device, dtype, W):
    g = torch.Generator().manual_seed(W)
    embed = torch.randn(19, W, generator=g).to(dtype)
    toks, pos = torch.tensor([3, 0, 18, 7, 7, 1]), torch.tensor([0, 1, 2, 33, 4097, 100000], dtype=torch.int32)
    freq = tn.sinusoid_frequencies(W, 10000.0, device)
    x, xc = tn.embed_sinusoid(toks.to(device), pos.to(device), embed.to(device), freq, want_copy=True)
    want = embed[toks].to(F64) + torch.stack([O.position_vector(int(p), W) for p in pos])
    assert x.dtype == torch.float32 and xc.dtype == dtype
    assert float((x.cpu().to(F64) - want).abs().max()) < 2e-6 * max(1.0, float(want.abs().max()))
    assert torch.equal(xc.cpu(), x.cpu().to(dtype))
    assert tn.embed_sinusoid(toks.to(device), pos.to(device), embed.to(device), freq)[1] is None


def _norm_weights(W, g, dtype):
    return ((0.3 + torch.rand(1, generator=g)).to(dtype), (1 + 0.4 * torch.randn(W, generator=g)).to(dtype),
            (0.5 * torch.randn(W, generator=g)).to(dtype))


def _on(n, device):
    return tuple(t.to(device) for t in n)


def _wide(n):
    return tuple(t.to(F64) for t in n)


@pytest.mark.parametrize("device,dtype", OP_CASES)
@pytest.mark.parametrize("T,W", [(1, 8), (5, 50), (3, 257), (40, 1032), (700, 64), (2, 4100)])
def test_tanh_norm_closing_launch(device, dtype, T, W):
    """x + N_b(y) and what is handed on, with y as a tensor, as slabs and as routed experts in pieces, and a pass entered."""
    g = torch.Generator().manual_seed(T + W)
    b, n = _norm_weights(W, g, dtype), _norm_weights(W, g, dtype)
    x = 3 * torch.randn(T, W, generator=g)
    y = (2 * torch.randn(T, W, generator=g)).to(dtype)
    lim = 2e-6 if is32(dtype) else 1e-2

    def check(z, got, nxt, copy, lim_x=2e-6):
        want = x.to(F64) + O.dyt(z, *_wide(b)) if z is not None else x.to(F64)
        assert rel_err(got[0].cpu(), want) < lim_x
        if nxt:
            h = O.dyt(want, *_wide(n))
            assert got[2].dtype == dtype and rel_err(got[2].float().cpu(), h) < max(lim, lim_x)
            if got[1] is not None:
                assert rel_err(got[1].cpu(), h) < max(4e-6, lim_x)
        elif copy:
            assert torch.equal(got[2].cpu(), got[0].cpu().to(dtype))
        else:
            assert got[2] is None

    for nxt, w32, copy in ((True, True, False), (True, False, False), (False, False, True), (False, False, False)):
        got = tn.norm_add(x.clone().to(device), y.to(device), _on(b, device), _on(n, device) if nxt else None, dtype, w32, copy)
        check(y.to(F64), got, nxt, copy)
        assert not w32 or got[1] is not None
    check(None, tn.norm_add(x.clone().to(device), None, None, _on(n, device), dtype), True, False)
    for S in (1, 3):
        sl = torch.randn(S, T, W, generator=g)
        check(sl.to(F64).sum(0), tn.norm_add(x.clone().to(device), sl.to(device), _on(b, device), _on(n, device), dtype), True,
              False)
    k = 3
    ys, inv = torch.randn(T * k, W, generator=g).to(dtype), torch.randperm(T * k, generator=g)
    wt, sh, sg = torch.rand(T, k, generator=g), torch.randn(T, W, generator=g).to(dtype), 3 * torch.randn(T, 5, generator=g)
    z = (ys.to(F64)[inv].view(T, k, W) * wt.to(F64).unsqueeze(-1)).sum(1)
    for shared in (False, True):
        r = tn.Routed(ys.to(device), inv.to(device), wt.to(device), sh.to(device) if shared else None,
                      sg.to(device)[:, 4] if shared else None)
        check(z + (torch.sigmoid(sg[:, 4:5].to(F64)) * sh.to(F64) if shared else 0),
              tn.norm_add(x.clone().to(device), r, _on(b, device), _on(n, device), dtype, True), True, False)
    p, c, s = torch.randn(T, W, generator=g), torch.randn(T, W, generator=g), torch.randn(W, generator=g).to(dtype)
    out, _, h = tn.enter_pass(p.to(device), c.to(device), s.to(device), torch.empty(T, W, device=device), _on(n, device), dtype)
    want = p.to(F64) + c.to(F64) + s.to(F64)
    assert rel_err(out.cpu(), want) < 2e-6 and rel_err(h.float().cpu(), O.dyt(want, *_wide(n))) < lim


@pytest.mark.parametrize("device,dtype", OP_CASES)
def test_logit_soft_cap(device, dtype):
    z = (20 * torch.randn(3, 1003, generator=torch.Generator().manual_seed(1))).to(dtype)
    for cap in (5.0, 30.0):
        want = cap * torch.tanh(z.to(F64) / cap)
        assert rel_err(tn.softcap_(z.clone().to(device), cap).float().cpu(), want) < (2e-6 if is32(dtype) else 1e-2)


def _delta_inputs(lens, H, G, D, V, g, dtype, strength=1.0):
    """Per sequence: projections (q | k | v, raw), decay logits, write-strength logits; shared bias and decay rates."""
    seqs = []
    for n in lens:
        seqs.append(((torch.randn(n, 2 * G * D + H * V, generator=g)).to(dtype), strength * torch.randn(n, H * D, generator=g),
                     (2 * torch.randn(n, H + 2, generator=g)).to(dtype)))
    return seqs, torch.randn(H * D, generator=g).to(dtype), (0.7 * torch.randn(H, generator=g)).to(dtype)


def _delta_want(seq, bias, a_log, H, G, D, V):
    x, z, beta = (t.to(F64) for t in seq)
    n = x.shape[0]
    q, k = O.unit(x[:, :G * D].reshape(n, G, D)) * D ** -0.5, O.unit(x[:, G * D:2 * G * D].reshape(n, G, D))
    f = torch.exp(-torch.exp(a_log.to(F64)).view(1, H, 1) * O.softplus(z + bias.to(F64)).view(n, H, D))
    return O.delta_rule(q, k, x[:, 2 * G * D:].reshape(n, H, V), f, torch.sigmoid(beta[:, 2:]))


DELTA_SHAPES = [(2, 2, 8, 8), (4, 2, 16, 24), (3, 1, 20, 5), (2, 1, 50, 33), (1, 1, 64, 64), (2, 2, 128, 80), (2, 1, 100, 20),
                (1, 1, 7, 3), (2, 1, 160, 12), (1, 1, 256, 8), (6, 3, 12, 40)]


@pytest.mark.parametrize("device,dtype", OP_CASES)
@pytest.mark.parametrize("H,G,D,V", DELTA_SHAPES)
def test_delta_rule_of_unequal_rows_in_portions(device, dtype, H, G, D, V):
    """Three sequences in one batch, cut in several ways (both sides of a chunk's length), dirty slots, a padding row."""
    g = torch.Generator().manual_seed(H + D + V)
    lens, slot = [75, 3, 33], [3, 1, 0]
    seqs, bias, a_log = _delta_inputs(lens, H, G, D, V, g, dtype)
    want = [_delta_want(s, bias, a_log, H, G, D, V) for s in seqs]
    state = delta_rule.alloc_state(5, H, D, V, device).fill_(11.0)
    for plan in ([[75], [3], [33]], [[1], [1], [1]], [[2, 1, 30, 7, 16, 1, 15, 3], [2, 1], [17, 16]], [[40, 17, 16, 2], [1, 2], [4]]):
        cuts = [portions_of(n, p) for n, p in zip(lens, plan)]
        at, got = [0, 0, 0], [[], [], []]
        while any(cuts):
            rows = [i for i in range(3) if cuts[i]]
            size = [cuts[i].pop(0) for i in rows]
            cu = [0]
            for c in size + [1]:
                cu.append(cu[-1] + c)
            parts = [torch.cat([seqs[i][j][at[i]:at[i] + c] for i, c in zip(rows, size)] + [seqs[0][j][:1]]).to(device)
                     for j in range(3)]
            o = delta_rule.delta_scan(parts[0], 0, G * D, 2 * G * D, G, parts[1], bias.to(device), a_log.to(device),
                                      parts[2][:, 2:], D ** -0.5, i32(cu, device), i32([at[i] for i in rows] + [0], device),
                                      i32([slot[i] for i in rows] + [-1], device), state, max_q=max(size))
            assert float(o[cu[-2]:].abs().max()) == 0.0
            for j, i in enumerate(rows):
                got[i].append(o[cu[j]:cu[j + 1]].cpu())
                at[i] += size[j]
        for i in range(3):
            lim = 2e-5 if is32(dtype) else 1e-4  # bf16: hardware exponentials in the chunked form
            assert rel_err(torch.cat(got[i]).reshape(lens[i], -1), want[i][0].reshape(lens[i], -1)) < 10 * lim, plan
            assert rel_err(state[slot[i]].cpu().reshape(1, -1), want[i][1].transpose(1, 2).reshape(1, -1)) < 10 * lim, plan
    assert float(state[2].min()) == 11.0 and float(state[4].max()) == 11.0  # nobody else's slot is touched


@pytest.mark.parametrize("device,dtype", OP_CASES)
def test_delta_rule_far_key_and_erased_key(device, dtype):
    """Slow decays: a key written once is read hundreds of tokens later in spite of everything written since (its direction
    is kept free), and a second write to the same key replaces the value. Strong decays underflow without harm."""
    H, G, D, V, n = 2, 1, 32, 16, 400
    g = torch.Generator().manual_seed(3)
    x = torch.zeros(n, 2 * G * D + H * V)
    x[:, :2 * D] = torch.randn(n, 2 * D, generator=g)
    x[:, :D], x[:, D] = 0.0, 0.0  # every query asks for channel 0 alone; no key has it ...
    x[:, 0] = 1.0
    x[5, D:2 * D] = 0.0
    x[5, D] = 1.0  # ... but the sixth token's
    x[300, D:2 * D] = x[5, D:2 * D]
    x[:, 2 * D:] = torch.randn(n, H * V, generator=g)
    seq = (x.to(dtype), torch.full((n, H * D), -9.0), torch.full((n, H + 2), 8.0).to(dtype))
    bias, a_log = torch.zeros(H * D).to(dtype), torch.tensor([-1.0, -3.0]).to(dtype)

    def run(seq, sizes):
        st, at, out = delta_rule.alloc_state(1, H, D, V, device).fill_(5.0), 0, []
        for c in portions_of(n, sizes):
            p = [t[at:at + c].to(device) for t in seq]
            out.append(delta_rule.delta_scan(p[0], 0, D, 2 * D, G, p[1], bias.to(device), a_log.to(device), p[2][:, 2:],
                                             D ** -0.5, i32([0, c], device), i32([at], device), i32([0], device), st, max_q=c).cpu())
            at += c
        return torch.cat(out)

    want, _ = _delta_want(seq, bias, a_log, H, G, D, V)
    v5 = x[5, 2 * D:].to(dtype).to(F64).view(H, V)
    assert rel_err(want[299].reshape(1, -1), (v5 * D ** -0.5).reshape(1, -1)) < 0.1  # the far value is what is read
    assert rel_err(want[399].reshape(1, -1), (v5 * D ** -0.5).reshape(1, -1)) > 0.5  # and replaced later
    for sizes in ([n], [1], [299, 1, 1, 99], [6, 2, 200, 16]):
        got = run(seq, sizes)
        assert rel_err(got[5:].reshape(n - 5, -1), want[5:].reshape(n - 5, -1)) < (1e-4 if is32(dtype) else 1e-3), sizes
    strong = (seq[0], torch.full((n, H * D), 60.0), seq[2])
    want, _ = _delta_want(strong, bias, a_log, H, G, D, V)
    for sizes in ([n], [1]):
        got = run(strong, sizes)
        assert torch.isfinite(got).all() and float((got.to(F64) - want).abs().max()) < 1e-5


@pytest.mark.parametrize("device,dtype", OP_CASES)
def test_short_convolution_without_bias(device, dtype):
    g = torch.Generator().manual_seed(9)
    for C, taps in ((24, 3), (40, 1), (136, 2), (10, 5)):
        w, h = torch.randn(C, taps, generator=g).to(dtype), torch.randn(37, C + 3, generator=g).to(dtype)
        want = O.silu(O.causal_conv(h[:, :C].to(F64), w.to(F64)))
        for sizes in ([37], [1], [2], [20, 1, 16]):
            hist = torch.full((2, taps - 1, C), 9.0, device=device) if taps > 1 else None
            at, got = 0, []
            for c in portions_of(37, sizes):
                got.append(sw.conv_silu(h[at:at + c].to(device)[:, :C], w.to(device), None, hist, i32([0, c], device),
                                        i32([at], device), i32([1], device), c).float().cpu())
                at += c
            assert rel_err(torch.cat(got), want) < (1e-5 if is32(dtype) else 1e-2), (C, taps, sizes)


@pytest.mark.parametrize("device,dtype", OP_CASES)
@pytest.mark.parametrize("V", [20, 64, 7])
def test_normed_readout_behind_a_sigmoid_gate(device, dtype, V):
    g = torch.Generator().manual_seed(V)
    T, H = 5, 3
    o, gate, w = torch.randn(T, H, V, generator=g), (2 * torch.randn(T, H * V, generator=g)).to(dtype), torch.randn(V, generator=g).to(dtype)
    y = gla_ops.gla_out(o.to(device), gate.to(device), w.to(device), 1e-5, gate_act="sigmoid")
    want = O.rms_norm(o.to(F64), w.to(F64), 1e-5).reshape(T, -1) * torch.sigmoid(gate.to(F64))
    assert rel_err(y.float().cpu(), want) < (1e-5 if is32(dtype) else 1e-2)
    y = gla_ops.gla_out(o.to(device), gate.to(device), w.to(device), 1e-5)
    want = O.rms_norm(o.to(F64), w.to(F64), 1e-5).reshape(T, -1) * O.silu(gate.to(F64))
    assert rel_err(y.float().cpu(), want) < (1e-5 if is32(dtype) else 1e-2)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("E,k,count,keep", [(8, 2, 4, 2), (8, 4, 4, 3), (6, 3, 1, 1), (16, 5, 8, 5), (96, 6, 6, 2), (160, 8, 8, 3),
                                            (4, 1, 4, 1), (12, 12, 3, 3), (9, 2, 3, 1)])
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_corrected_group_limited_choice(device, E, k, count, keep, dtype):
    """Corrections large enough to move the choice, negative sums among them: a group left out counts as minus infinity."""
    g = torch.Generator().manual_seed(E + k)
    T, router = 64, {"experts": E, "top": k, "groups": {"count": count, "keep": keep}, "scale": 1.7}
    z = 2 * torch.randn(T, E + 1, generator=g)
    moved = 0
    for corr in (0.3 * torch.randn(E, generator=g), -1.0 - torch.rand(E, generator=g), torch.zeros(E)):
        corr = corr.to(dtype)
        wt, ids = moe_ops.moe_corrected_topk(z.to(device)[:, :E], k, count, keep, corr.to(device), 1.7)
        want = O.route(z[:, :E].to(F64), corr.to(F64), router)
        plain = O.route(z[:, :E].to(F64), torch.zeros(E, dtype=F64), dict(router, groups=None))
        for t in range(T):
            chosen, w = want[t]
            assert ids[t].tolist() == chosen
            assert float((wt[t].cpu().to(F64) - w).abs().max()) < 1e-5
            moved += set(chosen) != set(plain[t][0])
    assert moved > 0 or k == E


def _latent_case(H, D, V, R, n, probe, seed, scale):
    """Queries, latents and expansions of one sequence; `probe` = (query position, key position): that key's score stands
    out for every head of that query."""
    g = torch.Generator().manual_seed(seed)
    q, c = torch.randn(n, H, D, generator=g), torch.randn(n, R, generator=g)
    uk, uv = torch.randn(H * D, R, generator=g) / R ** 0.5, torch.randn(H * V, R, generator=g) / R ** 0.5
    sink = 0.5 + torch.rand(H, generator=g)
    if probe is not None:
        qi, kj = probe
        c[kj] = 0.0
        for h in range(H):
            c[kj] += 4.0 * uk.view(H, D, R)[h].T @ q[qi, h] / H ** 0.5
    return q, c, uk, uv, sink


def _latent_want(q, c, uk, uv, sink, scale, dtype, eps):
    """Dense attention with expanded keys and values on the operands as stored; the sink joins the denominator."""
    n, H, D = q.shape
    cn = O.rms_norm(seen(c, dtype), torch.ones(c.shape[1], dtype=F64), eps)
    k, v = (cn @ seen(uk, dtype).T).view(n, H, D), (cn @ seen(uv, dtype).T).view(n, H, -1)
    s = torch.einsum("ihd,jhd->hij", seen(q, dtype), k) * scale
    s = s.masked_fill(torch.ones(n, n).triu(1).bool(), float("-inf"))
    s = torch.cat([s, seen(sink, dtype).view(H, 1, 1).expand(H, n, 1)], -1)
    p = torch.softmax(s, -1)[..., :n]
    return torch.einsum("hij,jhv->ihv", p, v).reshape(n, -1)


def _run_latent(q, c, uk, uv, sink, scale, dtype, device, sizes, pages, eps, nsplit=1, matrix_cores=True):
    n, H, D = q.shape
    R = c.shape[1]
    V = uv.shape[0] // H
    cache = lattn.alloc_latent_cache(max(pages) + 2, R, 0, dtype, device).fill_(50.0)
    table = lattn.rotary_table(1.0, 0, n + 1, device)
    bt = torch.tensor([pages], dtype=torch.int32, device=device)
    qd, cd, ukd, uvd, sk = (t.to(dtype).to(device) for t in (q, c, uk, uv, sink))
    ones, out, at = torch.ones(R, dtype=dtype, device=device), [], 0
    for m in portions_of(n, sizes):
        pos = torch.arange(at, at + m, dtype=torch.int32, device=device)
        lattn.latent_prep(cd[at:at + m], 0, R, 0, None, ones, pos, slots_of(pages, at, at + m, device), cache, table, eps)
        ql = torch.bmm(qd[at:at + m].transpose(0, 1).float(), ukd.view(H, D, R).float()).transpose(0, 1).to(dtype).contiguous()
        o = lattn.latent_attention(qd[at:at + m].contiguous(), ql, cache, bt, i32([0, m], device), i32([at + m], device), m, D, 0,
                                   scale, 0, table, nsplit=nsplit if m == 1 else 1, matrix_cores=matrix_cores, sink=sk)
        out.append(lattn.expand_values(o, uvd).float().cpu())
        at += m
    return torch.cat(out)


@pytest.mark.parametrize("device,dtype", OP_CASES)
@pytest.mark.parametrize("H,D,V,R", [(2, 8, 12, 24), (3, 20, 5, 64), (4, 16, 24, 128), (1, 8, 8, 256), (17, 16, 16, 64), (2, 16, 40, 512),
                                     (5, 10, 7, 33)])
def test_latent_attention_without_positions_far_keys_pages_portions_and_splits(device, dtype, H, D, V, R):
    n, pages, eps = 140, [3, 1, 4, 9, 2], 1e-5
    scale = 1.0 / math.sqrt(D)
    for k, (qi, kj) in enumerate(((139, 0), (139, 1), (138, 31), (131, 32), (100, 63), (97, 64), (96, 95), (64, 64), (33, 0), (1, 0))):
        case = _latent_case(H, D, V, R, n, (qi, kj), 5 + k % 3, scale)
        want = _latent_want(*case, scale, dtype, eps)[qi:qi + 1]
        for sizes, ns in (([n], 1), ([qi, 1, n], 1 + 3 * (k % 2)), ([max(qi - 1, 1), 2, n], 1)):
            got = _run_latent(*case, scale, dtype, device, sizes, pages, eps, ns)
            assert rel_err(got[qi:qi + 1], want) < tol(dtype), (qi, kj, sizes, ns)
    case = _latent_case(H, D, V, R, n, None, 1, scale)
    want = _latent_want(*case, scale, dtype, eps)
    for sizes, ns, mc in (([n], 1, True), ([n], 1, False), ([1], 5, True), ([1], 1, False), ([2], 1, True),
                          ([3, 17, 1, 1, 64, 31, 2, 33], 4, True)):
        assert rel_err(_run_latent(*case, scale, dtype, device, sizes, pages, eps, ns, mc), want) < tol(dtype), (sizes, ns, mc)
    without = _latent_want(*case[:4], torch.full((H,), -1e4), scale, dtype, eps)
    assert rel_err(without[:3], want[:3]) > 0.1  # leaving the sink out shows at the first tokens


@pytest.mark.gpu
@pytest.mark.parametrize("H,R", [(1, 64), (2, 512), (5, 200)])
def test_expanded_keys_and_values_of_long_prompt_portions(H, R):
    """Heads of 128 in bf16: rows of unequal portions and contexts in one batch, dirty pages, keys far away and at the edges
    of pages and key tiles, the sink at the first tokens; against dense attention and against the route over the latents."""
    D = V = 128
    scale, eps, dtype, dev = 1.0 / math.sqrt(D), 1e-5, torch.bfloat16, "cuda"
    rows = [(300, 300, (299, 0)), (130, 257, (256, 64)), (97, 97, (96, 63)), (200, 201, (200, 199)), (128, 384, (300, 31))]
    cache = torch.full((64, PAGE, R), 60.0, dtype=dtype, device=dev)
    bt, free = torch.zeros(len(rows), 13, dtype=torch.int32), list(range(1, 64))
    random.Random(R).shuffle(free)
    cases, qs, cu, ck = [], [], [0], [0]
    first = _latent_case(H, D, V, R, 1, None, 3, scale)
    for b, (n, ctx, probe) in enumerate(rows):
        q, c, _, _, _ = _latent_case(H, D, V, R, ctx, probe, 11 + b, scale)
        case = (q, c, *first[2:])
        pages = [free.pop() for _ in range((ctx + PAGE - 1) // PAGE)]
        bt[b, :len(pages)] = torch.tensor(pages)
        cases.append(case)
        pos = torch.arange(ctx, dtype=torch.int32, device=dev)
        lattn.latent_prep(c.to(dtype).to(dev), 0, R, 0, None, torch.ones(R, dtype=dtype, device=dev), pos,
                          slots_of(pages, 0, ctx, dev), cache, lattn.rotary_table(1.0, 0, ctx, dev), eps)
        qs.append(q[-n:])
        cu.append(cu[-1] + n)
        ck.append(ck[-1] + ctx)
    q = torch.cat(qs).to(dtype).to(dev)
    uk, uv, sink = (t.to(dtype).to(dev) for t in first[2:])
    bt = bt.to(dev)
    got = lattn.expanded_attention(q, cache, bt, i32(cu, dev), i32(ck, dev), 300, uk, uv, scale, sink).float().cpu()
    ctx = i32([r[1] for r in rows], dev)
    other = lattn.expand_values(lattn.latent_attention(q, lattn.absorb_keys(q, uk), cache, bt, i32(cu, dev), ctx, 300, D, 0, scale,
                                                       0, lattn.rotary_table(1.0, 0, 400, dev), sink=sink), uv).float().cpu()
    for b, (n, _, _) in enumerate(rows):
        want = _latent_want(*cases[b], scale, dtype, eps)[-n:]
        assert rel_err(got[cu[b]:cu[b + 1]].reshape(n, -1), want) < tol(dtype), b
        assert rel_err(other[cu[b]:cu[b + 1]], want) < tol(dtype), b


@pytest.mark.parametrize("device,dtype", OP_CASES)
@pytest.mark.parametrize("T,H,V,R", [(1, 2, 8, 32), (16, 3, 20, 64), (17, 1, 130, 96), (64, 4, 64, 128), (65, 2, 16, 64), (5, 2, 7, 33)])
def test_values_from_attended_latents(device, dtype, T, H, V, R):
    g = torch.Generator().manual_seed(T)
    o, uv = torch.randn(T, H, R, generator=g).to(dtype), (torch.randn(H * V, R, generator=g) / R ** 0.5).to(dtype)
    want = torch.einsum("thr,hvr->thv", o.to(F64), uv.to(F64).view(H, V, R)).reshape(T, -1)
    assert rel_err(lattn.expand_values(o.to(device), uv.to(device)).float().cpu(), want) < (2e-5 if is32(dtype) else 1e-2)


# ------------------------------------------------------------------------------------ the model in the engine
def dense(ff):
    return {"kind": "dense", "ff": ff}


def moe(experts=6, top=2, ff=20, shared=28, groups=(3, 2), scale=1.6):
    return {"kind": "moe", "expert": {"ff": ff}, "shared": {"ff": shared} if shared else None,
            "router": {"experts": experts, "top": top, "scale": scale,
                       "groups": {"count": groups[0], "keep": groups[1]} if groups else None}}


def delta(heads=4, kv=2, dim=12, vdim=20, conv=4, ra=5, rg=7, mlp=None):
    return {"type": "channel_delta", "mlp": mlp,
            "mixer": {"conv": conv, "dim": dim, "heads": heads, "kv_heads": kv, "vdim": vdim, "decay_rank": ra, "gate_rank": rg}}


def latent(heads=3, dim=12, vdim=10, q_rank=22, kv_rank=36, scale=0.4, mlp=None):
    return {"type": "latent_attention", "mlp": mlp,
            "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "q_rank": q_rank, "kv_rank": kv_rank, "scale": scale}}


def config(layers, loop=None, width=48, vocab=101, eps=1e-5, cap=12.0):
    return {"architecture": "Keginex", "layers": layers, "logit_softcap": cap, "loop": dict(zip(("start", "stop", "times"), loop))
            if loop else None, "norm": {"eps": eps}, "vocab": vocab, "width": width}


MIXED = config([latent(mlp=dense(40)), delta(mlp=moe()), latent(2, 10, 16, 9, 64), delta(1, 1, 16, 8, 2, 3, 2, mlp=moe(8, 3, 12, 0, None))],
               loop=(1, 3, 2))
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
def test_whole_prompt_and_every_layer_run(device, dtype):
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
        toks = tokens_of(120, MIXED["vocab"], 2)
        for k, sizes in enumerate(([1], [60, 1], [2], [3, 64, 2, 31, 1, 1, 5], [1, 32, 32, 32, 1], [17, 16, 15])):
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
    # one head everywhere, equal sizes everywhere, factors of 1, a loop over everything
    config([delta(1, 1, 16, 16, 1, 16, 16, dense(16)), latent(1, 16, 16, 16, 16, 1.0, moe(2, 1, 16, 16, None, 1.0))], (0, 2, 2), width=16),
    # sizes that are no multiples of 8 or of each other, no loop, no feed-forward in places
    config([latent(5, 10, 14, 11, 30, 0.2, moe(9, 4, 10, 6, (3, 2), 0.7)), delta(6, 2, 10, 14, 3, 3, 9), latent(1, 6, 4, 5, 18, 0.9, dense(30)),
            delta(3, 1, 22, 9, 5, 1, 1, dense(22))], width=40, vocab=67, eps=1e-3),
    config([delta(2, 2, 8, 8, 2, 2, 3)], (0, 1, 3), width=24),  # recurrent alone: no paged cache at all
    config([latent(2, 8, 8, 8, 16, 0.5), latent(2, 8, 8, 8, 16, 0.5, moe(4, 2, 8, 8, (2, 1)))], (1, 2, 1), width=24),  # no state
    # nothing a multiple of 4, a loop of one layer, the last layers inside the loop, no soft cap
    config([delta(3, 3, 7, 5, 3, 3, 2, dense(9)), latent(3, 6, 7, 13, 25, 0.6, moe(6, 3, 7, 5, (2, 2))), delta(2, 1, 9, 11, 4, 2, 5)], (2, 3, 3),
           width=50, vocab=59, cap=0.0),
    # sizes the matrix-core paths take
    config([delta(2, 1, 128, 64, 4, 16, 16, moe(8, 2, 64, 64, (4, 2))), latent(16, 64, 64, 64, 512, 0.1, moe(8, 2, 64, 128, (4, 2))),
            delta(2, 2, 64, 128, 4, 8, 8, dense(128)), latent(4, 32, 32, 64, 256, 0.2), latent(4, 32, 32, 64, 128, 0.2), delta(1, 1, 160, 24)],
           (1, 3, 2), width=64),
]


@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("which", range(len(SHAPES)))
def test_other_sizes_loops_constants_and_orders(device, dtype, which):
    cfg = SHAPES[which]
    eng, w = make_engine(cfg, device, dtype)
    try:
        toks = tokens_of(70, cfg["vocab"], 20 + which)
        key = ("shapes", which, device, dtype)
        check(replay(eng, cut("w", toks, [len(toks)])), toks, w, cfg, dtype, "w", key=key)
        check(replay(eng, cut("c", toks, [7, 2, 33, 1, 1, 20, 1])), toks, w, cfg, dtype, "c", key=key)
    finally:
        eng.destroy()


@pytest.mark.parametrize("device,dtype", CASES)
def test_long_portions_of_wide_heads(device, dtype):
    """Heads of 128: long portions take the route over expanded keys and values, short ones and decoding the one over the
    latents, through the same cache; cut at and around page and tile edges, beside another request."""
    cfg = config([latent(2, 128, 128, 24, 64, 0.12), delta(2, 1, 64, 64, mlp=dense(64))], loop=(0, 1, 2), width=64)
    eng, w = make_engine(cfg, device, dtype)
    try:
        toks, short = tokens_of(200, cfg["vocab"], 31), tokens_of(40, cfg["vocab"], 32)
        key = ("wide", device, dtype)
        for k, sizes in enumerate(([200], [100, 100], [96, 1, 103], [3, 97, 2, 98])):
            check(replay(eng, cut(f"r{k}", toks, sizes)), toks, w, cfg, dtype, f"r{k}", key=key)
        steps = [[("a", toks[:160], list(range(160)), False), ("b", short, list(range(40)), True)],
                 [("a", toks[160:], list(range(40)), True)]]
        got = replay(eng, steps)
        check(got, toks, w, cfg, dtype, "a", key=key)
        check(got, short, w, cfg, dtype, "b")
    finally:
        eng.destroy()


@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("seed", [1, 2, 3])
def test_random_shapes_orders_and_schedules(device, dtype, seed):
    """Random layer lists (mixer kinds and sizes, loops, constants, with and without feed-forward) fed through random
    schedules of up to three live requests: portions of 1 .. 100 tokens, requests that skip steps."""
    rng = random.Random(seed)
    for case in range(2):
        width, vocab, layers = rng.choice([32, 48, 72]), rng.choice([37, 101]), []
        for _ in range(rng.randint(1, 3)):
            ff = rng.choice([None, dense(rng.choice([8, 20, 64])),
                             moe(*rng.choice([(4, 2), (8, 3), (6, 1)]), rng.choice([8, 64]), rng.choice([0, 12, 64]),
                                 rng.choice([None, (2, 1), (2, 2)]), rng.choice([1.0, 2.2]))])
            kv = rng.choice([1, 2])
            if rng.random() < 0.5:
                layers.append(delta(kv * rng.choice([1, 2]), kv, rng.choice([8, 12, 64, 128]), rng.choice([8, 20, 64]), rng.choice([1, 2, 4]),
                                    rng.choice([1, 4, 16]), rng.choice([1, 4, 16]), ff))
            else:
                layers.append(latent(rng.choice([1, 2, 5]), rng.choice([8, 12, 64]), rng.choice([8, 20, 64]), rng.choice([8, 22]),
                                     rng.choice([16, 64, 128, 40]), rng.choice([0.1, 0.3]), ff))
        a = rng.randrange(len(layers))
        loop = rng.choice([None, (a, rng.randint(a + 1, len(layers)), rng.randint(1, 3))])
        cfg = config(layers, loop, width, vocab, rng.choice([1e-5, 1e-6]), rng.choice([6.0, 30.0]))
        reqs = {f"q{i}": tokens_of(rng.choice([1, 2, 17, 60, 120]), vocab, 7 + 100 * case + i) for i in range(rng.randint(1, 3))}
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
    cfg = config([delta(2, 1, mlp=dense(24)), latent(2)], loop=(1, 2, 2))
    eng, w = make_engine(cfg, device, dtype)
    try:
        for n in (1, 2, 3, 5):
            toks = tokens_of(n, cfg["vocab"], 40 + n)
            check(replay(eng, cut(f"s{n}", toks, [1])), toks, w, cfg, dtype, f"s{n}")
            check(replay(eng, cut(f"w{n}", toks, [n])), toks, w, cfg, dtype, f"w{n}")
        toks = tokens_of(200, cfg["vocab"], 44)
        check(replay(eng, cut("long", toks, [20, 1])), toks, w, cfg, dtype, "long")
    finally:
        eng.destroy()


def test_what_a_fault_would_look_like():
    """Leaving out the correction, the pass vectors, the embedding's second way in, the sink or the shared expert's gate
    changes the logits by far more than the tolerances: the comparisons above can see each."""
    from areal_vllm_amd.models import build_model

    m = build_model(ModelConfig.from_hf_dict(MIXED), dtype=torch.float32)
    m.flatten()
    m.init_weights(seed=3)
    w, toks = weights_of(m), tokens_of(30, MIXED["vocab"], 5)
    want, _ = O.forward(MIXED, w, toks)
    W = MIXED["width"]
    faults = {"loop.step": lambda t: 0 * t, "loop.in": lambda t: torch.cat([t[:, :W], 0 * t[:, W:]], 1),
              "l0.mix.sink": lambda t: t - 1e3, "l1.mlp.shared.sg": lambda t: 0 * t, "l1.mix.b": lambda t: 0 * t,
              "l1.mix.dt_bias": lambda t: t + 3.0, "l1.mlp.correction": lambda t: 0 * t - t}
    for name, f in faults.items():
        got, _ = O.forward(MIXED, dict(w, **{name: f(w[name])}), toks)
        assert rel_err(got, want) > 0.01, name


@pytest.mark.parametrize("device,dtype", CASES)
def test_greedy_generation_through_the_engine(device, dtype):
    """The engine's own entry point: prompts of unequal length generated together, prefill plans, then decode plans
    (captured graphs on the GPU), more requests than request slots."""
    cfg = config([delta(2, 1, mlp=dense(24)), latent(2, mlp=moe()), delta(1, 1, 8, 8)], loop=(1, 2, 2), vocab=61)
    eng, w = make_engine(cfg, device, dtype, max_running=3, score=False)
    try:
        prompts = [tokens_of(n, cfg["vocab"], 50 + n) for n in (3, 41, 18, 1, 50)]
        res = eng.generate_blocking(prompts, max_new_tokens=10, greedy=True)
        agree = 0
        for p, r in zip(prompts, res):
            assert r.finish_reason == "length" and len(r.output_tokens) == 10
            want = O.greedy(cfg, w, p, 10 if is32(dtype) else 1)
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
    configuration, the ranks of the low-rank projections by tensors' shapes, the weights come through the engine's loader;
    several decode steps per plan."""
    cfg_dict = config([delta(2, 1, 8, 8, 3, 3, 4, dense(20)), latent(2, 8, 8, 10, 16, 0.5, moe(4, 2, 8, 8, (2, 1)))], (0, 1, 2), width=32, vocab=53)
    w = weights_of(saved_model(cfg_dict, tmp_path, torch.bfloat16, 9))
    with open(tmp_path / "config.json") as f:
        saved = json.load(f)
    for l in saved["layers"]:  # a checkpoint whose configuration does not name the ranks
        l["mixer"].pop("decay_rank", None)
        l["mixer"].pop("gate_rank", None)
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

    cfg_dict = config([delta(2, 1, 8, 8, 3, 3, 4, dense(20)), latent(2, 8, 8, 10, 16, 0.5)], (1, 2, 2), width=32, vocab=53)
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
    assert cfg.family == "keginex" and cfg.n_layers == 4 and cfg.has_recurrent_state and not cfg.tie_word_embeddings
    assert cfg.rms_norm_eps == 1e-3 and cfg.logit_softcap == 12.0 and cfg.pass_starts == {} and cfg.layer_runs == [0, 1, 2, 3]
    looped = ModelConfig.from_hf_dict(MIXED)
    assert looped.layer_runs == [0, 1, 2, 1, 2, 3] and looped.pass_starts == {1: 0, 3: 1}
    assert not ModelConfig.from_hf_dict(SHAPES[3]).has_recurrent_state
    from areal_vllm_amd.models import build_model

    for i, d in enumerate((SHAPES[1], MIXED)):
        path, cfg = tmp_path / str(i), ModelConfig.from_hf_dict(d)
        m = saved_model(d, path, torch.float32, 4)
        assert sum(t.numel() for t in m.checkpoint_tensors().values()) == cfg.n_params()
        cfg2 = ModelConfig.from_pretrained(str(path))
        assert cfg2.layers == cfg.layers and cfg2.loop == cfg.loop and cfg2.logit_softcap == cfg.logit_softcap
        m2 = build_model(cfg2, dtype=torch.float32)
        m2.flatten()
        m2.load_checkpoint(str(path))
        for (n1, a), (n2, b) in zip(m.checkpoint_tensors().items(), m2.checkpoint_tensors().items()):
            assert n1 == n2 and torch.equal(a, b)
        with pytest.raises(KeyError):
            m2.assign_named_tensors(dict(m2.checkpoint_tensors(), **{"l0.norm3": torch.zeros(40)}))
        no_ff = [j for j, l in enumerate(cfg.layers) if l["mlp"] is None][0]  # what a missing feed-forward would own is not read
        m2.assign_named_tensors({f"l{no_ff}.norm2": torch.zeros(40), f"l{no_ff}.norm2b.alpha": torch.zeros(())})
    bad = delta()
    del bad["mixer"]["gate_rank"]
    for l in (dict(delta(), type="conv"), delta(heads=3, kv=2), bad, delta(mlp={"kind": "other"}), latent(mlp=moe(7, 2))):
        with pytest.raises(ValueError):
            ModelConfig.from_hf_dict(config([l]))
    with pytest.raises(ValueError):
        ModelConfig.from_hf_dict(config([latent()], (0, 2, 1)))
