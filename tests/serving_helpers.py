"""Helpers of the serving tests of layer-list decoders: error measures, replay of token steps through the engine."""
import numpy as np
import torch

from areal_vllm_amd.api.cli_args import InferenceServerConfig
from areal_vllm_amd.inference.engine import NativeInferenceEngine
from areal_vllm_amd.models.config import ModelConfig

F64 = torch.float64
PAGE = 32


def is32(dtype):
    return dtype in ("float32", torch.float32)


def tol(dtype):
    return 2e-4 if is32(dtype) else 6e-2


def row_errors(got, want):
    """Per row: rms of the difference (mean taken off) over the rms of the reference row."""
    got, want = torch.as_tensor(got).to(F64), torch.as_tensor(want).to(F64)
    d = got - want
    d = d - d.mean(-1, keepdim=True)
    ref = (want - want.mean(-1, keepdim=True)).pow(2).mean(-1).sqrt().clamp(min=1e-9)
    return d.pow(2).mean(-1).sqrt() / ref


def rel_err(got, want):
    return float(row_errors(got, want).max())


def rows_agree(got, want, dtype):
    """32-bit: the median row (of more than two) within the tolerance, every row within ten times it. bf16: the median row
    within the tolerance and nine rows of ten within three times it. A sublayer's output that happens to be close to zero
    is blown up by the norm behind it, rounding included: single rows of a tiny random model may be off by their own
    size in 16-bit arithmetic of any kind."""
    e = row_errors(got, want)
    median = e.numel() <= 2 or bool(e.median() < tol(dtype))
    if is32(dtype):
        return median and bool(e.max() < 10 * tol(dtype))
    return median and bool((e < 3 * tol(dtype)).double().mean() >= 0.9)


def i32(x, device):
    return torch.tensor(x, dtype=torch.int32, device=device)


def slots_of(pages, lo, hi, device):
    return torch.tensor([pages[p // PAGE] * PAGE + p % PAGE for p in range(lo, hi)], dtype=torch.int64, device=device)


def seen(x, dtype):
    """What the kernels see of a tensor held in `dtype`, as float64."""
    return x.to(dtype).to(F64)


def portions_of(n, sizes):
    """Portion sizes that add up to n; the last of `sizes` repeats."""
    out, at, i = [], 0, 0
    while at < n:
        c = min(sizes[min(i, len(sizes) - 1)], n - at)
        out.append(c)
        at += c
        i += 1
    return out


def tokens_of(n, vocab, seed):
    return torch.randint(0, vocab, (n,), generator=torch.Generator().manual_seed(seed)).tolist()


def make_engine(cfg_dict, device, dtype, num_pages=40, max_running=4, context=512, score=True):
    cfg = ModelConfig.from_hf_dict(cfg_dict)
    srv = InferenceServerConfig(model_path="", dtype=dtype, context_length=context, max_running_requests=max_running,
                                num_continuous_decode_steps=1, max_prefill_tokens=context)
    eng = NativeInferenceEngine(srv, model_config=cfg, device=torch.device(device), num_pages=num_pages,
                                score_mode=score)
    eng.initialize(load_weights=False)
    return eng, weights_of(eng.model)


def weights_of(model):
    return {k: v.detach().cpu().to(F64) for k, v in model.checkpoint_tensors().items()}


def replay(eng, steps):
    """steps: lists of (request id, tokens, wanted places, ends after this step) -> {id: {position: logits}}."""
    out, fed, live = {}, {}, set()
    for step in steps:
        for rid, _, _, _ in step:
            if rid not in live:
                eng.open_replay(rid)
                live.add(rid)
                fed[rid] = 0
        logits = eng.replay_step([(rid, toks, want) for rid, toks, want, _ in step])
        at = 0
        for rid, toks, want, end in step:
            for w in want:
                out.setdefault(rid, {})[fed[rid] + w] = logits[at]
                at += 1
            fed[rid] += len(toks)
            if end:
                eng.close_replay(rid)
                live.discard(rid)
        assert at == logits.shape[0]
    return out


def cut(rid, tokens, sizes):
    """One request alone, fed in portions of the given sizes (the last repeats); every position is wanted."""
    steps, at = [], 0
    for c in portions_of(len(tokens), sizes):
        steps.append([(rid, tokens[at:at + c], list(range(c)), at + c == len(tokens))])
        at += c
    return steps


def rows_of(got, rid, n):
    return torch.from_numpy(np.stack([got[rid][p] for p in range(n)]))
