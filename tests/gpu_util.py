"""Helpers of GPU tests: tensors to and from the device, what the kernels read of a step, and a runner driven by a schedule."""

from __future__ import annotations

from types import SimpleNamespace

import numpy as np
import torch

DEV = "cuda:0"
PAGE = 16


def ops():
    from miniserve_amd.kernels import ops as o

    o.library()
    return o


def dev(a, dtype=torch.float32):
    return torch.tensor(np.asarray(a), dtype=dtype, device=DEV).contiguous()


def rounded(a, dtype):
    """What a kernel is given when ``a`` is stored in ``dtype``."""
    return dev(a, dtype).float().cpu().numpy().astype(np.float64)


def close(got, want, dtype, what="", tol=None):
    got = got.float().cpu().numpy().astype(np.float64)
    assert np.isfinite(got).all(), f"{what}: not all numbers"
    scale = max(float(np.abs(want).max()), 1e-30)
    tol = tol or (2e-5 if dtype == torch.float32 else 1.2e-2)
    worst = float(np.abs(got - want).max())
    assert worst <= tol * scale, f"{what}: max |diff| {worst:.3e} > {tol * scale:.3e}"


def step_batch(lens, starts, slots=None):
    """What the kernels read of a step: rows of ``lens`` new tokens behind ``starts`` cached ones."""
    pos = np.concatenate([np.arange(s, s + n) for n, s in zip(lens, starts)])
    row = np.concatenate([np.full(n, i) for i, n in enumerate(lens)])
    flat = np.arange(int(sum(lens)))
    single = np.concatenate([np.full(n, n == 1) for n in lens])
    n_dec = int(single.sum())
    mixed = 0 < n_dec < len(flat)
    b = SimpleNamespace(num_rows=len(lens), num_tokens=int(sum(lens)), positions=dev(pos, torch.int32), token_row=dev(row, torch.int32),
                        row_start=dev(np.concatenate(([0], np.cumsum(lens))), torch.int32), starts=dev(starts, torch.int32),
                        state_slots=dev(list(range(len(lens))) if slots is None else slots, torch.int32),
                        num_decode_tokens=n_dec, decode_tokens=dev(flat[single], torch.int32) if mixed else None,
                        prefill_tokens=dev(flat[~single], torch.int32) if mixed else None,
                        max_kv_len=max(s + n for n, s in zip(lens, starts)), row_lens=list(lens), row_starts_host=list(starts), memo={})
    b.is_decode = n_dec == len(flat)
    return b


def in_steps(lens, steps, slots, run):
    """Feed sequences of ``lens`` tokens through ``run(batch, parts)`` in ``steps`` (lists of how many tokens each sequence brings;
    what a sequence does not have any more is left out). ``parts`` are ``(sequence, first, count)`` in batch order; ``run`` returns
    one row per token. Returns each sequence's rows."""
    at, got = [0] * len(lens), [[] for _ in lens]
    for step in steps:
        parts = [(i, at[i], min(c, lens[i] - at[i])) for i, c in enumerate(step)]
        parts = [p for p in parts if p[2] > 0]
        if not parts:
            continue
        out = run(step_batch([c for _, _, c in parts], [s for _, s, _ in parts], [slots[i] for i, _, _ in parts]), parts)
        off = 0
        for i, _, c in parts:
            got[i].append(out[off : off + c])
            off += c
            at[i] += c
    assert at == list(lens), "the steps do not cover the sequences"
    return [torch.cat(g) for g in got]


def make_runner(folder, dtype, pool_tokens, slots, **kw):
    from miniserve_amd.engine.runner import ModelRunner
    from miniserve_amd.loading import load_model

    return ModelRunner(load_model(folder, dtype, DEV), kv_pool_tokens=pool_tokens, max_running=slots, **kw)


def run_schedule(runner, requests, steps):
    """``steps``: lists of ``(request, count)``; every position's logits are asked for. A request is admitted at its
    first entry and released when its last token has run. Returns request -> ``[T, vocab]``."""
    from miniserve_amd.engine.batch import StepRow

    at = {r: 0 for r in requests}
    live, got = {}, {r: [] for r in requests}
    for step in steps:
        rows, who = [], []
        for r, n in step:
            if r not in live:
                live[r] = runner.acquire()
            rows.append(StepRow(live[r], requests[r][at[r] : at[r] + n], list(range(n))))
            who += [r] * n
            at[r] += n
        logits = runner.step(rows).cpu().numpy()
        for r, row in zip(who, logits):
            got[r].append(row)
        for r, _ in step:
            if at[r] == len(requests[r]):
                runner.release(live.pop(r))
    assert not live and all(at[r] == len(requests[r]) for r in requests)
    return {r: np.stack(v) for r, v in got.items()}


def portions(total, sizes):
    out, i = [], 0
    while total > 0:
        n = min(sizes[i % len(sizes)], total)
        out.append(n)
        total -= n
        i += 1
    return out
