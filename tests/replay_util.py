"""Helpers of the tests that replay requests through the engine and compare them with a plain implementation."""
import random
from types import SimpleNamespace

import numpy as np
import torch

from gpu_util import DEV

DT = {"float32": torch.float32, "bfloat16": torch.bfloat16}
F = torch.float64


def row_errors(got, want):
    """rms of every row's error (mean taken off) in units of the row's own rms."""
    d = got - want
    d = d - d.mean(-1, keepdims=True)
    w = want - want.mean(-1, keepdims=True)
    return np.sqrt((d ** 2).mean(-1)) / np.sqrt((w ** 2).mean(-1))


def replay(model, dtype, steps, max_tokens, page_size=16, max_live=4):
    """Run ``steps`` ([(entries, end)], entries [(id, tokens, want)]) through the engine's trace replayer; returns
    {(id, position): logits row} and the replayer."""
    from pico_vllm_amd.engine.replay import TraceReplayer
    rp = TraceReplayer(model, dtype, max_tokens, page_size, max_live)
    fed, rows = {}, {}
    for k, (entries, end) in enumerate(steps):
        out = rp.run_step({"step": k, "entries": [{"id": r, "tokens": t, "want": list(w)} for r, t, w in entries], "end": list(end)})
        at = 0
        for r, t, w in entries:
            for x in w:
                rows[(r, fed.get(r, 0) + x)] = out[at]
                at += 1
            fed[r] = fed.get(r, 0) + len(t)
        for r in end:
            fed.pop(r, None)
        rp.runner.manager.check()
    return rows, rp


def requests(vocab, lengths, seed=0):
    rng = random.Random(seed)
    return {f"r{i}": [rng.randrange(vocab) for _ in range(n)] for i, n in enumerate(lengths)}


def cut(tokens, sizes, tail=0):
    """Portions of changing sizes, the last ``tail`` tokens one by one."""
    out, at, k = [], 0, 0
    body = len(tokens) - tail
    while at < body:
        n = min(sizes[k % len(sizes)], body - at)
        out.append(n)
        at += n
        k += 1
    return out + [1] * tail


def alone(reqs, portions_of):
    """Every request by itself, in the portions that ``portions_of`` gives."""
    steps = []
    for rid, toks in reqs.items():
        at = 0
        parts = portions_of(toks)
        for i, n in enumerate(parts):
            steps.append(([(rid, toks[at:at + n], range(n))], [rid] if i == len(parts) - 1 else []))
            at += n
    return steps


def roundup(n, m=64):
    return -(-n // m) * m


def mixed_steps(reqs, page, seed, max_live=3, tail=12):
    """At most ``max_live`` requests live: portions of changing size of some beside single tokens of others, now and then
    a request left out of a step.  Returns the steps and the most tokens live requests held (rounded up to pages)."""
    rng = random.Random(seed)
    waiting, live, steps = list(reqs), {}, []
    sizes = [17, 2, 40, 6, 29]
    peak = 0
    while waiting or live:
        while waiting and len(live) < max_live:
            live[waiting.pop(0)] = 0
        entries, end = [], []
        for rid in list(live):
            toks, at = reqs[rid], live[rid]
            if rng.random() < 0.2 and len(live) > 1:
                continue
            last = len(toks) - at <= tail
            n = 1 if last else min(sizes[rng.randrange(len(sizes))], len(toks) - tail - at)
            entries.append((rid, toks[at:at + n], range(n)))
            live[rid] = at + n
            if live[rid] == len(toks):
                end.append(rid)
        peak = max(peak, sum(roundup(live[r], page) for r in live))
        for rid in end:
            del live[rid]
        if entries:
            steps.append((entries, end))
    return steps, roundup(peak)


def step_ctx(new_lens, prefix_lens, slots):
    """The few arrays of a step that kernels with a state read."""
    pos, seq, cu = [], [], [0]
    for b, (n, p) in enumerate(zip(new_lens, prefix_lens)):
        pos += list(range(p, p + n))
        seq += [b] * n
        cu.append(cu[-1] + n)
    i32 = lambda v: torch.tensor(v, dtype=torch.int32, device=DEV)
    return SimpleNamespace(num_seqs=len(new_lens), num_tokens=len(pos), positions=i32(pos), token_seq=i32(seq), cu_seqlens=i32(cu),
                           state_slots=i32(slots), all_decode=max(new_lens) == 1)


def close(got, want, dtype, scale=1.0):
    tol = (2e-5 if dtype == "float32" else 2e-2) * scale * max(1.0, float(want.abs().max()))
    err = float((got.double().cpu() - want.double().cpu()).abs().max())
    assert err <= tol, (err, tol)


def rounded(t, dtype):
    """What the kernels see of a float64 tensor: its values in the storage type."""
    return t.to(DT[dtype]).to(F)


class MixerAlone:
    """One mixer with a cache of its own, fed rows of activations: pages and slots from the cache manager, in steps."""

    def __init__(self, spec, tensors, dtype, page=8, num_pages=64, max_seqs=4, max_tokens=600):
        from pico_vllm_amd.cache.manager import CacheManager
        from pico_vllm_amd.cache.storage import CacheStorage
        from pico_vllm_amd.engine.batch import BatchBuffers
        from pico_vllm_amd.parts.registry import build_part
        self.dtype, self.dt = dtype, DT[dtype]
        self.part = build_part("mixer", spec, act_dtype=self.dt)
        kept = {}
        for p in self.part.param_specs():
            t = tensors[p.name]
            assert tuple(t.shape) == tuple(p.shape), p.name
            kept[p.name] = t.to(torch.float32 if dtype == "float32" or p.role in ("norm", "f32") else torch.bfloat16)
        self.part.load(kept, torch.device(DEV), self.dt)
        spec = self.part.cache_spec()
        specs = {0: spec} if spec.kind != "several" else {(0,) + path: leaf for path, leaf in spec.leaves()}
        self.manager = CacheManager(specs, page, num_pages, max_seqs)
        self.storage = CacheStorage(self.manager, specs, self.dt, torch.device(DEV))
        self.buffers = BatchBuffers(torch.device(DEV), max_tokens, max_seqs, max_tokens // page + 1, max(1, len(self.manager.groups)))

    def step(self, entries):
        """entries: [(request, rows [n, width])], single rows first; returns the mixer's outputs, one tensor an entry."""
        from pico_vllm_amd.engine.batch import SeqStep, build_context
        entries = sorted(entries, key=lambda e: len(e[1]) != 1)
        for r, h in entries:
            try:
                self.manager.num_computed(r)
            except KeyError:
                assert self.manager.add_request(r)
            assert self.manager.grow(r, self.manager.num_computed(r) + len(h))
        self.storage.reset_state(self.manager.take_fresh_slots())
        seqs = [SeqStep(r, [0] * len(h), ()) for r, h in entries]
        ctx = build_context(seqs, self.manager, self.buffers, self.dt, 8)
        y = self.part.forward(torch.cat([h for _, h in entries]).to(DEV, self.dt).contiguous(), ctx, self.storage.layer(0))
        y = (y.float().sum(0) if y.dim() == 3 else y.float()).double().cpu()
        out, at = {}, 0
        for r, h in entries:
            self.manager.advance(r, self.manager.num_computed(r) + len(h))
            out[r] = y[at:at + len(h)]
            at += len(h)
        return out
