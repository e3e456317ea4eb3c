"""The Tubusun decoder in the engine against the plain implementation: each mechanism's kernels alone, each mixer alone and
both side by side, then whole prompts, decoding through the cache and the state, portions down to two tokens, mixed batches in
a small pool with few state slots, keys at the edges of windows, states that reach far back, long decoding, and greedy
generation through the entry point."""
import random

import numpy as np
import pytest
import torch

import plain_tubusun as P
from begasun_configs import write_model
from gpu_util import DEV
from replay_util import DT, F, MixerAlone, alone, close, cut, mixed_steps, replay, requests, rounded, roundup, row_errors, step_ctx
from tubusun_configs import CONFIGS, config, dense, left, model_dir, moe, pair, right, tensors_of

pytestmark = pytest.mark.gpu

# rms of a position's error over its logits (mean taken off), in units of the logits' own rms there
BOUND = {"float32": 3e-5, "bfloat16": 8e-2}
PAGE = {"a": 16, "b": 8, "c": 32, "d": 16, "e": 16}
# A position's error may be a few times what rounding alone does there (the largest of a few draws: itself random), and
# never less than the floor is asked of it; one position in fifty (at least one a comparison) may lie over its limit, up to
# CAP.  Where rounding may choose another expert (a gap between scores below CLOSE) only CAP is asked.  A fault of the engine
# (a wrong key, a lost state) moves whole stretches of positions.
OVER_YARDSTICK = {"float32": 5.0, "bfloat16": 3.0}
CAP = {"float32": 1e-3, "bfloat16": 2.0}
CLOSE = {"float32": 1e-6, "bfloat16": 1e-2}
YARD_DRAWS = 6

_plain = {}


class Model:
    """A configuration with its tensors, and what the plain implementation makes of requests to it."""

    def __init__(self, name, cfg=None, tensors=None):
        self.name = name
        self.cfg, self.tensors = (CONFIGS[name], tensors_of(name)) if cfg is None else (cfg, tensors)

    def logits(self, tokens):
        """(logits, the smallest gap of any layer's choice) of every position."""
        key = (self.name, tuple(tokens))
        if key not in _plain:
            margins = []
            z = P.forward(self.cfg, self.tensors, tokens, margins=margins).numpy()
            _plain[key] = z, (torch.stack(margins).min(0).values.numpy() if margins else np.full(len(tokens), np.inf))
        return _plain[key]

    def yardstick(self, tokens, dtype):
        """What rounding alone does to every position's logits, in the units of ``row_errors``.  float32: all of it in float32
        (other orders of summation than the engine's).  bfloat16: every activation between the parts rounded to 8 bits, up or
        down at random; the largest of a few draws."""
        key = (self.name, tuple(tokens), dtype)
        if key not in _plain:
            want, _ = self.logits(tokens)
            if dtype == "float32":
                draws = [P.forward(self.cfg, self.tensors, tokens, dtype=torch.float32).numpy().astype(np.float64)]
            else:
                draws = [P.forward(self.cfg, self.tensors, tokens, rounding=P.stochastic_bfloat16(100 + i)).numpy() for i in range(YARD_DRAWS)]
            _plain[key] = np.max([row_errors(d, want) for d in draws], axis=0)
        return _plain[key]

    def compare(self, dtype, rows, reqs, bound=None):
        floor = BOUND[dtype] if bound is None else bound
        errs, over, yards = [], [], []
        for (rid, pos), got in rows.items():
            toks = reqs[rid]
            want, margin = self.logits(toks)
            e = float(row_errors(got[None], want[pos][None])[0])
            assert e <= CAP[dtype], f"{self.name} {dtype}: {rid} position {pos}: {e:.3g}"
            if margin[pos] < CLOSE[dtype]:
                continue
            errs.append(e)
            yards.append(float(self.yardstick(toks, dtype)[pos]))
            limit = max(floor, OVER_YARDSTICK[dtype] * yards[-1])
            if not e <= limit:
                over.append(f"{rid} position {pos}: {e:.3g} > {limit:.3g}")
        assert len(over) <= max(1, len(errs) // 50), f"{self.name} {dtype}: {over}"
        if len(errs) >= 5:
            # the median position: half the floor, or (a model that rounding moves more) what the median yardstick says
            assert np.median(errs) <= max(floor / 2, np.median(yards)), f"{self.name} {dtype}: median {np.median(errs):.3g}"


def compare(name, dtype, rows, reqs, **kw):
    Model(name).compare(dtype, rows, reqs, **kw)


# ---------------------------------------------------------------------------------------------------------------
# each mechanism's kernels alone
# ---------------------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("T,H,slabs", [(5, 72, 1), (3, 128, 3), (2, 43, 2), (3, 4100, 2), (70, 1536, 1)])
def test_a_vector_joins_the_stream_with_a_sublayers_output(dtype, T, H, slabs):
    from pico_vllm_amd.ops import kernels
    g = torch.Generator().manual_seed(T + H)
    x, w, wn, vec = torch.randn(T, H, generator=g), torch.randn(H, generator=g), torch.randn(H, generator=g), torch.randn(H, generator=g)
    y = torch.randn(slabs, T, H, generator=g) if slabs > 1 else rounded(torch.randn(T, H, generator=g), dtype).float()
    want = x.to(F) + P.rms((y.sum(0) if slabs > 1 else y).to(F), 1e-3) * w.to(F) + vec.to(F)
    for norm in (False, True):
        resid = x.to(DEV)
        got = kernels.norm_add_norm(resid, y.to(DEV) if slabs > 1 else y.to(DEV, DT[dtype]), w.to(DEV), 1e-3, wn.to(DEV) if norm else None, 1e-5,
                                    out_dtype=DT[dtype] if norm else None, vector=vec.to(DEV))
        close(resid, want, "float32")
        if norm:
            close(got, P.rms(want, 1e-5) * wn.to(F), dtype)
    resid = x.to(DEV)
    kernels.add_vector(resid, vec.to(DEV))
    assert torch.equal(resid.cpu(), x + vec)
    table = rounded(torch.randn(9, H, generator=g), dtype)
    ids = torch.tensor([0, 8, 3, 3], dtype=torch.int32)
    close(kernels.embedding(table.to(DEV, DT[dtype]), ids.to(DEV), scale=3.0, vector=vec.to(DEV)), table[ids.long()] * 3.0 + vec.to(F), "float32")


@pytest.mark.parametrize("M,N,K", [(1, 24, 128), (8, 7, 192), (33, 256, 64), (64, 16, 136), (300, 40, 128), (5, 10, 44)])
def test_gelu_as_a_kernel_and_as_an_epilogue_and_a_product_in_pieces_with_a_bias(M, N, K):
    from pico_vllm_amd.ops import kernels
    from pico_vllm_amd.ops.linear import Linear
    g = torch.Generator().manual_seed(M + N)
    x, w = rounded(torch.randn(M, K, generator=g), "bfloat16"), rounded(torch.randn(N, K, generator=g) * 2 * K ** -0.5, "bfloat16")
    b = rounded(torch.randn(N, generator=g), "bfloat16")
    z = x @ w.T + b
    for dtype in ("float32", "bfloat16"):
        lin = Linear(w.to(DEV, DT[dtype]), b.to(DEV, DT[dtype]))
        close(lin.gelu(x.to(DEV, DT[dtype])), P.gelu_erf(z), dtype)
        y = lin.partial(x.to(DEV, DT[dtype]))
        close(y.float().sum(0) if y.dim() == 3 else y, z, dtype)
        zr = rounded(3 * z, dtype)
        close(kernels.gelu(zr.to(DEV, DT[dtype])), P.gelu_erf(zr), dtype)


def test_a_small_product_in_pieces_has_its_bias_once():
    from pico_vllm_amd.ops import kernels
    from pico_vllm_amd.ops.linear import Linear
    N, K = 256, 2048
    assert kernels.skinny_k_splits(N, K) > 1
    g = torch.Generator().manual_seed(0)
    x, w, b = (rounded(torch.randn(*s, generator=g), "bfloat16") for s in ((3, K), (N, K), (N,)))
    y = Linear(w.to(DEV, torch.bfloat16), (100 * b).to(DEV, torch.bfloat16)).partial(x.to(DEV, torch.bfloat16))
    assert y.dim() == 3
    close(y.sum(0), x @ w.T + rounded(100 * b, "bfloat16"), "float32", scale=5)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("T", [5, 90])
@pytest.mark.parametrize("H,G,dk,dv,rot", [(6, 2, 128, 64, 32), (3, 1, 24, 40, 10), (8, 2, 64, 32, 64), (1, 1, 64, 16, 0), (5, 5, 7, 1, 4), (2, 2, 32, 32, 2),
                                           (4, 2, 160, 160, 32)])
def test_rotation_unit_norm_and_store_for_few_and_many_tokens(dtype, T, H, G, dk, dv, rot):
    from pico_vllm_amd.ops import kernels
    g = torch.Generator().manual_seed(H * dk)
    page, pages = 8, 14
    cols = (H + G) * dk + G * dv
    x = rounded(3 * torch.randn(T, cols + 16 - cols % 8, generator=g, dtype=F), dtype)
    x[1] *= 2.0 ** -10                                                     # (so small that eps counts)
    pos = torch.arange(40, 40 + T, dtype=torch.int32)
    slots = torch.tensor([(t * 5) % (page * pages) if t != 4 else -1 for t in range(T)], dtype=torch.int32)
    table = None
    if rot:
        inv = torch.tensor([300.0 ** (-2.0 * i / rot) for i in range(rot // 2)], dtype=F).float()
        table = kernels.rope_table(pos.to(DEV), inv.to(DEV))
    kc = torch.zeros(pages, G, page, dk, dtype=DT[dtype], device=DEV)
    vc = torch.zeros(pages, G, dv, page, dtype=DT[dtype], device=DEV)
    for off in (0, 8):                                                     # the columns may start anywhere in a wider row
        wide = torch.cat([torch.zeros(T, off, dtype=F), x], dim=1)
        q = kernels.qk_norm_store(wide.to(DEV, DT[dtype]), off, off + H * dk, off + (H + G) * dk, H, G, G, dk, dv, 1, kernels.QK_NORM_UNIT, None, None,
                                  1e-4, table, rot, slots.to(DEV), kc, vc, pairs=True)
        want_q = P.rms(P.rotate_pairs(x[:, :H * dk].reshape(T, H, dk), pos, rot, 300.0), 1e-4)
        want_k = P.rms(P.rotate_pairs(x[:, H * dk:(H + G) * dk].reshape(T, G, dk), pos, rot, 300.0), 1e-4)
        close(q.view(T, H, dk), want_q, dtype, scale=0.5)
        for t, s in enumerate(slots.tolist()):
            if s >= 0:
                close(kc[s // page, :, s % page, :], want_k[t], dtype, scale=0.5)
                assert torch.equal(vc[s // page, :, :, s % page].double().cpu(), x[t, (H + G) * dk:cols].view(G, dv))
    empty = sorted(set(range(page * pages)) - set(slots.tolist()))
    assert all(float(kc[s // page, :, s % page, :].float().abs().max()) == 0 for s in empty)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_rotation_of_neighbours_with_weights_and_halves_without(dtype):
    """The other combinations of the launch: neighbours with weights, halves without."""
    from pico_vllm_amd.ops import kernels
    g = torch.Generator().manual_seed(3)
    H, G, dk, dv, rot = 3, 1, 32, 16, 12
    wq, wk = 1 + 0.3 * torch.randn(dk, generator=g), 1 + 0.3 * torch.randn(dk, generator=g)
    inv = torch.tensor([50.0 ** (-2.0 * i / rot) for i in range(rot // 2)], dtype=F).float()
    for T in (4, 80):
        x = rounded(torch.randn(T, (H + G) * dk + G * dv, generator=g, dtype=F), dtype)
        pos = torch.arange(T, dtype=torch.int32)
        table = kernels.rope_table(pos.to(DEV), inv.to(DEV))
        kc, vc = torch.zeros(10, G, 8, dk, dtype=DT[dtype], device=DEV), torch.zeros(10, G, dv, 8, dtype=DT[dtype], device=DEV)
        args = (0, H * dk, (H + G) * dk, H, G, G, dk, dv, 1, kernels.QK_NORM_UNIT)
        u = P.rms(x[:, :H * dk].reshape(T, H, dk), 1e-5)
        slots = torch.arange(T, dtype=torch.int32, device=DEV)
        q = kernels.qk_norm_store(x.to(DEV, DT[dtype]), *args, wq.to(DEV), wk.to(DEV), 1e-5, table, rot, slots, kc, vc, pairs=True)
        close(q.view(T, H, dk), P.rotate_pairs(u * wq.to(F), pos, rot, 50.0), dtype)
        q = kernels.qk_norm_store(x.to(DEV, DT[dtype]), *args, None, None, 1e-5, table, rot, slots, kc, vc)
        order = [i // 2 + (i % 2) * (rot // 2) for i in range(rot)] + list(range(rot, dk))      # halves as neighbours, and back
        back = [order.index(i) for i in range(dk)]
        close(q.view(T, H, dk), P.rotate_pairs(u[..., order], pos, rot, 50.0)[..., back], dtype)


ATT_SHAPES = [(6, 2, 64, 64), (3, 1, 24, 40), (8, 2, 64, 32), (20, 1, 32, 16), (2, 2, 32, 96), (5, 5, 7, 1)]      # heads, kv heads, keys, values


@pytest.mark.parametrize("H,G,dk,dv", ATT_SHAPES)
def test_attention_with_sinks_a_gate_a_head_and_a_factor_into_a_wider_buffer(H, G, dk, dv):
    """Both kernels, prompts and single tokens, in all their cuts; sinks from far below every score to so far above that
    the keys keep no weight."""
    from pico_vllm_amd.ops import kernels
    from pico_vllm_amd.ops.attention_bias_fast import FastBiasAttention, supported
    g = torch.Generator().manual_seed(H * dk + dv)
    n, page = 200, 8
    order = torch.randperm(n // page, generator=g).int()
    sinks = torch.tensor([-50.0, 3.0, 8.0, 1000.0, 0.0] * 4)[:H]
    for window in (0, 1, 37, 64):
        for lens in ([n], [130, 1], [1, 1]):               # new tokens of a sequence that ends at n, and of one that ends at 40
            ends = [n, 40][:len(lens)]
            cu = torch.tensor([0] + list(np.cumsum(lens)), dtype=torch.int32)
            T = int(cu[-1])
            q = rounded(torch.randn(T, H * dk, generator=g, dtype=F), "bfloat16")
            gate = rounded(torch.randn(T, H + 3, generator=g, dtype=F), "bfloat16")
            ks = [rounded(torch.randn(G, e, dk, generator=g, dtype=F), "bfloat16") for e in ends]
            vs = [rounded(torch.randn(G, e, dv, generator=g, dtype=F), "bfloat16") for e in ends]
            kc = torch.full((n // page + 5, G, page, dk), 9.0, dtype=F)
            vc = torch.full((n // page + 5, G, dv, page), 9.0, dtype=F)
            bt = torch.full((len(lens), n // page), -1, dtype=torch.int32)
            for b, e in enumerate(ends):
                for j in range(-(-e // page)):
                    pg = int(order[j]) if b == 0 else n // page + j
                    bt[b, j] = pg
                    m = min(page, e - j * page)
                    kc[pg, :, :m] = ks[b][:, j * page:j * page + m]
                    vc[pg, :, :, :m] = vs[b][:, j * page:j * page + m].transpose(1, 2)
            pos = torch.cat([torch.arange(e - m, e) for e, m in zip(ends, lens)]).int()
            seq = torch.tensor(sum([[b] * m for b, m in enumerate(lens)], []), dtype=torch.int32)
            want = torch.zeros(T, H * dv, dtype=F)
            for t in range(T):
                b, p = int(seq[t]), int(pos[t])
                lo = max(0, p - window + 1) if window else 0
                for h in range(H):
                    s = (ks[b][h // (H // G), lo:p + 1] @ q[t, h * dk:(h + 1) * dk]) * 0.3
                    a = P.sink_softmax(s[None], torch.ones(1, len(s), dtype=torch.bool), sinks[h].to(F))[0]
                    want[t, h * dv:(h + 1) * dv] = (a @ vs[b][h // (H // G), lo:p + 1]) * torch.sigmoid(gate[t, h]) * 0.7
            dev = lambda t, dt: t.to(DEV, DT[dt]).contiguous()
            i32 = lambda t: t.to(DEV).contiguous()
            for dt in ("float32", "bfloat16"):
                wide = torch.full((T, H * dv + 12), 5.0, dtype=DT[dt], device=DEV)
                kernels.attn_bias_plain(dev(q, dt), dev(kc, dt), dev(vc, dt), i32(bt), i32(pos), i32(seq), H, G, dk, dv, 0.3, window,
                                        gate=dev(gate, dt), gate_heads=True, sinks=sinks.to(DEV), out=wide[:, 4:4 + H * dv], out_scale=0.7)
                close(wide[:, 4:4 + H * dv], want, dt)
                assert float((wide[:, :4].float() - 5).abs().max()) == 0 and float((wide[:, 4 + H * dv:].float() - 5).abs().max()) == 0
            if supported(dk, dv):
                fast = FastBiasAttention(H, G, dk, dv, 0.3, window, gated=True, gate_heads=True, sink=True, out_scale=0.7)
                fast.sinks = sinks.to(DEV)
                assert (fast.tuned is not None) == (dk == dv)
                if fast.tuned is not None:                 # the prompt kernel for keys and values of one size, in its shapes
                    ctx_lens = torch.tensor(ends, dtype=torch.int32, device=DEV)
                    for teams in (1, 2, 3, 4, 6):
                        wide = torch.full((T, H * dv + 12), 5.0, dtype=torch.bfloat16, device=DEV)
                        fast.tuned.prefill(dev(q, "bfloat16"), dev(kc, "bfloat16"), dev(vc, "bfloat16"), i32(bt), i32(cu), ctx_lens, len(lens), 0.3,
                                           teams=teams, out=wide[:, 4:4 + H * dv], finish=(True, fast.sinks, dev(gate, "bfloat16"), 0.7))
                        close(wide[:, 4:4 + H * dv], want, "bfloat16")
                        assert float((wide[:, :4].float() - 5).abs().max()) == 0 and float((wide[:, 4 + H * dv:].float() - 5).abs().max()) == 0
                for split, chunks in ((True, 1), (True, 3), (False, 1)):
                    wide = torch.full((T, H * dv + 12), 5.0, dtype=torch.bfloat16, device=DEV)
                    fast.run(dev(q, "bfloat16"), dev(kc, "bfloat16"), dev(vc, "bfloat16"), i32(bt), i32(cu), i32(pos), len(lens), split=split,
                             chunks=chunks, gate=dev(gate, "bfloat16"), out=wide[:, 4:4 + H * dv])
                    close(wide[:, 4:4 + H * dv], want, "bfloat16")
                    assert float((wide[:, :4].float() - 5).abs().max()) == 0 and float((wide[:, 4 + H * dv:].float() - 5).abs().max()) == 0


GLA_SHAPES = [(2, 64, 64), (3, 9, 11), (1, 1, 3), (4, 32, 80), (2, 160, 96), (2, 5, 1), (3, 96, 32), (2, 128, 128), (1, 256, 64),
              (3, 40, 24), (2, 8, 136), (1, 72, 200)]      # heads, keys, values


def lightning_rows(H, dk, dv, T, seed, dtype):
    g = torch.Generator().manual_seed(seed)
    cols = 2 * H * dk + 2 * H * dv
    return rounded(torch.randn(T, cols, generator=g, dtype=F), dtype)


def lightning_plain(y, H, dk, dv, decay, S0=None):
    T = len(y)
    q, k = (P.silu(y[:, i * H * dk:(i + 1) * H * dk]).view(T, H, dk) for i in (0, 1))
    v = P.silu(y[:, 2 * H * dk:2 * H * dk + H * dv]).view(T, H, dv)
    return P.decayed_sums(q, k, v, decay, S0)


def lightning_run(y, H, dk, dv, decay, ctx, state, dtype, chunk=0):
    from pico_vllm_amd.ops import kernels
    return kernels.gla_scan(y.to(DEV, DT[dtype]), 0, H * dk, 2 * H * dk, None, ctx.cu_seqlens, ctx.state_slots, state, ctx.num_seqs, H, dk, dv, 1.0,
                            chunk=chunk, head_decay=torch.tensor(decay, device=DEV), silu=True)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("H,dk,dv", GLA_SHAPES)
def test_the_recurrence_whole_in_portions_and_in_chunks(dtype, H, dk, dv):
    T = 150
    decay = [float(d) for d in torch.tensor([0.4, 0.97, 1.0, 0.85][:H])]
    y = lightning_rows(H, dk, dv, T, H + dk, dtype)
    s0 = torch.randn(H, dk, dv, generator=torch.Generator().manual_seed(dk))
    want, last = lightning_plain(y, H, dk, dv, decay, s0.to(F))
    results = []
    for portions in ([T], [2, 70, 1, 50, 27]):
        state = torch.full((4, H, dk, dv), 3.0, device=DEV)
        state[2] = s0.to(DEV)
        at, outs = 0, []
        for n in portions:
            outs.append(lightning_run(y[at:at + n], H, dk, dv, decay, step_ctx([n], [at], [2]), state, dtype))
            at += n
        got = torch.cat(outs).view(T, H, dv)
        results.append((got, state.clone()))
        close(got, want, "float32", scale=2)                   # (float32 behind the stored operands in both engines)
        close(state[2], last, "float32", scale=2)
        assert float((state[[0, 1, 3]] - 3).abs().max()) == 0
    assert torch.equal(results[0][0], results[1][0]) and torch.equal(results[0][1], results[1][1])       # the cut changes no bit
    # chunks side by side, several sequences of unequal length, one going on from a state
    lens, slots = [64, 1, 0, 65, 20], [1, 0, 4, 2, 3]
    state = torch.zeros(6, H, dk, dv, device=DEV)
    state[2] = s0.to(DEV)
    got = lightning_run(y, H, dk, dv, decay, step_ctx(lens, [0, 0, 0, 7, 0], slots), state, dtype, chunk=64).view(T, H, dv)
    at = 0
    for n, slot in zip(lens, slots):
        if n:
            o, S = lightning_plain(y[at:at + n], H, dk, dv, decay, s0.to(F) if slot == 2 else None)
            close(got[at:at + n], o, "float32", scale=2)
            close(state[slot], S, "float32", scale=2)
        at += n
    assert float(state[[4, 5]].abs().max()) == 0


@pytest.mark.parametrize("chunk", [0, 64])
def test_a_first_token_is_kept_for_hundreds_of_tokens_or_forgotten(chunk):
    """Zero keys behind the first token: its outer product, decayed, is all that later queries read."""
    H, d, T = 2, 16, 700
    decay = [0.9995, 0.5]
    y = torch.zeros(T, 4 * H * d, dtype=F)
    y[:, :H * d] = 2.0
    y[0] = 2.0
    state = torch.zeros(2, H, d, d, device=DEV)
    outs = [lightning_run(y[a:b], H, d, d, decay, step_ctx([b - a], [a], [1]), state, "bfloat16", chunk=chunk) for a, b in ((0, 300), (300, 699), (699, T))]
    one = float(P.silu(torch.tensor(2.0, dtype=F)))
    got = torch.cat(outs).view(T, H, d).double().cpu()
    n = torch.arange(T, dtype=F)
    for h in range(H):
        want = d * one ** 3 * torch.tensor(decay[h]).float().double() ** n
        assert float(((got[:, h, 0] - want).abs() / want.clamp_min(1e-25)).max()) < 1e-3
    assert float(got[-1, 0, 0]) > 0.5 * float(got[0, 0, 0])


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("T,N", [(3, 22), (1, 257), (5, 2049), (2, 8192), (90, 1536), (4, 1)])
def test_the_norm_over_all_heads_and_its_gate(dtype, T, N):
    from pico_vllm_amd.ops import kernels
    g = torch.Generator().manual_seed(N)
    o, w = torch.randn(T, N, generator=g) * 3, 1 + 0.3 * torch.randn(N, generator=g)
    x = rounded(torch.randn(T, N + 9, generator=g, dtype=F), dtype)
    want = P.rms(o.to(F), 1e-2) * w.to(F) * torch.sigmoid(x[:, 5:5 + N])
    close(kernels.gated_row_norm(o.to(DEV), x.to(DEV, DT[dtype]), 5, w.to(DEV), 1e-2), want, dtype)
    wide = torch.full((T, N + 16), 5.0, dtype=DT[dtype], device=DEV)
    kernels.gated_row_norm(o.to(DEV), x.to(DEV, DT[dtype]), 5, w.to(DEV), 1e-2, out=wide[:, 8:8 + N])
    close(wide[:, 8:8 + N], want, dtype)
    assert float((wide[:, :8].float() - 5).abs().max()) == 0 and float((wide[:, 8 + N:].float() - 5).abs().max()) == 0


@pytest.mark.parametrize("H,G,dk,dv,rot,lh,ldk,ldv", [(6, 2, 64, 64, 32, 3, 64, 128), (3, 1, 24, 40, 10, 2, 9, 11), (20, 1, 32, 16, 0, 1, 200, 70), (2, 2, 7, 1, 6, 4, 1, 1),
                                                      (4, 2, 160, 96, 160, 2, 130, 65)])
def test_both_sides_of_a_step_of_single_tokens_in_one_launch(H, G, dk, dv, rot, lh, ldk, ldv):
    from pico_vllm_amd.ops import kernels
    g = torch.Generator().manual_seed(H * dk)
    T, page, pages = 5, 8, 6
    left_cols = (H + G) * dk + G * dv
    at = -(-left_cols // 8) * 8
    x = rounded(2 * torch.randn(T, at + 2 * lh * (ldk + ldv), generator=g, dtype=F), "bfloat16")
    xd = x.to(DEV, torch.bfloat16)
    i32 = lambda *v: torch.tensor(v, dtype=torch.int32, device=DEV)
    slots, state_slots = i32(5, 11, -1, 47, 0), i32(2, 0, 3, 5, 1)
    decay = [0.3, 0.99, 1.0, 0.8][:lh]
    table = kernels.rope_table(i32(9, 70, 0, 300, 41), torch.tensor([100.0 ** (-2.0 * i / rot) for i in range(rot // 2)]).to(DEV)) if rot else None
    caches = [(torch.zeros(pages, G, page, dk, dtype=torch.bfloat16, device=DEV), torch.zeros(pages, G, dv, page, dtype=torch.bfloat16, device=DEV)) for _ in range(2)]
    s0 = torch.randn(5, lh, ldk, ldv, generator=g)           # the slot 5 of the fourth token does not exist
    state = s0.to(DEV)
    q, o = kernels.pair_open(xd, (0, H * dk, (H + G) * dk, H, G, dk, dv), 1e-3, table, rot, slots, *caches[0],
                             (at, at + lh * ldk, at + 2 * lh * ldk, lh, ldk, ldv), state_slots, torch.tensor(decay, device=DEV), state)
    q2 = kernels.qk_norm_store(xd, 0, H * dk, (H + G) * dk, H, G, G, dk, dv, 1, kernels.QK_NORM_UNIT, None, None, 1e-3, table, rot, slots, *caches[1], pairs=True)
    close(q, q2, "bfloat16", scale=0.3)
    close(caches[0][0], caches[1][0].double(), "bfloat16", scale=0.3)
    assert torch.equal(caches[0][1], caches[1][1])
    for t, slot in enumerate(state_slots.tolist()):
        if slot < 5:
            want, last = lightning_plain(x[t:t + 1, at:], lh, ldk, ldv, [float(d) for d in torch.tensor(decay)], s0[slot].to(F))
            close(o[t].view(lh, ldv), want[0], "float32", scale=2)
            close(state[slot], last, "float32", scale=2)
    assert torch.equal(state[4].cpu(), s0[4])


@pytest.mark.parametrize("T,H,dv,pieces,N", [(1, 6, 64, 7, 384), (5, 3, 40, 2, 22), (9, 20, 16, 64, 4096), (2, 1, 256, 33, 1), (3, 5, 1, 3, 1025)])
def test_pieces_put_together_beside_the_norm_over_all_heads(T, H, dv, pieces, N):
    from pico_vllm_amd.ops import kernels
    g = torch.Generator().manual_seed(T * H + N)
    po, mx, l = torch.randn(pieces, T * H, dv, generator=g), 5 * torch.randn(pieces, T * H, generator=g), 1 + torch.rand(pieces, T * H, generator=g)
    if pieces > 2:
        mx[1, ::2], l[1, ::2], po[1, ::2] = -float("inf"), 0.0, 0.0      # a piece in which a column saw no key
    sinks = torch.tensor([1.0, 500.0, -30.0, 4.0] * 5)[:H]
    gate, lgate = (rounded(torch.randn(T, n + 5, generator=g, dtype=F), "bfloat16") for n in (H, N))
    o, w = torch.randn(T, N, generator=g), 1 + 0.3 * torch.randn(N, generator=g)
    out, lout = (torch.full((T, n + 8), 5.0, dtype=torch.bfloat16, device=DEV) for n in (H * dv, N))
    bf = lambda t: t.to(DEV, torch.bfloat16)
    kernels.pair_close(po.to(DEV), torch.stack([mx, l], -1).to(DEV), sinks.to(DEV), bf(gate)[:, 2:], 0.7, out[:, 3:3 + H * dv], o.to(DEV), bf(lgate)[:, 1:],
                       w.to(DEV), 1e-3, lout[:, 8:])
    e = torch.exp(mx.to(F))
    den = (e * l.to(F)).sum(0).view(T, H) + torch.exp(sinks.to(F))
    want = (e[..., None] * po.to(F)).sum(0).view(T, H, dv) / den[..., None] * torch.sigmoid(gate[:, 2:2 + H])[..., None] * 0.7
    close(out[:, 3:3 + H * dv], want.reshape(T, H * dv), "bfloat16")
    close(lout[:, 8:], P.rms(o.to(F), 1e-3) * w.to(F) * torch.sigmoid(lgate[:, 1:1 + N]), "bfloat16")
    assert all(float((v.float() - 5).abs().max()) == 0 for v in (out[:, :3], out[:, 3 + H * dv:], lout[:, :8]))


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("E,top,groups,keep,D", [(8, 2, 4, 2, 64), (16, 4, 4, 3, 128), (9, 3, 3, 2, 72), (5, 1, 1, 1, 44), (4, 2, 4, 2, 40), (160, 8, 8, 3, 96),
                                                 (12, 5, 2, 2, 50), (256, 16, 64, 5, 64), (130, 6, 130, 9, 32)])
def test_the_choice_of_experts_by_groups(dtype, E, top, groups, keep, D):
    from pico_vllm_amd.ops import kernels
    g = torch.Generator().manual_seed(E + top)
    T = 150
    x, w = rounded(torch.randn(T, D, generator=g, dtype=F), dtype), (torch.randn(E, D, generator=g) * 2 * D ** -0.5).float()
    r = {"experts": E, "top": top, "groups": {"count": groups, "keep": keep}}
    want_e, want_w = P.route(x, w.to(F), r)
    far = P.route_margin(x, w.to(F), r) > 1e-6
    assert int(far.sum()) > T // 2
    best = P.route(x, w.to(F), {"experts": E, "top": top})[0].sort(-1).values
    assert keep == groups or groups == E or not torch.equal(best, want_e.sort(-1).values)             # the groups matter
    outs = []
    for n in (T, 60, 1):                                     # many tokens; few: logits and choice in one launch
        e, s = kernels.moe_router_groups(x[:n].to(DEV, DT[dtype]), w.to(DEV), groups, keep, top)
        outs.append((e, s))
        ok = far[:n]
        assert torch.equal(e.cpu().long()[ok], want_e[:n][ok])
        assert float((s.double().cpu() - want_w[:n])[ok].abs().max()) < 1e-5
    for e, s in outs[1:]:
        assert torch.equal(e, outs[0][0][:len(e)]) and torch.equal(s, outs[0][1][:len(e)])


def test_among_equal_experts_and_groups_the_first_is_chosen():
    from pico_vllm_amd.ops import kernels
    x = torch.ones(1, 4, device=DEV)
    for z, groups, keep, top, want in (([1.0] * 8, 4, 2, 3, [0, 1, 2]), ([0.0, 2.0, 2.0, 0.0, 2.0, 0.0], 3, 2, 3, [1, 2, 0]), ([-200.0] * 6, 3, 1, 2, [0, 1]),
                                       ([200.0] * 6, 3, 1, 2, [0, 1]), ([5.0, -300.0, 1.0, 4.9, -9.0, 3.0], 3, 1, 2, [3, 2])):
        w = torch.zeros(len(z), 4)
        w[:, 0] = torch.tensor(z)
        for T in (1, 70):
            e, _ = kernels.moe_router_groups(x.repeat(T, 1), w.to(DEV), groups, keep, top)
            assert e.tolist() == [want] * T, (z, e[0])


@pytest.mark.parametrize("T,E,top,F_,D", [(3, 5, 2, 24, 40), (1, 8, 4, 64, 128), (40, 8, 2, 40, 72), (300, 6, 3, 96, 64), (7, 9, 3, 21, 44), (33, 4, 1, 16, 24)])
def test_experts_with_the_weight_on_their_output(T, E, top, F_, D):
    """Gate and up of several times the limit; weights of the inputs' size, so that a weight on the input would show."""
    from pico_vllm_amd.ops import kernels
    g = torch.Generator().manual_seed(T + E)
    x = rounded(torch.randn(T, D, generator=g, dtype=F), "bfloat16")
    gu = rounded(torch.randn(E, 2 * F_, D, generator=g, dtype=F) * 2 * D ** -0.5, "bfloat16")
    dn = rounded(torch.randn(E, D, F_, generator=g, dtype=F) * F_ ** -0.5, "bfloat16")
    experts = torch.stack([torch.randperm(E, generator=g)[:top] for _ in range(T)]).int()
    weights = 0.1 + 0.9 * torch.rand(T, top, generator=g)
    want = torch.zeros(T, D, dtype=F)
    for t in range(T):
        for e, w in zip(experts[t].tolist(), weights[t].to(F)):
            want[t] += w * P.expert(x[t:t + 1], gu[e, :F_], gu[e, F_:], dn[e], 0.8)[0]
    args = lambda dt: [v.to(DEV, DT[dt]) for v in (x, gu, dn)] + [experts.to(DEV), weights.to(DEV), 0.8, 1.702]
    for dt in ("float32", "bfloat16"):
        close(kernels.moe_experts_plain(*args(dt), mode=kernels.MOE_CLIPPED_OUT), want, dt)
    if kernels.moe_fast_ok(*args("bfloat16")[:3]):
        for grouped in (False, True):
            y = kernels.moe_experts(*args("bfloat16"), grouped=grouped, mode=kernels.MOE_CLIPPED_OUT)
            close(y.sum(0) if y.dim() == 3 else y, want, "bfloat16")


# ---------------------------------------------------------------------------------------------------------------
# each mixer alone and both together, with pages and slots from the cache manager
# ---------------------------------------------------------------------------------------------------------------
def mixer_case(side, m, width, seed):
    """(part, its tensors by the part's names, the plain function) of one side of a layer or of both."""
    from pico_vllm_amd.config.tubusun import TubusunConfig, _mixer_spec
    whole = {"left": (m, right(1, 8, 8)), "right": (left(1, 1, 8, 8), m)}.get(side)
    cfg = config(8, width, [(pair(*whole) if whole else m, None)])
    pre = "l0.mix." + (side + "." if side != "both" else "")
    t = {n[len(pre):]: v for n, v in P.random_model(cfg, seed).items() if n.startswith(pre)}
    c = TubusunConfig.from_dict(cfg)
    spec = _mixer_spec(c, c.layers[0].mixer)
    if side != "both":
        spec = spec.params[side]
        f = {"left": P.attention, "right": P.lightning}[side]
        return spec, t, lambda h, w: f(h, {k: v.to(F) for k, v in w.items()}, m, 1e-5) @ w["o"].to(F).T
    return spec, t, lambda h, w: P.parallel(h, {k: v.to(F) for k, v in w.items()}, m, 1e-5)


MIXER_CASES = {
    "attention": ("left", left(3, 1, 24, 40, window=21, rot_dims=10), 72), "attention without window": ("left", left(4, 2, 64, 64, rot_dims=32), 128),
    "attention on matrix cores": ("left", left(8, 2, 64, 32, window=48, rot_dims=64), 96), "attention to itself alone": ("left", left(2, 1, 32, 32, window=1), 64),
    "attention of many heads": ("left", left(20, 1, 32, 16, window=70, rot_dims=6), 64),
    "lightning": ("right", right(3, 9, 11), 72), "lightning of one head": ("right", right(1, 64, 64), 128), "lightning wide": ("right", right(2, 160, 96), 64),
    "both": ("both", pair(left(3, 1, 24, 40, window=21, rot_dims=10), right(3, 9, 11), 0.6, 1.5), 72),
    "both on matrix cores": ("both", pair(left(6, 2, 64, 64, window=48, rot_dims=16), right(4, 64, 32), -0.7, 2.0), 128)}


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("case", sorted(MIXER_CASES))
def test_a_mixer_alone_in_portions_and_mixed_batches(case, dtype):
    side, m, width = MIXER_CASES[case]
    spec, t, plain = mixer_case(side, m, width, seed=len(case))
    g = torch.Generator().manual_seed(7)
    lens = {"r0": 190, "r1": 43, "r2": 96}
    rows = {r: rounded(torch.randn(n, width, generator=g, dtype=F), dtype) for r, n in lens.items()}
    want = {r: plain(h, t) for r, h in rows.items()}
    mx = MixerAlone(spec, t, dtype)
    steps = [{"r0": 150}, {"r0": 2, "r1": 17}, {"r0": 1, "r1": 1, "r2": 70}, {"r0": 1, "r1": 1, "r2": 1}, {"r1": 5, "r2": 2}, {"r0": 20, "r2": 1}]
    at = dict.fromkeys(lens, 0)
    got = {r: [] for r in lens}
    while any(at[r] < n for r, n in lens.items()):
        step = steps.pop(0) if steps else {r: 1 for r in lens}
        entries = [(r, rows[r][at[r]:at[r] + min(n, lens[r] - at[r])]) for r, n in step.items() if at[r] < lens[r]]
        out = mx.step(entries)
        for r, h in entries:
            got[r].append(out[r])
            at[r] += len(h)
    for r in lens:
        y = torch.cat(got[r])
        scale = float(want[r].pow(2).mean().sqrt())
        err = (y - want[r]).pow(2).mean(-1).sqrt() / scale
        assert float(err.max()) < (3e-5 if dtype == "float32" else 6e-2), (r, int(err.argmax()), float(err.max()))
        assert float(err.median()) < (5e-6 if dtype == "float32" else 1.5e-2), (r, float(err.median()))
    if dtype == "float32":                                # whole at once: the same bits
        again = MixerAlone(spec, t, dtype).step([("r0", rows["r0"])])["r0"]
        assert torch.equal(again, torch.cat(got["r0"]))


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("window", [0, 48])
@pytest.mark.parametrize("H,G,dk,dv", [(3, 1, 26, 40), (4, 2, 64, 64), (8, 2, 64, 32)])
def test_one_key_that_stands_out(H, G, dk, dv, window, dtype):
    """Weights under which a row that asks for mark x fits the one row that carries mark x and nothing else: at the first
    position, on both sides of page borders, just inside and just outside the window, hundreds of tokens back without one;
    asked for by single tokens and inside portions.  What comes out is that row's value if the window reaches it."""
    rot, width = 8, 96
    asked = ({47: 0, 48: 0, 60: 13, 61: 13, 130: 128, 131: 84, 132: 84, 300: 253, 301: 253, 302: 255, 303: 256, 420: 373, 421: 373, 448: 447} if window else
             {300: 0, 301: 7, 302: 8, 303: 255, 304: 256, 420: 63, 421: 64, 448: 1})
    n = len(asked)
    m = left(H, G, dk, dv, window=window, rot_dims=rot, base=100.0, scale=60.0 / dk)
    spec, t, plain = mixer_case("left", m, width, seed=3)
    t = {k: v.clone() for k, v in t.items()}
    for k in ("q", "k", "v", "g"):
        t[k][:, :2 * n] = 0                               # columns 0 .. n - 1 ask for marks, n .. 2 n - 1 carry them
    for x in range(n):
        for name, heads, col in (("q", H, x), ("k", G, n + x)):
            for h in range(heads):                        # an entry a mark of every head, behind what is turned
                t[name][h * dk + rot + x] = 0
                t[name][h * dk + rot + x, col] = 1
    g = torch.Generator().manual_seed(11)
    h = torch.randn(450, width, generator=g, dtype=F)
    h[:, :2 * n] = 0
    for x, (i, j) in enumerate(asked.items()):
        h[i, x] = h[j, n + x] = 60.0
    h = rounded(h, dtype)
    want = plain(h, t)
    rms_of = lambda v: float(v.pow(2).mean().sqrt())
    from plain_tubusun import attention as plain_attention
    other = lambda size: plain_attention(h, {k: v.to(F) for k, v in t.items()}, dict(m, mask={"size": size}), 1e-5) @ t["o"].to(F).T
    if window:                                            # a window that is one token off would show, on either side
        less, more = other(window - 1), other(window + 1)
        for i, j in asked.items():
            if i - j == window - 1:
                assert rms_of(want[i] - less[i]) > 0.3 * rms_of(want[i])
            if i - j == window:
                assert rms_of(want[i] - more[i]) > 0.3 * rms_of(want[i])
        assert sum(i - j == window for i, j in asked.items()) >= 5 and sum(i - j == window - 1 for i, j in asked.items()) >= 5
    else:
        for i, j in asked.items():                        # leaving the key out would show
            without = plain(torch.cat([h[:j], h[j + 1:i + 1]]), t)[-1]
            assert rms_of(want[i] - without) > 0.3 * rms_of(want[i])
    for cuts in ([(0, 300)] + [(i, i + 1) for i in range(300, 305)] + [(305, 421), (421, 422), (422, 448), (448, 450)],
                 [(0, 40), (40, 42), (42, 48), (48, 49), (49, 61), (61, 62), (62, 128)] + [(i, i + 1) for i in range(128, 134)] + [(134, 450)]):
        mx = MixerAlone(spec, t, dtype)
        got = torch.cat([mx.step([("r", h[a:b])])["r"] for a, b in cuts])
        for i in asked:
            assert rms_of(got[i] - want[i]) < (3e-5 if dtype == "float32" else 3e-2) * rms_of(want[i]), i


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_the_first_tokens_and_their_sinks(dtype):
    """With few keys a sink takes much of the weight: left out or scaled it would show at the first positions."""
    m, width = left(4, 2, 64, 64, window=6, rot_dims=8, scale=0.01), 64
    spec, t, plain = mixer_case("left", m, width, seed=5)
    t["sink"] = torch.tensor([2.0, 0.5, 3.0, 1.0]).to(torch.bfloat16)
    h = rounded(torch.randn(40, width, generator=torch.Generator().manual_seed(1), dtype=F), dtype)
    want = plain(h, t)
    rms_of = lambda v: v.pow(2).mean(-1).sqrt()
    for changed in (torch.full((4,), -1e9), t["sink"] * 0.01, torch.zeros(4)):
        assert float((rms_of(want - plain(h, dict(t, sink=changed))) / rms_of(want)).min()) > 0.1
    for cuts in ([(0, 40)], [(i, i + 1) for i in range(40)], [(0, 2), (2, 4), (4, 5), (5, 7), (7, 40)]):
        mx = MixerAlone(spec, t, dtype)
        got = torch.cat([mx.step([("r", h[a:b])])["r"] for a, b in cuts])
        assert float((rms_of(got - want) / rms_of(want)).max()) < (3e-5 if dtype == "float32" else 3e-2)


# ---------------------------------------------------------------------------------------------------------------
# whole models through the engine
# ---------------------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_the_stream_after_every_layer_run(name, dtype):
    """Every run of every layer, the vector of a pass taken off again where the layer's last launch has added it."""
    from pico_vllm_amd.engine.batch import SeqStep
    from pico_vllm_amd.engine.step import ModelRunner
    from pico_vllm_amd.parts.model import load_model
    from pico_vllm_amd.parts.norm import STREAM_VECTOR
    toks = requests(CONFIGS[name]["vocab"], [29], seed=3)["r0"]
    m = load_model(model_dir(name), dtype)
    seen = []
    for blk in m.layers:
        def forward(resid, pending, ctx, cache, blk=blk):
            vec = ctx.shared.get(STREAM_VECTOR)
            r, p = type(blk).forward(blk, resid, pending, ctx, cache)
            assert p is None and STREAM_VECTOR not in ctx.shared
            seen.append(r - vec if vec is not None else r.clone())
            return r, p
        blk.forward = forward
    run = ModelRunner(m, 8, 16, 2, 64, 64)
    run.manager.add_request("x")
    run.manager.grow("x", len(toks))
    run.step([SeqStep("x", toks, [28])])
    want, drawn = [], []
    P.forward(CONFIGS[name], tensors_of(name), toks, trace=want)
    P.forward(CONFIGS[name], tensors_of(name), toks, trace=drawn, rounding=P.stochastic_bfloat16(1))
    assert len(seen) == len(want)
    for a, b, r in zip(seen, want, drawn):
        off = lambda v: float(((v.double().cpu() - b).pow(2).mean(-1).sqrt() / b.pow(2).mean(-1).sqrt()).median())
        assert off(a) < (2e-6 if dtype == "float32" else 1.5 * off(r))


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_whole_prompts_and_token_by_token_from_the_first_token(name, dtype):
    reqs = requests(CONFIGS[name]["vocab"], [150, 1, 37], seed=1)
    rows, _ = replay(model_dir(name), dtype, alone(reqs, lambda t: [len(t)]), roundup(150), PAGE[name])
    compare(name, dtype, rows, reqs)
    one = {"r2": reqs["r2"]}
    rows1, _ = replay(model_dir(name), dtype, alone(one, lambda t: [1] * len(t)), roundup(37), PAGE[name])
    compare(name, dtype, rows1, one)
    if dtype == "float32":
        for key, row in rows1.items():
            assert np.array_equal(row, rows[key])         # decoded through cache and state: the same bits as the prompt


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_portions_of_many_sizes_down_to_two_tokens_then_decoding(name, dtype):
    reqs = requests(CONFIGS[name]["vocab"], [190], seed=2)
    rows, _ = replay(model_dir(name), dtype, alone(reqs, lambda t: cut(t, [2, 33, 5, 70, 3, 16], tail=60)), roundup(190), PAGE[name])
    compare(name, dtype, rows, reqs)
    if dtype == "float32":
        whole, _ = replay(model_dir(name), dtype, alone(reqs, lambda t: [len(t)]), roundup(190), PAGE[name])
        for key, row in rows.items():
            assert np.array_equal(row, whole[key])


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_mixed_batches_in_a_pool_that_holds_what_is_live(name, dtype):
    """Seven unequal requests, at most three live, in a pool that holds just the live ones and with three state slots:
    pages and slots are used again; each request against itself alone."""
    lengths = [70, 33, 120, 9, 64, 47, 101]
    reqs = requests(CONFIGS[name]["vocab"], lengths, seed=4)
    steps, peak = mixed_steps(reqs, PAGE[name], seed=7)
    rows, rp = replay(model_dir(name), dtype, steps, peak, PAGE[name], max_live=3)
    compare(name, dtype, rows, reqs)
    m = rp.runner.manager
    assert all(g.pool.num_free == g.pool.num_pages for g in m.groups) and m.slots.num_free == 3      # all given back
    if dtype == "float32":
        solo, _ = replay(model_dir(name), dtype, alone(reqs, lambda t: [len(t)]), roundup(max(lengths)), PAGE[name])
        for key, row in rows.items():
            assert np.array_equal(row, solo[key])               # what else is in the batch changes no bit


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_long_prompts_cut_into_chunks_and_decoding_behind_them(dtype):
    """Portions long enough that the bfloat16 engine cuts the recurrence into chunks and the attention takes its prompt
    shapes, several of them in a step."""
    reqs = requests(CONFIGS["b"]["vocab"], [420, 300], seed=8)
    steps = [([("r0", reqs["r0"][:130], range(130))], []), ([("r0", reqs["r0"][130:390], range(260)), ("r1", reqs["r1"][:275], range(275))], [])]
    at = {"r0": 390, "r1": 275}
    for k in range(30):
        entries = [(r, reqs[r][at[r] + k:at[r] + k + 1], [0]) for r in at if at[r] + k < len(reqs[r])]
        steps.append((entries, [r for r, _, _ in entries if at[r] + k + 1 == len(reqs[r])]))
    rows, _ = replay(model_dir("b"), dtype, steps, roundup(420) + roundup(300), 16)
    compare("b", dtype, rows, reqs)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_long_decoding(dtype):
    reqs = requests(CONFIGS["b"]["vocab"], [330], seed=6)
    rows, _ = replay(model_dir("b"), dtype, alone(reqs, lambda t: cut(t, [30], tail=300)), roundup(330), PAGE["b"])
    compare("b", dtype, rows, reqs)


def test_sharp_attention_at_a_windows_edge_in_every_pass_of_a_loop():
    """Scales so large that every query's softmax sits on very few keys, some of them the last that the window reaches: a
    key read from a wrong place, or one too many, shows in the logits."""
    cfg = config(64, 64, [(pair(left(4, 1, 16, 16, window=40, rot_dims=4, base=50.0, scale=1.2), right(1, 4, 4), 1.0, 0.1), dense(32)),
                          (pair(left(2, 2, 12, 8, rot_dims=12, base=50.0, scale=1.2), right(1, 4, 4), 1.0, 0.1), moe(16, 4, 2, 1.0))], loop=(0, 2, 2), cap=10.0)
    t = P.random_model(cfg, 5)
    for k in t:
        if k.endswith("sink"):
            t[k] -= 6
    toks = requests(64, [400], seed=9)["r0"]
    want = P.forward(cfg, t, toks).numpy()
    for size in (39, 41):                                       # a window of one less or more is far beyond the bound
        off = dict(cfg, layers=[dict(cfg["layers"][0], mixer=dict(cfg["layers"][0]["mixer"], left=dict(cfg["layers"][0]["mixer"]["left"], mask={"size": size}))),
                                cfg["layers"][1]])
        assert float(np.quantile(row_errors(P.forward(off, t, toks).numpy(), want)[50:], 0.2)) > 1e-3
    d = write_model(cfg, t, "tubusun_edge_")
    reqs = {"r0": toks}
    for portions in (lambda x: [len(x)], lambda x: cut(x, [2, 61, 8, 130], tail=60)):
        rows, _ = replay(d, "float32", alone(reqs, portions), roundup(400), 8)
        Model("edge", cfg, t).compare("float32", rows, reqs, bound=1e-4)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("graphs", [False, True])
@pytest.mark.parametrize("name", ["b", "d"])
def test_greedy_generation_through_the_entry_point(name, dtype, graphs):
    from pico_vllm_amd import LLM, SamplingParams
    vocab = CONFIGS[name]["vocab"]
    prompts = [[t % vocab for t in p] for p in ([5, 17, 3, 200, 41], [9] * 19, [77, 2], list(range(60, 130)), [1], [250, 3, 3, 8, 100, 100])]
    llm = LLM(model=model_dir(name), dtype=dtype, block_size=8, num_gpu_blocks=48, max_seq_len=160, max_num_seqs=3,
              max_num_batched_tokens=24, use_cuda_graph=graphs, max_batch_size=4)
    outs = llm.generate(prompts, SamplingParams(max_new_tokens=12, temperature=0.0, ignore_eos=True))
    cfg, t = CONFIGS[name], tensors_of(name)
    close_calls = 0
    for p, o in zip(prompts, outs):
        assert len(o.token_ids) == 12
        toks = list(p)
        for tok in o.token_ids:
            margins = []
            logits = P.forward(cfg, t, toks, margins=margins)[-1]
            slack = 1e-4 if dtype == "float32" else 0.1 * float(logits.std())
            if float(torch.stack(margins).min()) < CLOSE[dtype] and float(logits[tok]) < float(logits.max()) - slack:
                close_calls += 1                              # rounding may have chosen another expert somewhere
            else:
                assert float(logits[tok]) >= float(logits.max()) - slack, (dtype, p, o.token_ids, tok, int(logits.argmax()))
            toks.append(tok)
    assert close_calls <= (0 if dtype == "float32" else 6)
    llm.engine.runner.manager.check()


def test_recorded_steps_give_the_tokens_of_unrecorded_ones():
    """Decode steps, prompt portions and mixed steps from graphs, replayed many times with eager work between them."""
    from pico_vllm_amd import LLM, SamplingParams
    prompts = [[(7 * i + k) % 256 for i in range(n)] for k, n in enumerate((40, 3, 17, 90, 1, 64))]
    outs = []
    for graphs in (False, True):
        llm = LLM(model=model_dir("b"), dtype="bfloat16", block_size=8, num_gpu_blocks=64, max_seq_len=160, max_num_seqs=3,
                  max_num_batched_tokens=32, use_cuda_graph=graphs, max_batch_size=4)
        outs.append([o.token_ids for o in llm.generate(prompts, SamplingParams(max_new_tokens=25, temperature=0.0, ignore_eos=True))])
    assert outs[0] == outs[1]


def test_the_replay_program_in_a_subprocess():
    import json
    import os
    import subprocess
    import tempfile
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    name = "a"
    reqs = requests(CONFIGS[name]["vocab"], [40, 23, 31], seed=8)
    steps = []
    for rid, toks in reqs.items():
        parts = cut(toks, [9, 2, 14], tail=5)
        at = 0
        for i, n in enumerate(parts):
            steps.append({"step": len(steps), "entries": [{"id": rid, "tokens": toks[at:at + n], "want": list(range(n))}],
                          "end": [rid] if i == len(parts) - 1 else []})
            at += n
    with tempfile.TemporaryDirectory() as out:
        r = subprocess.run([os.path.join(root, "bin", "trace_run"), "--model", model_dir(name), "--dtype", "float32", "--out", out,
                            "--max-tokens", "64"], input="\n".join(json.dumps(s) for s in steps) + "\n", capture_output=True,
                           text=True, timeout=600)
        assert r.returncode == 0, r.stderr[-2000:]
        assert r.stdout.split("\n")[:-1] == [f"done {s['step']}" for s in steps]
        rows, fed = {}, {}
        for s in steps:
            e = s["entries"][0]
            a = np.fromfile(os.path.join(out, f"{s['step']}.f32"), dtype="<f4").reshape(len(e["want"]), -1)
            for w, row in zip(e["want"], a):
                rows[(e["id"], fed.get(e["id"], 0) + w)] = row
            fed[e["id"]] = fed.get(e["id"], 0) + len(e["tokens"])
    compare(name, "float32", rows, reqs)


def test_the_command_line_on_a_model_folder_of_this_design(capsys):
    from pico_vllm_amd import run
    assert run.main(["--model", model_dir("d"), "--prompt-ids", "5,17,3", "--prompt-ids", "9", "--max-new-tokens", "6",
                     "--ignore-eos", "--dtype", "float32", "--num-gpu-blocks", "16", "--max-seq-len", "64"]) == 0
    lines = [l for l in capsys.readouterr().out.splitlines() if l.startswith("[")]
    assert len(lines) == 2
    cfg, t = CONFIGS["d"], tensors_of("d")
    for line, prompt in zip(lines, ([5, 17, 3], [9])):
        toks = list(prompt)
        for tok in (int(x) for x in line.split(")")[1].split()):
            logits = P.forward(cfg, t, toks)[-1]
            assert float(logits[tok]) >= float(logits.max()) - 1e-4
            toks.append(tok)


# ---------------------------------------------------------------------------------------------------------------
# configurations drawn at random
# ---------------------------------------------------------------------------------------------------------------
def draw_config(seed, fast=False):
    """Sizes, head counts, order of layers, windows, constants, loops: all drawn; returns (config, page size).  ``fast``:
    sizes that the matrix-core kernels take."""
    rng = random.Random(4000 + seed)
    width = rng.choice([128, 192, 256] if fast else [40, 63, 72, 96, 128])
    layers = []
    for _ in range(rng.randint(1, 4)):
        G = rng.choice([1, 2])
        d, dv = rng.choice([(32, 32), (64, 64), (64, 32), (32, 64)] if fast else [(6, 6), (10, 12), (16, 16), (40, 20), (24, 24)])
        l = left(G * rng.choice([1, 2, 3]), G, d, dv, window=rng.choice([0, 1, 2, 15, 16, 17, 50, 90]), rot_dims=rng.choice([0, 2, d // 2 // 2 * 2, d]),
                 base=rng.choice([100.0, 5e5]))
        r = right(rng.randint(1, 4), *rng.choice([(32, 32), (64, 64), (16, 96), (128, 32)] if fast else [(1, 1), (5, 9), (16, 16), (33, 20), (8, 70)]),
                  slowest=rng.choice([0.9, 0.99, 1.0]))
        E, groups = rng.choice([(4, None), (6, (3, 2)), (8, (2, 1)), (8, (4, 3)), (12, (1, 1)), (16, (8, 5))])
        top = rng.randint(1, min(5, E if groups is None else groups[1] * E // groups[0]))
        ff = rng.choice([None, dense(rng.choice([24, 96])), moe(rng.choice([16, 40]), E, top, rng.choice([0.5, 3.0]), groups)])
        layers.append((pair(l, r, rng.choice([None, 0.5, 2.0]), rng.choice([None, 0.3, 1.7])), ff))
    loop = None
    if rng.random() < 0.7:
        a = rng.randrange(len(layers))
        loop = (a, rng.randint(a, len(layers)), rng.randint(1, 3))
    cfg = config(rng.choice([50, 131, 300]), width, layers, eps=rng.choice([1e-5, 1e-6]), embed_scale=rng.choice([None, 0.3, 7.0]),
                 cap=rng.choice([None, 5.0, 30.0]), loop=loop)
    return cfg, rng.choice([8, 16, 32])


@pytest.mark.parametrize("seed", range(12))
def test_configurations_drawn_at_random_in_mixed_batches(seed):
    cfg, page = draw_config(seed, fast=seed >= 8)
    t = P.random_model(cfg, seed)
    d = write_model(cfg, t, f"tubusun_drawn{seed}_")
    lengths = [60, 21, 150, 7, 45] if seed < 8 else [260, 90, 33, 140]
    reqs = requests(cfg["vocab"], lengths, seed=seed)
    steps, peak = mixed_steps(reqs, page, seed=seed)
    for dtype in ("float32", "bfloat16"):
        rows, _ = replay(d, dtype, steps, peak, page, max_live=3)
        Model(f"drawn{seed}", cfg, t).compare(dtype, rows, reqs)
