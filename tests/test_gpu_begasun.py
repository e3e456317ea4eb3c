"""The Begasun decoder in the engine against the plain implementation: each mechanism's kernels alone, each mixer alone,
then whole prompts, decoding through the cache and the state, portions down to two tokens, mixed batches in a small pool
with few state slots, keys and states that reach far back, long decoding, and greedy generation through the entry point."""
import functools
import random

import numpy as np
import pytest
import torch

import plain_begasun as P
from begasun_configs import CONFIGS, attention, config, latent, model_dir, rglru, tensors_of, write_model
from gpu_util import DEV
from replay_util import DT, F, MixerAlone, alone, close, cut, mixed_steps, replay, requests, rounded, roundup, row_errors, step_ctx

pytestmark = pytest.mark.gpu

# rms of a position's error over its logits (mean taken off), in units of the logits' own rms there
BOUND = {"float32": 3e-5, "bfloat16": 8e-2}
PAGE = {"a": 16, "b": 8, "c": 32, "d": 16, "e": 16}


@functools.lru_cache(maxsize=None)
def _named(name):
    return CONFIGS[name], tensors_of(name)


_plain = {}
YARD_DRAWS = 6


def plain_logits(name, tokens, cfg=None, tensors=None):
    key = (name, tuple(tokens))
    if key not in _plain:
        if cfg is None:
            cfg, tensors = _named(name)
        _plain[key] = P.forward(cfg, tensors, tokens).numpy()
    return _plain[key]


def yardstick(name, tokens, dtype, cfg=None, tensors=None):
    """What rounding alone does to every position's logits, in the units of ``row_errors``: the plain implementation
    with the rounding in question against itself in float64.  float32: all of it in float32 (other orders of summation
    than the engine's).  bfloat16: every activation between the parts rounded to 8 bits, up or down at random; the
    largest of a few draws."""
    key = (name, tuple(tokens), dtype)
    if key not in _plain:
        want = plain_logits(name, tokens, cfg, tensors)
        if cfg is None:
            cfg, tensors = _named(name)
        if dtype == "float32":
            draws = [P.forward(cfg, tensors, tokens, dtype=torch.float32).numpy().astype(np.float64)]
        else:
            draws = [P.forward(cfg, tensors, tokens, rounding=P.stochastic_bfloat16(100 + i)).numpy() for i in range(YARD_DRAWS)]
        _plain[key] = np.max([row_errors(d, want) for d in draws], axis=0)
    return _plain[key]


# A position's error may be a few times what rounding alone does there (the largest of a few draws: itself random), and
# never less than the floor is asked of it; one position in fifty (at least one a comparison) may lie over its limit, up to
# CAP.  A fault of the engine (a wrong key, a lost state) moves whole stretches of positions.
OVER_YARDSTICK = {"float32": 5.0, "bfloat16": 3.0}
CAP = {"float32": 1e-3, "bfloat16": 1.0}


def compare(name, dtype, rows, reqs, bound=None, cfg=None, tensors=None):
    floor = BOUND[dtype] if bound is None else bound
    errs, over, yards = [], [], []
    for (rid, pos), got in rows.items():
        toks = reqs[rid.split("#")[0]]
        e = float(row_errors(got[None], plain_logits(name, toks, cfg, tensors)[pos][None])[0])
        errs.append(e)
        yards.append(float(yardstick(name, toks, dtype, cfg, tensors)[pos]))
        limit = max(floor, OVER_YARDSTICK[dtype] * yards[-1])
        if not e <= limit:
            over.append(f"{rid} position {pos}: {e:.3g} > {limit:.3g}")
            assert e <= CAP[dtype], f"{name} {dtype}: {over[-1]}"
    assert len(over) <= max(1, len(errs) // 50), f"{name} {dtype}: {over}"
    if len(errs) >= 5:
        # the median position: half the floor, or (a model that rounding moves more) what the median yardstick says
        assert np.median(errs) <= max(floor / 2, np.median(yards)), f"{name} {dtype}: median {np.median(errs):.3g}"


# ---------------------------------------------------------------------------------------------------------------
# each mechanism's kernels alone
# ---------------------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("T,H,slabs", [(5, 72, 1), (33, 128, 3), (2, 43, 2), (3, 4100, 2), (2, 4098, 1), (1, 8, 8), (2, 16384, 1), (70, 1536, 1)])
def test_norm_of_the_output_sum_and_norm_of_the_sum(dtype, T, H, slabs):
    from pico_vllm_amd.ops import kernels
    g = torch.Generator().manual_seed(T + H)
    x, w, wn = torch.randn(T, H, generator=g), torch.randn(H, generator=g), 1 + 0.3 * torch.randn(H, generator=g)
    eps, eps_next = 1e-3, 1e-5
    y = torch.randn(slabs, T, H, generator=g) if slabs > 1 else rounded(torch.randn(T, H, generator=g), dtype).float()
    yd = y.to(DEV) if slabs > 1 else y.to(DEV, DT[dtype])
    want = x.to(F) + P.rms((y.sum(0) if slabs > 1 else y).to(F), eps) * w.to(F)
    for how in ("nothing", "rows", "norm", "strided"):
        resid = x.to(DEV)
        if how == "strided":                               # into the first columns of a wider buffer
            wide = torch.full((T, 2 * H), 7.0, dtype=DT[dtype], device=DEV)
            got = kernels.norm_add_norm(resid, yd, w.to(DEV), eps, out=wide[:, :H])
            assert float((wide[:, H:].float() - 7).abs().max()) == 0
        elif how == "norm":
            got = kernels.norm_add_norm(resid, yd, w.to(DEV), eps, wn.to(DEV), eps_next, out_dtype=DT[dtype])
        else:
            got = kernels.norm_add_norm(resid, yd, w.to(DEV), eps, out_dtype=DT[dtype] if how == "rows" else None)
        close(resid, want, "float32")
        if how == "nothing":
            assert got is None
        else:
            assert got.dtype == DT[dtype]
            close(got, P.rms(want, eps_next) * wn.to(F) if how == "norm" else want, dtype)


def test_a_rows_norm_does_not_depend_on_the_rows_beside_it():
    from pico_vllm_amd.ops import kernels
    g = torch.Generator().manual_seed(1)
    x, y, w = torch.randn(80, 500, generator=g), torch.randn(80, 500, generator=g), torch.randn(500, generator=g)
    many = x.to(DEV)
    n_many = kernels.norm_add_norm(many, y.to(DEV), w.to(DEV), 1e-5, w.to(DEV), 1e-5, out_dtype=torch.float32)
    for t in (0, 41, 79):
        one = x[t:t + 1].to(DEV)
        n_one = kernels.norm_add_norm(one, y[t:t + 1].to(DEV), w.to(DEV), 1e-5, w.to(DEV), 1e-5, out_dtype=torch.float32)
        assert torch.equal(one[0], many[t]) and torch.equal(n_one[0], n_many[t])


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_rows_into_a_part_of_a_buffer(dtype):
    from pico_vllm_amd.ops import kernels
    x = torch.randn(6, 50, generator=torch.Generator().manual_seed(2))
    buf = torch.zeros(6, 111, dtype=DT[dtype], device=DEV)
    kernels.store_rows(x.to(DEV), buf[:, 7:57])
    assert torch.equal(buf[:, 7:57].cpu(), x.to(DT[dtype])) and float(buf[:, :7].abs().max()) == 0 and float(buf[:, 57:].abs().max()) == 0


@pytest.mark.parametrize("M,N,K", [(1, 48, 128), (8, 40, 192), (33, 320, 64), (64, 34, 136), (70, 200, 256), (300, 64, 128)])
def test_the_clipped_activation_as_a_kernel_and_as_an_epilogue(M, N, K):
    """Gate and up of several times the limit, so that every branch of the clamps is taken."""
    from pico_vllm_amd.ops import kernels
    from pico_vllm_amd.ops.linear import Linear
    g = torch.Generator().manual_seed(M + N)
    x, w = rounded(torch.randn(M, K, generator=g), "bfloat16"), rounded(torch.randn(2 * N, K, generator=g) * 3 * K ** -0.5, "bfloat16")
    z = x @ w.T
    for limit, alpha in ((1.5, 1.702), (0.3, 1.0)):
        assert float((z > limit).double().mean()) > 0.1 and float((z < -limit).double().mean()) > 0.1
        act = lambda z: z[:, :N].clamp(max=limit) * torch.sigmoid(alpha * z[:, :N].clamp(max=limit)) * (z[:, N:].clamp(-limit, limit) + 1)
        close(Linear(w.to(DEV, torch.bfloat16)).clipped_glu(x.to(DEV, torch.bfloat16), limit, alpha), act(z), "bfloat16")
        for dtype in ("float32", "bfloat16"):
            zr = rounded(z, dtype)
            close(kernels.clipped_glu(zr.to(DEV, DT[dtype]), limit, alpha), act(zr), dtype)


@pytest.mark.parametrize("M,N,K", [(1, 24, 128), (8, 7, 192), (33, 256, 64), (64, 16, 136), (300, 40, 128), (5, 10, 44)])
def test_the_gated_token_row_as_a_kernel_and_as_an_epilogue(M, N, K):
    from pico_vllm_amd.ops import kernels
    from pico_vllm_amd.ops.linear import Linear
    g = torch.Generator().manual_seed(M + N)
    V, col = 19, 5
    x, w = rounded(torch.randn(M, K, generator=g), "bfloat16"), rounded(torch.randn(N, K, generator=g) * 2 * K ** -0.5, "bfloat16")
    table = rounded(torch.randn(V, col + N + 3, generator=g), "bfloat16")
    ids = torch.randint(0, V, (M,), generator=g, dtype=torch.int32)
    z = x @ w.T
    e = table[ids.long()][:, col:col + N]
    close(Linear(w.to(DEV, torch.bfloat16)).gelu_token(x.to(DEV, torch.bfloat16), ids.to(DEV), table.to(DEV, torch.bfloat16), col),
          P.gelu_tanh(z) * e, "bfloat16")
    for dtype in ("float32", "bfloat16"):
        zr = rounded(4 * z, dtype)
        for td in ("float32", "bfloat16"):
            close(kernels.gelu_token(zr.to(DEV, DT[dtype]), ids.to(DEV), table.to(DEV, DT[td]), col), P.gelu_tanh(zr) * e, dtype)


@pytest.mark.parametrize("M", [3, 64, 90, 300])
def test_a_products_float32_sums(M):
    from pico_vllm_amd.ops.linear import Linear
    g = torch.Generator().manual_seed(M)
    x, w = rounded(torch.randn(M, 640, generator=g), "bfloat16"), rounded(torch.randn(320, 640, generator=g), "bfloat16")
    y = Linear(w.to(DEV, torch.bfloat16)).sums(x.to(DEV, torch.bfloat16))
    assert y.dtype == torch.float32 and y.dim() == 3
    close(y.sum(0), x @ w.T, "float32")
    close(Linear(w.to(DEV, torch.float32)).sums(x.to(DEV, torch.float32)).sum(0), x @ w.T, "float32")


def conv_rows(x, w, bias, lens, prefix, slots, state, dtype):
    from pico_vllm_amd.ops import kernels
    ctx = step_ctx(lens, prefix, slots)
    return kernels.causal_conv(x.to(DEV, DT[dtype]), w.shape[0], w.t().contiguous().to(DEV), bias.to(DEV), ctx, state, 1,
                               single=ctx.all_decode, activation="none")


@pytest.mark.parametrize("T", [5, 90])
@pytest.mark.parametrize("H,G,dk,dv,rot", [(12, 2, 128, 128, 64), (3, 1, 24, 40, 8), (8, 2, 64, 32, 64), (1, 1, 64, 16, 0), (5, 5, 10, 12, 4), (2, 2, 32, 32, 2),
                                           (4, 2, 160, 160, 32)])
def test_head_norm_rotation_and_store_for_few_and_many_tokens(T, H, G, dk, dv, rot):
    """bfloat16: units of up to 128 entries of many tokens go two entries a lane; every head of q and of k by itself."""
    from pico_vllm_amd.ops import kernels
    g = torch.Generator().manual_seed(H * dk)
    page, pages = 8, 14
    cols = (H + G) * dk + G * dv
    x = rounded(3 * torch.randn(T, cols + (2 if cols % 2 == 0 else 3), generator=g, dtype=F), "bfloat16")
    wq, wk = 1 + 0.3 * torch.randn(dk, generator=g), 1 + 0.3 * torch.randn(dk, generator=g)
    pos = torch.arange(40, 40 + T, dtype=torch.int32)
    slots = torch.tensor([(t * 5) % (page * pages) if t != 4 else -1 for t in range(T)], dtype=torch.int32)
    table = None
    if rot:
        table = kernels.rope_table(pos.to(DEV), torch.tensor(P.frequencies(rot, 300.0)[0], dtype=torch.float32).to(DEV))
    kc = torch.zeros(pages, G, page, dk, dtype=torch.bfloat16, device=DEV)
    vc = torch.zeros(pages, G, dv, page, dtype=torch.bfloat16, device=DEV)
    q = kernels.qk_norm_store(x.to(DEV, torch.bfloat16), 0, H * dk, (H + G) * dk, H, G, G, dk, dv, 1, kernels.QK_NORM_UNIT, wq.to(DEV), wk.to(DEV),
                              1e-2, table, rot, slots.to(DEV), kc, vc)
    want_q = P.rotate_half(P.rms(x[:, :H * dk].view(T, H, dk), 1e-2) * wq.to(F), pos, rot, 300.0)
    want_k = P.rotate_half(P.rms(x[:, H * dk:(H + G) * dk].view(T, G, dk), 1e-2) * wk.to(F), pos, rot, 300.0)
    close(q.view(T, H, dk), want_q, "bfloat16", scale=0.5)
    assert float((q.view(T, H, dk).double().cpu() - want_q).abs().mean()) < 2e-3 * float(want_q.abs().mean()) * 2
    for t, s in enumerate(slots.tolist()):
        if s >= 0:
            close(kc[s // page, :, s % page, :], want_k[t], "bfloat16", scale=0.5)
            assert torch.equal(vc[s // page, :, :, s % page].double().cpu(), x[t, (H + G) * dk:cols].view(G, dv))
    empty = sorted(set(range(page * pages)) - set(slots.tolist()))
    assert all(float(kc[s // page, :, s % page, :].float().abs().max()) == 0 for s in empty)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("C,taps", [(36, 4), (128, 2), (40, 1), (21, 5)])
def test_the_convolution_without_activation(dtype, C, taps):
    g = torch.Generator().manual_seed(C)
    x = rounded(torch.randn(29, C + 3, generator=g, dtype=F), dtype)
    w, b = torch.randn(C, taps, generator=g), torch.randn(C, generator=g)
    want = P.causal_conv(x[:, :C], w.to(F), b.to(F))
    for portions in ([29], [2, 13, 1, 1, 12], [1] * 29):
        state = torch.full((3, C, taps), 7.0, device=DEV)
        state[1] = 0
        at, outs = 0, []
        for n in portions:
            outs.append(conv_rows(x[at:at + n], w, b, [n], [at], [1], state, dtype))
            at += n
        close(torch.cat(outs), want, dtype)
        assert float(state[1, :, 0].abs().max()) == 0 and float((state[[0, 2]] - 7).abs().max()) == 0


LRU_SHAPES = [(36, 3, 4), (40, 40, 1), (21, 1, 5), (128, 4, 2), (96, 1, 3), (192, 2, 4), (16, 2, 2), (560, 2, 3), (72, 1, 2)]   # channels, parts, taps


def lru_weights(C, parts, taps, seed, dtype):
    g = torch.Generator().manual_seed(seed)
    n = C // parts
    w = {"ra": rounded(torch.randn(parts, n, n, generator=g) * n ** -0.5, dtype), "ri": rounded(torch.randn(parts, n, n, generator=g) * n ** -0.5, dtype),
         "ra.b": 0.5 * torch.randn(parts, n, generator=g), "ri.b": 0.5 * torch.randn(parts, n, generator=g),
         "lam": -4 + 3 * (2 * torch.rand(C, generator=g) - 1)}
    dev = {"gates": tuple(w[k].transpose(1, 2).contiguous().to(DEV, DT[dtype]) for k in ("ra", "ri")),
           "gates_out_in": tuple(w[k].contiguous().to(DEV, DT[dtype]) for k in ("ra", "ri")),
           "br": w["ra.b"].reshape(-1).to(DEV), "bi": w["ri.b"].reshape(-1).to(DEV),
           "decay": (-8.0 * P.softplus(w["lam"].to(F))).float().to(DEV)}
    return {k: v.to(F) for k, v in w.items()}, dev


def lru_run(u, y, d, lens, prefix, slots, state, hist, dtype, chunked=False):
    from pico_vllm_amd.ops import kernels
    ctx = step_ctx(lens, prefix, slots)
    return kernels.lru_scan(u.to(DEV, DT[dtype]).contiguous(), y.to(DEV, DT[dtype]), d["gates"], d["br"], d["bi"], d["decay"], ctx, state, hist,
                            w_out_in=d["gates_out_in"], chunked=chunked)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("C,parts,taps", LRU_SHAPES)
def test_the_recurrence_whole_in_portions_and_in_chunks(dtype, C, parts, taps):
    w, d = lru_weights(C, parts, taps, C + taps, dtype)
    g = torch.Generator().manual_seed(C)
    T = 150
    u, y = rounded(torch.randn(T, C, generator=g, dtype=F), dtype), rounded(torch.randn(T, C + 5, generator=g, dtype=F), dtype)
    s0 = torch.randn(C, generator=g)
    S, last = P.lru_scan(*P.lru_gates(u, w, parts), S0=s0.to(F))
    want = S * P.gelu_tanh(y[:, :C])
    results = []
    for portions in ([T], [2, 70, 1, 50, 27]):
        state = torch.full((4, C, taps), 3.0, device=DEV)
        state[2, :, 0] = s0.to(DEV)
        at, outs = 0, []
        for n in portions:
            outs.append(lru_run(u[at:at + n], y[at:at + n], d, [n], [at], [2], state, taps - 1, dtype))
            at += n
        got = torch.cat(outs)
        results.append((got, state.clone()))
        close(got, want, dtype)
        close(state[2, :, 0], last, "float32")
        assert float((state[[0, 1, 3]] - 3).abs().max()) == 0 and (taps == 1 or float((state[2, :, 1:] - 3).abs().max()) == 0)
    assert torch.equal(results[0][0], results[1][0]) and torch.equal(results[0][1], results[1][1])       # the cut changes no bit
    if dtype == "bfloat16" and (C // parts) % 8 == 0:
        # chunks of 64 side by side, several sequences of unequal length, one going on from a state
        lens, slots = [64, 1, 0, 65, 20], [1, 0, 4, 2, 3]
        state = torch.zeros(6, C, taps, device=DEV)
        state[2, :, 0] = s0.to(DEV)
        got = lru_run(u, y, d, lens, [0, 0, 0, 7, 0], slots, state, taps - 1, dtype, chunked=True)
        at = 0
        for n, slot in zip(lens, slots):
            if n:
                S, last = P.lru_scan(*P.lru_gates(u[at:at + n], w, parts), S0=s0.to(F) if slot == 2 else None)
                close(got[at:at + n], S * P.gelu_tanh(y[at:at + n, :C]), dtype)
                close(state[slot, :, 0], last, "float32", scale=2)
            at += n
        assert float(state[[4, 5]].abs().max()) == 0


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("C,parts,taps", LRU_SHAPES)
def test_a_single_token_step_is_the_walk_of_one_token(dtype, C, parts, taps):
    """Convolution, gates, walk and output of a token a sequence in one launch: the same bits as the launches of a portion."""
    from pico_vllm_amd.ops import kernels
    w, d = lru_weights(C, parts, taps, C, dtype)
    g = torch.Generator().manual_seed(C + 1)
    T = 12
    cw, cb = torch.randn(C, taps, generator=g), torch.randn(C, generator=g)
    yx = [rounded(torch.randn(T, 2 * C, generator=g, dtype=F), dtype) for _ in range(3)]
    slots = [2, 0, 3]
    state = torch.zeros(5, C, taps, device=DEV)
    ref = torch.zeros(5, C, taps, device=DEV)
    cwd, cbd = cw.t().contiguous().to(DEV), cb.to(DEV)
    for b, rows in enumerate(yx):
        u = P.causal_conv(rows[:, C:], cw.to(F), cb.to(F)).to(DT[dtype]).to(F)
        S, _ = P.lru_scan(*P.lru_gates(u, w, parts))
        want = S * P.gelu_tanh(rows[:, :C])
        dev = rows.to(DEV, DT[dtype])
        ur = conv_rows(rows[:, C:], cw, cb, [T], [0], [slots[b]], ref, dtype)
        whole = kernels.lru_scan(ur, dev[:, :C], d["gates"], d["br"], d["bi"], d["decay"], step_ctx([T], [0], [slots[b]]), ref, taps - 1)
        close(whole, want, dtype)
        yx[b] = (dev, whole)
    for t in range(T):
        rows = torch.stack([dev[t] for dev, _ in yx])
        got = kernels.lru_step(rows[:, C:], rows[:, :C], cwd, cbd, d["gates"], d["br"], d["bi"], d["decay"], step_ctx([1] * 3, [t] * 3, slots), state)
        for b, (_, whole) in enumerate(yx):
            assert torch.equal(got[b], whole[t])
    assert torch.equal(state, ref) and float(state[[1, 4]].abs().max()) == 0


@pytest.mark.parametrize("chunked", [False, True])
def test_a_first_token_is_kept_for_hundreds_of_tokens_or_forgotten(chunked):
    """Decays of nearly one keep the first token's addend; large ones forget it.  Zero inputs behind the first token."""
    C, parts, T = 16, 2, 700
    d = lru_weights(C, parts, 1, 0, "bfloat16")[1]
    d["gates"] = d["gates_out_in"] = tuple(torch.zeros_like(t) for t in d["gates"])
    d["br"], d["bi"] = torch.zeros(C, device=DEV), torch.full((C,), 30.0, device=DEV)            # r = 1/2, i = 1
    sp = torch.full((C,), 1e-4)
    sp[::2] = 1.0
    d["decay"] = (-8.0 * sp).to(DEV)
    u = torch.zeros(T, C, dtype=F)
    u[0] = 1.0
    y = torch.full((T, C), 3.0, dtype=F)
    state = torch.zeros(2, C, 1, device=DEV)
    outs = [lru_run(u[a:b], y[a:b], d, [b - a], [a], [1], state, 0, "bfloat16", chunked=chunked) for a, b in ((0, 300), (300, 699), (699, T))]
    la = d["decay"].double().cpu() / 2
    S = torch.sqrt(1 - torch.exp(2 * la)) * torch.exp(la * (T - 1))
    assert float(S[1]) > 0.015 and float(S[0]) < 1e-100
    assert torch.allclose(state[1, :, 0].double().cpu(), S, rtol=1e-4, atol=1e-30)
    close(outs[-1][0], S * P.gelu_tanh(y[0]), "bfloat16")


# ---------------------------------------------------------------------------------------------------------------
# each mixer alone, with pages and slots from the cache manager
# ---------------------------------------------------------------------------------------------------------------
def mixer_case(kind, m, width, seed):
    cfg = config(8, width, [((kind, m), None)])
    t = {n[len("l0.mix."):]: v for n, v in P.random_model(cfg, seed).items() if n.startswith("l0.mix.")}
    from pico_vllm_amd.config.begasun import BegasunConfig, _mixer_spec
    c = BegasunConfig.from_dict(cfg)
    return _mixer_spec(c, c.layers[0]), t


def plain_mixer(kind, m, t, h, first_pos=0):
    return P.MIXERS[kind](h, {k: v.to(F) for k, v in t.items()}, m, 1e-5, first_pos)


MIXER_CASES = {
    "latent": (latent(3, 14, 6, 10, 20, scaling=(4.0, 24, 8.0, 1.0)), 72), "latent matrix cores": (latent(4, 40, 32, 24, 64, base=1e4), 128),
    "latent without rotation": (latent(2, 32, 0, 48, 32), 40), "latent many heads": (latent(20, 8, 32, 16, 32), 64),
    "attention": (attention(3, 1, 24, 40, rot_dims=10), 72), "attention one size": (attention(4, 2, 64, 64, rot_dims=32), 128),
    "attention two sizes": (attention(8, 2, 64, 32, rot_dims=64), 96), "attention of 96": (attention(6, 6, 96, 96, rot_dims=2), 64),
    "recurrence": (rglru(36, 3, 4), 72), "recurrence matrix cores": (rglru(192, 2, 4), 128), "recurrence one channel a block": (rglru(24, 24, 1), 40)}


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("case", sorted(MIXER_CASES))
def test_a_mixer_alone_in_portions_and_mixed_batches(case, dtype):
    (kind, m), width = MIXER_CASES[case]
    spec, t = mixer_case(kind, m, width, seed=len(case))
    g = torch.Generator().manual_seed(7)
    lens = {"r0": 190, "r1": 43, "r2": 96}
    rows = {r: rounded(torch.randn(n, width, generator=g, dtype=F), dtype) for r, n in lens.items()}
    want = {r: plain_mixer(kind, m, t, h) for r, h in rows.items()}
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
        assert float(err.max()) < (2e-5 if dtype == "float32" else 6e-2), (r, int(err.argmax()), float(err.max()))
        assert float(err.median()) < (5e-6 if dtype == "float32" else 1.5e-2), (r, float(err.median()))
    if dtype == "float32":                                # whole at once: the same bits
        again = MixerAlone(spec, t, dtype).step([("r0", rows["r0"])])["r0"]
        assert torch.equal(again, torch.cat(got["r0"]))


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("case", ["latent", "latent matrix cores", "attention", "attention one size", "attention two sizes"])
def test_one_key_that_stands_out(case, dtype):
    """Weights under which a row that asks for mark x fits the one row that carries mark x and nothing else: at the first
    position, on both sides of page borders and hundreds of tokens back, asked for by single tokens and inside portions.
    What comes out is that row's value; left out, something else does."""
    (kind, m), width = MIXER_CASES[case]
    rot = 0 if kind == "latent_attention" else 10
    m = dict(m, scale=4 * m["scale"]) if rot == 0 else dict(m, scale=8 * m["scale"], rot={"dims": rot, "base": 100.0})
    spec, t = mixer_case(kind, m, width, seed=3)
    asked = {300: 0, 301: 7, 302: 8, 303: 255, 304: 256, 420: 63, 421: 64, 448: 1}
    n, d = len(asked), m["dim"]
    t = {k: v.clone() for k, v in t.items()}
    for k in ("q", "k", "v", "dkv", "g"):
        if k in t:
            t[k][:, :2 * n] = 0                           # columns 0 .. n - 1 ask for marks, n .. 2 n - 1 carry them
    heads = m["heads"]
    step = d + m["rot_dim"] if kind == "latent_attention" else d
    for x in range(n):
        for hh in range(heads):                           # an entry a mark of every query, behind what is turned
            t["q"][hh * step + rot + x] = 0
            t["q"][hh * step + rot + x, x] = 1
        if kind == "latent_attention":
            t["dkv"][x] = 0
            t["dkv"][x, n + x] = 1
            for hh in range(heads):
                t["uk"][hh * d + x] = 0
                t["uk"][hh * d + x, x] = 1
        else:
            for g in range(m["kv_heads"]):
                t["k"][g * d + rot + x] = 0
                t["k"][g * d + rot + x, n + x] = 1
    g = torch.Generator().manual_seed(11)
    h = torch.randn(450, width, generator=g, dtype=F)
    h[:, :2 * n] = 0
    for x, (i, j) in enumerate(asked.items()):
        h[i, x] = h[j, n + x] = 30.0
    h = rounded(h, dtype)
    want = plain_mixer(kind, m, t, h)
    rms_of = lambda v: float(v.pow(2).mean().sqrt())
    for i, j in asked.items():                            # leaving the key out would show
        without = plain_mixer(kind, m, t, torch.cat([h[:j], h[j + 1:i + 1]]), first_pos=0)[-1]
        assert rms_of(want[i] - without) > 0.3 * rms_of(want[i])
    mx = MixerAlone(spec, t, dtype)
    got = torch.cat([mx.step([("r", h[a:b])])["r"] for a, b in
                     [(0, 300)] + [(i, i + 1) for i in range(300, 305)] + [(305, 421), (421, 422), (422, 448), (448, 450)]])
    for i in asked:
        assert rms_of(got[i] - want[i]) < (2e-5 if dtype == "float32" else 3e-2) * rms_of(want[i]), i


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("width", [44, 128])
def test_the_stream_made_anew_from_itself_and_the_input(dtype, width):
    """Whether the launch in front has left the stream's rows or not, and with a delta still pending."""
    from types import SimpleNamespace
    from pico_vllm_amd.ops import kernels
    from pico_vllm_amd.parts.input_mix import InputMix
    g = torch.Generator().manual_seed(width)
    T = 9
    w = rounded(torch.randn(width, 2 * width, generator=g) * width ** -0.5, dtype)
    x0, x, d = (torch.randn(T, width, generator=g) for _ in range(3))
    part = InputMix(width, name="", act_dtype=DT[dtype])
    part.load({"": w.to(DT[dtype])}, torch.device(DEV), DT[dtype])
    for how in ("fresh", "left", "pending"):
        ctx = SimpleNamespace(shared={})
        part.enter(x0.to(DEV), ctx)
        resid = x.to(DEV)
        cur = x.to(F)
        if how == "left":
            part.rows(ctx).rows.copy_(resid.to(DT[dtype]))
            part.rows(ctx).of = resid
        new, pending = part.mix(resid, d.to(DEV) if how == "pending" else None, ctx)
        if how == "pending":
            cur = (x + d).to(F)
        got = new if pending is None else new + pending.sum(0)
        assert got.dtype == torch.float32
        close(got, torch.cat([rounded(cur, dtype), rounded(x0, dtype)], dim=-1) @ w.T, "float32")
        assert part.rows(ctx).of is None                  # the next pass fills the rows again


# ---------------------------------------------------------------------------------------------------------------
# whole models through the engine
# ---------------------------------------------------------------------------------------------------------------
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
def test_long_decoding(dtype):
    reqs = requests(CONFIGS["b"]["vocab"], [330], seed=6)
    rows, _ = replay(model_dir("b"), dtype, alone(reqs, lambda t: cut(t, [30], tail=300)), roundup(330), PAGE["b"])
    compare("b", dtype, rows, reqs)


def test_sharp_attention_on_far_keys():
    """Scales so large that every query's softmax sits on very few keys, many of them hundreds of tokens back and on other
    pages, in both attentions and in every pass of the loop: a key read from a wrong place shows in the logits."""
    cfg = config(64, 64, [(attention(2, 1, 16, 16, rot_dims=4, base=50.0, scale=1.5), (32, 1.0)), (latent(2, 12, 4, 8, 16, scale=1.5, base=50.0), None),
                          (rglru(16, 2, 3), None)], loop=(0, 2, 2), side=4)
    t = P.random_model(cfg, 5)
    d = write_model(cfg, t, "begasun_far_")
    reqs = requests(64, [400], seed=9)
    for portions in (lambda x: [len(x)], lambda x: cut(x, [2, 61, 8, 130], tail=40)):
        rows, _ = replay(d, "float32", alone(reqs, portions), roundup(400), 8)
        compare("far", "float32", rows, reqs, bound=1e-4, cfg=cfg, tensors=t)


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
    for p, o in zip(prompts, outs):
        assert len(o.token_ids) == 12
        toks = list(p)
        for tok in o.token_ids:
            logits = P.forward(cfg, t, toks)[-1]
            slack = 1e-4 if dtype == "float32" else 0.08 * float(logits.std())
            assert float(logits[tok]) >= float(logits.max()) - slack, (dtype, p, o.token_ids, tok, int(logits.argmax()))
            toks.append(tok)
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
    """Sizes, head counts, order of layers, constants, loops: all drawn; returns (config, page size).  ``fast``: sizes that
    the matrix-core kernels take."""
    rng = random.Random(3000 + seed)
    width = rng.choice([128, 192, 256] if fast else [40, 63, 72, 96, 128])
    layers = []
    for _ in range(rng.randint(1, 4)):
        kind = rng.choice(["latent", "attention", "rglru"])
        ff = rng.choice([None, (24, 0.5), (64, 2.0)])
        G = rng.choice([1, 2])
        H = G * rng.choice([1, 2, 3])
        if kind == "attention":
            d, dv = rng.choice([(32, 32), (64, 64), (64, 32), (32, 64)] if fast else [(6, 6), (10, 12), (16, 16), (40, 20), (24, 24)])
            mixer = attention(H, G, d, dv, rot_dims=rng.choice([0, 2, d // 2 // 2 * 2, d]), base=rng.choice([100.0, 5e5]))
        elif kind == "latent":
            R, r = rng.choice([(32, 32), (64, 32), (64, 64), (32, 0)] if fast else [(5, 2), (20, 12), (33, 0), (16, 4)])
            mixer = latent(H, rng.choice([8, 20, 48]), r, rng.choice([8, 12, 40]), R, base=rng.choice([100.0, 5e5]),
                           scaling=rng.choice([None, (8.0, 64, 16.0, 1.0), (2.5, 32, 4.0, 0.5)]))
        else:
            n = rng.choice([32, 64, 96] if fast else [1, 5, 8, 24])
            B = rng.randint(1, 4)
            mixer = rglru(n * B, B, rng.randint(1, 5))
        layers.append((mixer, ff))
    loop = None
    if rng.random() < 0.7:
        a = rng.randrange(len(layers))
        loop = (a, rng.randint(a, len(layers)), rng.randint(1, 3))
    cfg = config(rng.choice([50, 131, 300]), width, layers, eps=rng.choice([1e-5, 1e-6]), embed_scale=rng.choice([None, 0.3, 7.0]),
                 logit_scale=rng.choice([None, 0.1, 3.0]), loop=loop, side=rng.choice([0, 3, 16]))
    return cfg, rng.choice([8, 16, 32])


@pytest.mark.parametrize("seed", range(12))
def test_configurations_drawn_at_random_in_mixed_batches(seed):
    cfg, page = draw_config(seed, fast=seed >= 8)
    t = P.random_model(cfg, seed)
    d = write_model(cfg, t, f"begasun_drawn{seed}_")
    lengths = [60, 21, 150, 7, 45] if seed < 8 else [260, 90, 33, 140]
    reqs = requests(cfg["vocab"], lengths, seed=seed)
    steps, peak = mixed_steps(reqs, page, seed=seed)
    for dtype in ("float32", "bfloat16"):
        rows, _ = replay(d, dtype, steps, peak, page, max_live=3)
        compare(f"drawn{seed}", dtype, rows, reqs, cfg=cfg, tensors=t)
