"""A plain, slow implementation of the Begasun decoder: whole sequences, no cache, float64 on the CPU, one function per
mechanism, written from the design's equations and sharing no code with the package.

Notation: T tokens at positions 0 .. T - 1, width D, eps the model's norm constant.  A weight dict maps checkpoint names
('l3.mix.q', 'side.embed', ..) to tensors; linear weights are [out, in] and applied as x W^T.

  model:   x = E[token] a (a = embedding.scale), x0 = x.  Layers in order, the looped span several times in a row, and in
           front of every pass of it x <- [x | x0] Wloop^T.
  layer i: x += s1 nz(mixer(nz(x; n1)); n1b); if it has a feed-forward x += s2 nz(ff(nz(x; n2)); n2b); then, with a token
           side, x += rms(Wp (gelu(Wg x) * side[token, part i])) w.   nz(x; w) = rms(x) (1 + w).
  logits = nz(x; final) Wh^T b (b = logit_scale).
"""
from __future__ import annotations

import math
from typing import Dict, List, Optional, Tuple

import torch

F64 = torch.float64

# A yardstick for what rounding alone does: with ``forward(..., rounding=f)`` every activation that passes from one part
# to the next (a product's output, a convolution's, an attention's, the stream as a product reads it) goes through f.
_rounding = None


def act(x: torch.Tensor) -> torch.Tensor:
    return x if _rounding is None else _rounding(x)


def stochastic_bfloat16(seed: int):
    """A rounding to bfloat16's 8 significant bits that rounds up or down at random, in proportion (unbiased); draws
    with different seeds are independent."""
    g = torch.Generator().manual_seed(seed)

    def f(x: torch.Tensor) -> torch.Tensor:
        ulp = torch.exp2(torch.floor(torch.log2(x.abs().clamp_min(1e-300))) - 7)
        return torch.floor(x / ulp + torch.rand(x.shape, generator=g, dtype=x.dtype)) * ulp
    return f


# ---- elementwise -------------------------------------------------------------------------------------------------------
def rms(x: torch.Tensor, eps: float) -> torch.Tensor:
    """x over its root mean square along the last axis, eps inside the root."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def norm_zero(x: torch.Tensor, w: torch.Tensor, eps: float) -> torch.Tensor:
    """An RMS norm whose weight is stored around zero."""
    return rms(x, eps) * (1.0 + w)


def gelu_tanh(z: torch.Tensor) -> torch.Tensor:
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def softplus(x: torch.Tensor) -> torch.Tensor:
    return torch.where(x > 30, x, torch.log1p(torch.exp(torch.clamp(x, max=30))))


# ---- rotation ----------------------------------------------------------------------------------------------------------
def frequencies(dims: int, base: float, scaling: Optional[dict] = None) -> Tuple[List[float], float]:
    """(f_i for the dims / 2 pairs, the factor on cosine and sine).  ``scaling``: factor, original, fast, slow: pairs
    that turn often within the original length stay, slow ones are stretched by the factor, a ramp between."""
    f = [base ** (-2.0 * i / dims) for i in range(dims // 2)]
    if not scaling:
        return f, 1.0
    pair = lambda turns: dims * math.log(scaling["original"] / (2.0 * math.pi * turns)) / (2.0 * math.log(base))
    lo = max(math.floor(pair(scaling["fast"])), 0)
    hi = min(math.ceil(pair(scaling["slow"])), dims - 1)
    out = []
    for i, fi in enumerate(f):
        r = min(1.0, max(0.0, (i - lo) / max(hi - lo, 0.001)))
        out.append(fi / scaling["factor"] * r + fi * (1.0 - r))
    return out, 0.1 * math.log(scaling["factor"]) + 1.0


def _cos_sin(positions, dims, base, scaling, dtype):
    f, mag = frequencies(dims, base, scaling)
    a = positions.to(dtype).view(-1, 1, 1) * torch.tensor(f, dtype=dtype)
    return torch.cos(a) * mag, torch.sin(a) * mag


def rotate_pairs(x: torch.Tensor, positions: torch.Tensor, dims: int, base: float, scaling: Optional[dict] = None) -> torch.Tensor:
    """x [T, heads, d]: of the first dims entries, 2i goes with 2i + 1."""
    if not dims:
        return x
    c, s = _cos_sin(positions, dims, base, scaling, x.dtype)
    u, v = x[..., 0:dims:2], x[..., 1:dims:2]
    turned = torch.stack([u * c - v * s, v * c + u * s], dim=-1).flatten(-2)
    return torch.cat([turned, x[..., dims:]], dim=-1)


def rotate_half(x: torch.Tensor, positions: torch.Tensor, dims: int, base: float, scaling: Optional[dict] = None) -> torch.Tensor:
    """x [T, heads, d]: of the first dims entries, i goes with i + dims / 2."""
    if not dims:
        return x
    c, s = _cos_sin(positions, dims, base, scaling, x.dtype)
    half = dims // 2
    u, v = x[..., :half], x[..., half:dims]
    return torch.cat([u * c - v * s, v * c + u * s, x[..., dims:]], dim=-1)


# ---- mixers ------------------------------------------------------------------------------------------------------------
def causal_softmax(s: torch.Tensor) -> torch.Tensor:
    """Scores [T, T] (query, key): softmax over keys j <= i."""
    T = s.shape[0]
    return torch.softmax(s.masked_fill(~torch.tril(torch.ones(T, T, dtype=torch.bool)), float("-inf")), dim=-1)


def latent_attention(h: torch.Tensor, w: Dict[str, torch.Tensor], m: dict, eps: float, first_pos: int = 0) -> torch.Tensor:
    """Every head's keys and values are made from the latent (no key is shared between heads but the rotated part)."""
    T = h.shape[0]
    H, d, r, dv, R = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    pos = torch.arange(first_pos, first_pos + T)
    rot = m.get("rot") or {}
    q = act(h @ w["q"].T).view(T, H, d + r)
    ckr = act(h @ w["dkv"].T)
    c = act(rms(ckr[:, :R], eps) * w["dkv.norm"])
    kr = act(rotate_pairs(ckr[:, R:].view(T, 1, r), pos, r, rot.get("base", 1.0), rot.get("scaling")))[:, 0]
    qr = act(rotate_pairs(q[..., d:], pos, r, rot.get("base", 1.0), rot.get("scaling")))
    ku = act(c @ w["uk"].T).view(T, H, d)
    v = act(c @ w["uv"].T).view(T, H, dv)
    gate = torch.sigmoid(act(h @ w["g"].T))                              # [T, H]
    out = torch.zeros(T, H, dv, dtype=h.dtype)
    for k in range(H):
        s = (q[:, k, :d] @ ku[:, k].T + qr[:, k] @ kr.T) * m["scale"]
        out[:, k] = (causal_softmax(s) @ v[:, k]) * gate[:, k:k + 1]
    return act(act(out.reshape(T, H * dv)) @ w["o"].T)


def attention(h: torch.Tensor, w: Dict[str, torch.Tensor], m: dict, eps: float, first_pos: int = 0) -> torch.Tensor:
    T = h.shape[0]
    H, G, d, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    pos = torch.arange(first_pos, first_pos + T)
    rot = m.get("rot") or {}
    turn = lambda x: rotate_half(x, pos, rot.get("dims", 0), rot.get("base", 1.0), rot.get("scaling"))
    q = act(turn(rms(act(h @ w["q"].T).view(T, H, d), eps) * w["q.norm"]))
    k = act(turn(rms(act(h @ w["k"].T).view(T, G, d), eps) * w["k.norm"]))
    v = act(h @ w["v"].T).view(T, G, dv)
    out = torch.zeros(T, H, dv, dtype=h.dtype)
    for a in range(H):
        g = a // (H // G)
        out[:, a] = causal_softmax((q[:, a] @ k[:, g].T) * m["scale"]) @ v[:, g]
    return act(act(out.reshape(T, H * dv)) @ w["o"].T)


def causal_conv(x: torch.Tensor, taps: torch.Tensor, bias: torch.Tensor, history: Optional[torch.Tensor] = None) -> torch.Tensor:
    """x [T, C], taps [C, K] (the last column is the current token's); inputs before the start are zero, or ``history``
    [K - 1, C] (oldest first)."""
    T, C = x.shape
    K = taps.shape[1]
    past = torch.zeros(K - 1, C, dtype=x.dtype) if history is None else history
    xx = torch.cat([past, x], dim=0)
    return sum(xx[j:j + T] * taps[:, j] for j in range(K)) + bias


def lru_gates(u: torch.Tensor, w: Dict[str, torch.Tensor], blocks: int) -> Tuple[torch.Tensor, torch.Tensor]:
    """(log a, what is added to the state) of every token and channel: u [T, C] in equal parts, each through its own pair
    of square matrices."""
    T, C = u.shape
    n = C // blocks
    r = torch.zeros_like(u)
    i = torch.zeros_like(u)
    for b in range(blocks):
        ub = u[:, b * n:(b + 1) * n]
        r[:, b * n:(b + 1) * n] = torch.sigmoid(ub @ w["ra"][b].T + w["ra.b"][b])
        i[:, b * n:(b + 1) * n] = torch.sigmoid(ub @ w["ri"][b].T + w["ri.b"][b])
    log_a = -8.0 * r * softplus(w["lam"])
    return log_a, torch.sqrt(-torch.expm1(2.0 * log_a)) * i * u


def lru_scan(log_a: torch.Tensor, add: torch.Tensor, S0: Optional[torch.Tensor] = None) -> Tuple[torch.Tensor, torch.Tensor]:
    """S_t = a_t S_(t-1) + add_t, channel by channel; (all S_t, the last)."""
    S = torch.zeros_like(add[0]) if S0 is None else S0
    out = torch.zeros_like(add)
    for t in range(add.shape[0]):
        S = torch.exp(log_a[t]) * S + add[t]
        out[t] = S
    return out, S


def rglru(h: torch.Tensor, w: Dict[str, torch.Tensor], m: dict, eps: float, first_pos: int = 0) -> torch.Tensor:
    y = act(gelu_tanh(h @ w["y"].T + w["y.b"]))
    u = act(causal_conv(act(h @ w["x"].T + w["x.b"]), w["conv"], w["conv.b"]))
    S, _ = lru_scan(*lru_gates(u, w, m["blocks"]))
    return act(act(S * y) @ w["o"].T)


MIXERS = {"latent_attention": latent_attention, "attention": attention, "rglru": rglru}


# ---- feed-forward, the token side, order, model --------------------------------------------------------------------------
def clipped_mlp(h: torch.Tensor, w: Dict[str, torch.Tensor], limit: float) -> torch.Tensor:
    g = torch.clamp(h @ w["gate"].T, max=limit)
    u = torch.clamp(h @ w["up"].T, min=-limit, max=limit)
    return act(act(g * torch.sigmoid(1.702 * g) * (u + 1.0)) @ w["down"].T)


def token_side(x: torch.Tensor, e: torch.Tensor, w: Dict[str, torch.Tensor], eps: float) -> torch.Tensor:
    """What a layer's token input adds to the stream; e [T, dim] the tokens' rows of this layer's part."""
    g = act(gelu_tanh(act(x) @ w["gate"].T) * e)
    return rms(act(g @ w["proj"].T), eps) * w["norm"]


def run_order(layers: int, loop: Optional[dict]) -> List[Tuple[int, bool]]:
    """(layer, whether a pass of the looped span starts in front of it)."""
    if not loop or loop["start"] >= loop["stop"]:
        return [(i, False) for i in range(layers)]
    a, b = loop["start"], loop["stop"]
    return ([(i, False) for i in range(a)] + [(i, i == a) for _ in range(loop["times"]) for i in range(a, b)]
            + [(i, False) for i in range(b, layers)])


def forward(cfg: dict, weights: Dict[str, torch.Tensor], tokens: List[int], dtype=F64, trace: Optional[list] = None,
            rounding=None) -> torch.Tensor:
    """Logits [T, vocab] of one sequence from position 0.  ``trace``: a list that receives the stream after every layer
    run.  ``rounding``: a function that every activation between the parts goes through (the stream itself stays as it
    is; what a product reads of it is rounded)."""
    global _rounding
    _rounding = rounding
    try:
        return _forward(cfg, weights, tokens, dtype, trace)
    finally:
        _rounding = None


def _forward(cfg, weights, tokens, dtype, trace):
    W = {n: (t.to(dtype) if t.is_floating_point() else t) for n, t in weights.items()}
    under = lambda p, ws: {n[len(p) + 1:]: t for n, t in ws.items() if n.startswith(p + ".")}
    eps = cfg["norm"]["eps"]
    tok = torch.tensor(tokens)
    x = W["embed"][tok] * (cfg.get("embedding") or {}).get("scale", 1.0)
    x0 = x
    side = cfg.get("token_side")
    for i, again in run_order(len(cfg["layers"]), cfg.get("loop")):
        if again:
            x = torch.cat([act(x), act(x0)], dim=-1) @ W["loop.in"].T
        layer, lw = cfg["layers"][i], under(f"l{i}", W)
        y = MIXERS[layer["type"]](act(norm_zero(x, lw["norm1"], eps)), under("mix", lw), layer["mixer"], eps)
        x = x + lw["ls1"] * norm_zero(y, lw["norm1b"], eps)
        if layer.get("mlp"):
            f = clipped_mlp(act(norm_zero(x, lw["norm2"], eps)), under("mlp", lw), layer["mlp"]["limit"])
            x = x + lw["ls2"] * norm_zero(f, lw["norm2b"], eps)
        if side:
            n = side["dim"]
            x = x + token_side(x, W["side.embed"][tok][:, i * n:(i + 1) * n], under("side", lw), eps)
        if trace is not None:
            trace.append(x.clone())
    return (act(norm_zero(x, W["final.norm"], eps)) @ W["head"].T) * cfg.get("logit_scale", 1.0)


# ---- random models -----------------------------------------------------------------------------------------------------
def tensor_shapes(cfg: dict) -> Dict[str, tuple]:
    """Name -> shape of every tensor a model of this configuration holds."""
    D, V, n = cfg["width"], cfg["vocab"], len(cfg["layers"])
    out = {"embed": (V, D), "final.norm": (D,), "head": (V, D)}
    if cfg.get("loop"):
        out["loop.in"] = (D, 2 * D)
    side = (cfg.get("token_side") or {}).get("dim", 0)
    if side:
        out["side.embed"] = (V, n * side)
    for i, layer in enumerate(cfg["layers"]):
        p, q, m = f"l{i}.", f"l{i}.mix.", layer["mixer"]
        out.update({p + "norm1": (D,), p + "norm1b": (D,), p + "ls1": (D,)})
        if layer["type"] == "latent_attention":
            H, d, r, dv, R = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
            out.update({q + "q": (H * (d + r), D), q + "dkv": (R + r, D), q + "dkv.norm": (R,), q + "uk": (H * d, R),
                        q + "uv": (H * dv, R), q + "g": (H, D), q + "o": (D, H * dv)})
        elif layer["type"] == "attention":
            H, G, d, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
            out.update({q + "q": (H * d, D), q + "k": (G * d, D), q + "v": (G * dv, D), q + "q.norm": (d,), q + "k.norm": (d,),
                        q + "o": (D, H * dv)})
        else:
            C, B, K = m["width"], m["blocks"], m["conv"]
            s = C // B
            out.update({q + "y": (C, D), q + "y.b": (C,), q + "x": (C, D), q + "x.b": (C,), q + "conv": (C, K), q + "conv.b": (C,),
                        q + "ra": (B, s, s), q + "ra.b": (B, s), q + "ri": (B, s, s), q + "ri.b": (B, s), q + "lam": (C,),
                        q + "o": (D, C)})
        if layer.get("mlp"):
            F = layer["mlp"]["ff"]
            out.update({p + "norm2": (D,), p + "norm2b": (D,), p + "ls2": (D,), p + "mlp.gate": (F, D), p + "mlp.up": (F, D),
                        p + "mlp.down": (D, F)})
        if side:
            out.update({p + "side.gate": (side, D), p + "side.proj": (D, side), p + "side.norm": (D,)})
    return out


def random_model(cfg: dict, seed: int) -> Dict[str, torch.Tensor]:
    """Random bfloat16 tensors for ``cfg``: matrices N(0, 1.5 / sqrt(in)), norm weights spread around the value they are
    stored around (zero, or one for the plain ones), scales around one half, lam such that channels forget within a
    few tokens or within hundreds."""
    g = torch.Generator().manual_seed(seed)
    out = {}
    for name, shape in tensor_shapes(cfg).items():
        last = name.rsplit(".", 1)[-1]
        spread = 2 * torch.rand(shape, generator=g) - 1
        gauss = torch.randn(shape, generator=g)
        if name.endswith((".q.norm", ".k.norm", ".dkv.norm", ".side.norm")):
            t = 1.0 + 0.3 * spread
        elif last in ("norm1", "norm1b", "norm2", "norm2b") or name == "final.norm":
            t = 0.3 * spread
        elif last in ("ls1", "ls2"):
            t = 0.5 + 0.3 * spread
        elif last == "lam":
            t = -4.0 + 3.0 * spread
        elif last == "b":
            t = 0.3 * gauss
        elif last == "conv":
            t = gauss / math.sqrt(shape[-1])
        elif name in ("embed", "side.embed"):
            t = gauss
        else:
            t = gauss * (1.5 / math.sqrt(shape[-1]))
        out[name] = t.to(torch.bfloat16)
    return out
