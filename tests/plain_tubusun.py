"""A plain, slow implementation of the Tubusun decoder: whole sequences, no cache, float64 on the CPU, one function per
mechanism, written from the design's equations and sharing no code with the package.

Notation: T tokens at positions 0 .. T - 1, width D, eps the model's norm constant, rms(x) = x / sqrt(mean(x^2) + eps).  A
weight dict maps checkpoint names ('l3.mix.left.q', 'loop.step', ..) to tensors; linear weights are [out, in] and applied as
x W^T.

  model:   x = E[token] a.  Layers in order, the looped span several times in a row; in front of pass t of it x += step[t].
  layer i: x += rms(mixer(rms(x) n1)) n1b; if it has a feed-forward x += rms(ff(rms(x) n2)) n2b.
  mixer:   ls attention(h) + rs lightning(h), both of the same h.
  logits = cap tanh(rms(x) n E^T / cap).
"""
from __future__ import annotations

import math
from typing import Dict, List, Optional, Tuple

import torch

F64 = torch.float64

# A yardstick for what rounding alone does: with ``forward(..., rounding=f)`` every activation that passes from one part
# to the next (a product's output, an attention's, the stream as a product reads it) goes through f.
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


def silu(z: torch.Tensor) -> torch.Tensor:
    return z / (1.0 + torch.exp(-z))


def gelu_erf(z: torch.Tensor) -> torch.Tensor:
    return 0.5 * z * (1.0 + torch.erf(z / math.sqrt(2.0)))


# ---- attention: rotation, then unit norms; a window; a sink a head; a gate a head -------------------------------------------
def rotate_pairs(x: torch.Tensor, positions: torch.Tensor, dims: int, base: float) -> torch.Tensor:
    """x [T, heads, d]: of the first dims entries, 2i goes with 2i + 1, turned by position base^(-2i / dims)."""
    if not dims:
        return x
    f = torch.tensor([base ** (-2.0 * i / dims) for i in range(dims // 2)], dtype=x.dtype)
    a = positions.to(x.dtype).view(-1, 1, 1) * f
    c, s = torch.cos(a), torch.sin(a)
    u, v = x[..., 0:dims:2], x[..., 1:dims:2]
    turned = torch.stack([u * c - v * s, v * c + u * s], dim=-1).flatten(-2)
    return torch.cat([turned, x[..., dims:]], dim=-1)


def seen(T: int, window: int) -> torch.Tensor:
    """[query, key]: whether a query sees a key: not behind it, and with a window at most window - 1 in front."""
    d = torch.arange(T).view(-1, 1) - torch.arange(T).view(1, -1)
    return (d >= 0) & (d < window) if window else d >= 0


def sink_softmax(s: torch.Tensor, visible: torch.Tensor, sink: torch.Tensor) -> torch.Tensor:
    """exp(s_ij) / (exp(sink) + sum over the visible keys)."""
    s = s.masked_fill(~visible, float("-inf"))
    m = torch.maximum(s.max(-1, keepdim=True).values, sink)
    e = torch.exp(s - m)
    return e / (e.sum(-1, keepdim=True) + torch.exp(sink - m))


def attention(h: torch.Tensor, w: Dict[str, torch.Tensor], m: dict, eps: float, first_pos: int = 0) -> torch.Tensor:
    T = h.shape[0]
    H, G, d, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    pos = torch.arange(first_pos, first_pos + T)
    rot = m.get("rot") or {}
    ready = lambda x: act(rms(rotate_pairs(x, pos, rot.get("dims", 0), rot.get("base", 1.0)), eps))
    q = ready(act(h @ w["q"].T).view(T, H, d))
    k = ready(act(h @ w["k"].T).view(T, G, d))
    v = act(h @ w["v"].T).view(T, G, dv)
    gate = torch.sigmoid(act(h @ w["g"].T))                                # [T, H]
    visible = seen(T, (m.get("mask") or {}).get("size", 0))
    out = torch.zeros(T, H, dv, dtype=h.dtype)
    for a in range(H):
        g = a // (H // G)
        p = sink_softmax((q[:, a] @ k[:, g].T) * m["scale"], visible, w["sink"][a])
        out[:, a] = (p @ v[:, g]) * gate[:, a:a + 1]
    return out.reshape(T, H * dv)


# ---- linear attention with a fixed decay a head -------------------------------------------------------------------------
def decayed_sums(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, decay, S0: Optional[torch.Tensor] = None
                 ) -> Tuple[torch.Tensor, torch.Tensor]:
    """q, k [T, H, d], v [T, H, dv]: S_t = decay_h S_(t-1) + k_t v_t^T, o_t = S_t^T q_t; (o [T, H, dv], the last S)."""
    T, H, d = k.shape
    S = torch.zeros(H, d, v.shape[-1], dtype=v.dtype) if S0 is None else S0
    g = torch.as_tensor(decay, dtype=v.dtype).view(H, 1, 1)
    out = torch.zeros_like(v)
    for t in range(T):
        S = g * S + k[t].unsqueeze(-1) * v[t].unsqueeze(-2)
        out[t] = (S * q[t].unsqueeze(-1)).sum(1)
    return out, S


def lightning(h: torch.Tensor, w: Dict[str, torch.Tensor], m: dict, eps: float, first_pos: int = 0) -> torch.Tensor:
    T = h.shape[0]
    H, d, dv = m["heads"], m["dim"], m["vdim"]
    q, k = (act(silu(act(h @ w[n].T))).view(T, H, d) for n in "qk")
    v = act(silu(act(h @ w["v"].T))).view(T, H, dv)
    o, _ = decayed_sums(q, k, v, m["decay"])
    return rms(o.reshape(T, H * dv), eps) * w["norm"] * torch.sigmoid(act(h @ w["g"].T))


def parallel(h: torch.Tensor, w: Dict[str, torch.Tensor], m: dict, eps: float, first_pos: int = 0) -> torch.Tensor:
    left, right = under("left", w), under("right", w)
    a = act(attention(h, left, m["left"], eps, first_pos)) @ left["o"].T
    b = act(lightning(h, right, m["right"], eps, first_pos)) @ right["o"].T
    return act(m.get("left_scale", 1.0) * a + m.get("right_scale", 1.0) * b)


# ---- feed-forwards ------------------------------------------------------------------------------------------------------
def dense_mlp(h: torch.Tensor, w: Dict[str, torch.Tensor]) -> torch.Tensor:
    return act(act(gelu_erf(h @ w["up"].T + w["up.b"])) @ w["down"].T + w["down.b"])


def route(h: torch.Tensor, router: torch.Tensor, r: dict) -> Tuple[torch.Tensor, torch.Tensor]:
    """(experts [T, top], their weights): scores sigmoid(z); the experts of the best groups (a group's score: the sum of its
    two largest), the largest scores among them; the lower index among equals."""
    s = torch.sigmoid(h @ router.T)
    T, E = s.shape
    may = s
    gr = r.get("groups")
    if gr:
        n = E // gr["count"]
        score = s.view(T, gr["count"], n).sort(-1, descending=True).values[..., :2].sum(-1)
        best = torch.argsort(score, dim=-1, descending=True, stable=True)[:, :gr["keep"]]
        allowed = torch.zeros(T, gr["count"], dtype=torch.bool).scatter_(1, best, True)
        may = s.masked_fill(~allowed.repeat_interleave(n, dim=1), -1.0)
    chosen = torch.argsort(may, dim=-1, descending=True, stable=True)[:, :r["top"]]
    return chosen, torch.gather(s, 1, chosen)


def route_margin(h: torch.Tensor, router: torch.Tensor, r: dict) -> torch.Tensor:
    """How far every token's choice is from another one: the smallest gap, of scores, between what is chosen and what is not
    (among groups, and among the experts that may be chosen).  A small value: rounding may choose the other."""
    s = torch.sigmoid(h @ router.T)
    T, E = s.shape
    gap = torch.full((T,), float("inf"), dtype=s.dtype)
    may, cols = s, E
    gr = r.get("groups")
    if gr:
        n = E // gr["count"]
        score = s.view(T, gr["count"], n).sort(-1, descending=True).values[..., :2].sum(-1)
        order = score.sort(-1, descending=True).values
        if gr["keep"] < gr["count"]:
            gap = torch.minimum(gap, (order[:, gr["keep"] - 1] - order[:, gr["keep"]]) / 2)
        best = torch.argsort(score, dim=-1, descending=True, stable=True)[:, :gr["keep"]]
        allowed = torch.zeros(T, gr["count"], dtype=torch.bool).scatter_(1, best, True)
        may, cols = s.masked_fill(~allowed.repeat_interleave(n, dim=1), -1.0), gr["keep"] * n
    if r["top"] < cols:
        order = may.sort(-1, descending=True).values
        gap = torch.minimum(gap, order[:, r["top"] - 1] - order[:, r["top"]])
    return gap


def expert(h: torch.Tensor, gate: torch.Tensor, up: torch.Tensor, down: torch.Tensor, limit: float) -> torch.Tensor:
    g = torch.clamp(h @ gate.T, max=limit)
    u = torch.clamp(h @ up.T, min=-limit, max=limit)
    return act(g * torch.sigmoid(1.702 * g) * (u + 1.0)) @ down.T


def routed_mlp(h: torch.Tensor, w: Dict[str, torch.Tensor], f: dict) -> torch.Tensor:
    chosen, ws = route(h, w["router"], f["router"])
    out = torch.zeros_like(h)
    for e in range(f["router"]["experts"]):
        rows, slot = (chosen == e).nonzero(as_tuple=True)
        if len(rows):
            y = expert(h[rows], w[f"e{e}.gate"], w[f"e{e}.up"], w[f"e{e}.down"], f["expert"]["limit"])
            out[rows] += ws[rows, slot].unsqueeze(-1) * y
    return act(out)


def feed_forward(h: torch.Tensor, w: Dict[str, torch.Tensor], f: dict) -> torch.Tensor:
    return dense_mlp(h, w) if f["kind"] == "dense" else routed_mlp(h, w, f)


# ---- order, model -------------------------------------------------------------------------------------------------------
def under(p: str, ws: Dict[str, torch.Tensor]) -> Dict[str, torch.Tensor]:
    return {n[len(p) + 1:]: t for n, t in ws.items() if n.startswith(p + ".")}


def run_order(layers: int, loop: Optional[dict]) -> List[Tuple[int, Optional[int]]]:
    """(layer, the number of the pass that starts in front of it or None)."""
    if not loop or loop["start"] >= loop["stop"]:
        return [(i, None) for i in range(layers)]
    a, b = loop["start"], loop["stop"]
    return ([(i, None) for i in range(a)] + [(i, t if i == a else None) for t in range(loop["times"]) for i in range(a, b)]
            + [(i, None) for i in range(b, layers)])


def forward(cfg: dict, weights: Dict[str, torch.Tensor], tokens: List[int], dtype=F64, trace: Optional[list] = None,
            rounding=None, margins: Optional[list] = None) -> torch.Tensor:
    """Logits [T, vocab] of one sequence from position 0.  ``trace``: a list that receives the stream after every layer
    run.  ``rounding``: a function that every activation between the parts goes through (the stream itself stays as it
    is; what a product reads of it is rounded).  ``margins``: a list that receives ``route_margin`` of every routed layer."""
    global _rounding
    _rounding = rounding
    try:
        return _forward(cfg, weights, tokens, dtype, trace, margins)
    finally:
        _rounding = None


def _forward(cfg, weights, tokens, dtype, trace, margins):
    W = {n: (t.to(dtype) if t.is_floating_point() else t) for n, t in weights.items()}
    eps = cfg["norm"]["eps"]
    x = W["embed"][torch.tensor(tokens)] * (cfg.get("embedding") or {}).get("scale", 1.0)
    for i, start in run_order(len(cfg["layers"]), cfg.get("loop")):
        if start is not None:
            x = x + W["loop.step"][start]
        layer, lw = cfg["layers"][i], under(f"l{i}", W)
        y = parallel(act(rms(x, eps) * lw["norm1"]), under("mix", lw), layer["mixer"], eps)
        x = x + rms(y, eps) * lw["norm1b"]
        if layer.get("mlp"):
            h = act(rms(x, eps) * lw["norm2"])
            if margins is not None and layer["mlp"]["kind"] == "moe":
                margins.append(route_margin(h, lw["mlp.router"], layer["mlp"]["router"]))
            x = x + rms(feed_forward(h, under("mlp", lw), layer["mlp"]), eps) * lw["norm2b"]
        if trace is not None:
            trace.append(x.clone())
    z = act(rms(x, eps) * W["final.norm"]) @ W["embed"].T
    cap = cfg.get("logit_softcap")
    return cap * torch.tanh(z / cap) if cap else z


# ---- random models -----------------------------------------------------------------------------------------------------
def tensor_shapes(cfg: dict) -> Dict[str, tuple]:
    """Name -> shape of every tensor a model of this configuration holds."""
    D, V = cfg["width"], cfg["vocab"]
    out = {"embed": (V, D), "final.norm": (D,)}
    if cfg.get("loop"):
        out["loop.step"] = (cfg["loop"]["times"], D)
    for i, layer in enumerate(cfg["layers"]):
        p, l, r = f"l{i}.", f"l{i}.mix.left.", f"l{i}.mix.right."
        out.update({p + n: (D,) for n in ("norm1", "norm1b", "norm2", "norm2b")})
        m = layer["mixer"]["left"]
        H, G, d, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
        out.update({l + "q": (H * d, D), l + "k": (G * d, D), l + "v": (G * dv, D), l + "sink": (H,), l + "g": (H, D), l + "o": (D, H * dv)})
        m = layer["mixer"]["right"]
        H, d, dv = m["heads"], m["dim"], m["vdim"]
        out.update({r + "q": (H * d, D), r + "k": (H * d, D), r + "v": (H * dv, D), r + "g": (H * dv, D), r + "o": (D, H * dv),
                    r + "norm": (H * dv,)})
        f = layer.get("mlp")
        if f and f["kind"] == "dense":
            out.update({p + "mlp.up": (f["ff"], D), p + "mlp.up.b": (f["ff"],), p + "mlp.down": (D, f["ff"]), p + "mlp.down.b": (D,)})
        elif f:
            for e in range(f["router"]["experts"]):
                out.update({p + f"mlp.e{e}.gate": (f["expert"]["ff"], D), p + f"mlp.e{e}.up": (f["expert"]["ff"], D),
                            p + f"mlp.e{e}.down": (D, f["expert"]["ff"])})
            out[p + "mlp.router"] = (f["router"]["experts"], D)
    return out


def random_model(cfg: dict, seed: int) -> Dict[str, torch.Tensor]:
    """Random bfloat16 tensors for ``cfg``: matrices N(0, 1.5 / sqrt(in)), norm weights spread around one, sinks of a few
    units, passes' vectors of the embeddings' size."""
    g = torch.Generator().manual_seed(seed)
    out = {}
    for name, shape in tensor_shapes(cfg).items():
        last = name.rsplit(".", 1)[-1]
        spread = 2 * torch.rand(shape, generator=g) - 1
        gauss = torch.randn(shape, generator=g)
        if last in ("norm", "norm1", "norm1b", "norm2", "norm2b"):
            t = 1.0 + 0.3 * spread
        elif last == "sink":
            t = 2.0 * gauss
        elif last == "b":
            t = 0.3 * gauss
        elif name == "embed":
            t = gauss * 1.5 / math.sqrt(shape[-1]) if cfg.get("logit_softcap") else gauss
        elif name == "loop.step":
            t = 0.7 * gauss
        else:
            t = gauss * (1.5 / math.sqrt(shape[-1]))
        out[name] = t.to(torch.bfloat16)
    return out
