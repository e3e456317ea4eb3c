"""Two mixers side by side that read the same input."""
from __future__ import annotations

from typing import Dict, List, Optional

import torch

from ..ops.linear import Linear
from .base import Mixer, OpenMixer, StepContext
from .registry import build_part, register_part
from .spec import CacheSpec, ParamSpec, PartSpec


@register_part("mixer", "mixer_pair")
class MixerPair(Mixer):
    """out = (rms(left(h)) * w_left + rms(right(h)) * w_right) / 2: two mixers of any kinds, each with the cache or state
    it asks for, their outputs RMS-normed over the model width with a weight each before they are averaged.  The pair
    hands both outputs and weights to an arrangement that norms and sums them in one launch (``forward_pair``; the
    arrangement "postnorm" does).  ``left`` / ``right``: the two mixers as PartSpecs; their tensors stand behind
    ``prefixes``; ``out_names``: the two weights."""

    graph_safe_prompts = True

    def __init__(self, hidden_size: int, left: PartSpec, right: PartSpec, norm_eps: float, prefixes=("left", "right"),
                 out_names=("left.out", "right.out"), act_dtype: torch.dtype = torch.bfloat16):
        self.hidden_size, self.norm_eps = hidden_size, float(norm_eps)
        self.prefixes, self.out_names = tuple(prefixes), tuple(out_names)
        self.left = build_part("mixer", left, act_dtype=act_dtype)
        self.right = build_part("mixer", right, act_dtype=act_dtype)
        self.act_dtype = act_dtype
        self.w_left: Optional[torch.Tensor] = None
        self.w_right: Optional[torch.Tensor] = None

    def cache_spec(self) -> CacheSpec:
        return CacheSpec("several", parts=(self.left.cache_spec(), self.right.cache_spec()))

    def param_specs(self) -> List[ParamSpec]:
        out = []
        for pre, part in zip(self.prefixes, (self.left, self.right)):
            out += [ParamSpec(f"{pre}.{p.name}", p.shape, p.role, p.std) for p in part.param_specs()]
        return out + [ParamSpec(n, (self.hidden_size,), role="norm") for n in self.out_names]

    def load(self, tensors: Dict[str, torch.Tensor], device, dtype) -> None:
        for pre, part in zip(self.prefixes, (self.left, self.right)):
            part.load({p.name: tensors[f"{pre}.{p.name}"] for p in part.param_specs()}, device, dtype)
        self.w_left, self.w_right = (tensors[n].to(device=device, dtype=torch.float32).contiguous() for n in self.out_names)

    def forward_pair(self, x: torch.Tensor, ctx: StepContext, cache):
        """(left's output, its weight, right's output, its weight); the outputs as their output projections leave them
        ([T, H], or float32 stacks of partial sums)."""
        left_cache, right_cache = cache
        return self.left.forward(x, ctx, left_cache), self.w_left, self.right.forward(x, ctx, right_cache), self.w_right

    def forward(self, x: torch.Tensor, ctx: StepContext, cache) -> torch.Tensor:
        raise NotImplementedError("a pair of mixers runs in an arrangement that norms and sums its two outputs (forward_pair)")


@register_part("mixer", "mixer_sum")
class MixerSum(Mixer):
    """out = left_scale left(h) + right_scale right(h): two open mixers (``base.OpenMixer``), each with the cache or state it asks
    for, whose products are made together: ONE product makes the columns of both from h, both cores write side by side into
    one buffer (with the scales on what they write, in float32 in front of its rounding), and ONE product over that buffer is
    the sum.  Each side's columns start on eight entries (rows of zeros between them), so that what reads them may read
    whole words.  A left side with ``core_beside`` may run both cores in launches of its own (a step of single tokens, where
    every launch is a chain of latencies).  ``left`` / ``right``: the two mixers as PartSpecs; their tensors stand behind ``prefixes``."""

    graph_safe_prompts = True
    ALIGN = 8

    def __init__(self, hidden_size: int, left: PartSpec, right: PartSpec, left_scale: float = 1.0, right_scale: float = 1.0,
                 prefixes=("left", "right"), act_dtype: torch.dtype = torch.bfloat16):
        self.hidden_size, self.prefixes, self.act_dtype = hidden_size, tuple(prefixes), act_dtype
        self.scales = (float(left_scale), float(right_scale))
        self.left = build_part("mixer", left, act_dtype=act_dtype)
        self.right = build_part("mixer", right, act_dtype=act_dtype)
        for part in self.sides:
            if not isinstance(part, OpenMixer):
                raise TypeError(f"a sum of mixers makes their products together: {type(part).__name__} does not open its own")
        up = lambda n: -(-n // self.ALIGN) * self.ALIGN
        rows = [sum(r for _, r in p.in_matrices()) for p in self.sides]
        cols = [p.out_matrix()[1] for p in self.sides]
        self.in_rows, self.out_cols = rows, cols
        self.in_at, self.in_total = (0, up(rows[0])), up(rows[0]) + up(rows[1])
        self.out_at, self.out_total = (0, up(cols[0])), up(cols[0]) + up(cols[1])
        self.proj: Optional[Linear] = None
        self.o: Optional[Linear] = None

    @property
    def sides(self):
        return (self.left, self.right)

    def cache_spec(self) -> CacheSpec:
        return CacheSpec("several", parts=tuple(p.cache_spec() for p in self.sides))

    def param_specs(self) -> List[ParamSpec]:
        return [ParamSpec(f"{pre}.{p.name}", p.shape, p.role, p.std) for pre, part in zip(self.prefixes, self.sides)
                for p in part.param_specs()]

    def load(self, tensors: Dict[str, torch.Tensor], device, dtype) -> None:
        D = self.hidden_size
        mine = [{p.name: tensors[f"{pre}.{p.name}"] for p in part.param_specs()} for pre, part in zip(self.prefixes, self.sides)]
        ws = [[t[n] for n, _ in part.in_matrices()] + [t[part.out_matrix()[0]]] for part, t in zip(self.sides, mine)]
        wdt = torch.float32 if any(w.dtype == torch.float32 for side in ws for w in side) else ws[0][0].dtype
        proj = torch.zeros(self.in_total, D, dtype=wdt)
        o = torch.zeros(D, self.out_total, dtype=wdt)
        for k, side in enumerate(ws):
            proj[self.in_at[k]:self.in_at[k] + self.in_rows[k]] = torch.cat([w.to(wdt) for w in side[:-1]], dim=0)
            o[:, self.out_at[k]:self.out_at[k] + self.out_cols[k]] = side[-1].to(wdt)
        self.proj, self.o = Linear(proj.to(device)), Linear(o.to(device))
        for part, t, scale in zip(self.sides, mine, self.scales):
            part.load_core(t, device, dtype, scale)

    def forward(self, x: torch.Tensor, ctx: StepContext, cache) -> torch.Tensor:
        y = self.proj(x)
        whole = sum(self.out_cols) == self.out_total
        out = (torch.empty if whole else torch.zeros)(x.shape[0], self.out_total, dtype=x.dtype, device=x.device)
        outs = [out[:, c:c + n] for c, n in zip(self.out_at, self.out_cols)]
        beside = getattr(self.left, "core_beside", None)
        if beside is None or not beside(self.right, y, *self.in_at, ctx, *cache, *outs):
            for part, own, i, o in zip(self.sides, cache, self.in_at, outs):
                part.core(y, i, ctx, own, o)
        return self.o.partial(out)
