"""A recurrent mixer with one state element a channel: a short causal convolution and a real-gated linear recurrence,
beside a gate branch."""
from __future__ import annotations

from typing import Dict, List, Optional

import torch

from ..ops import kernels
from ..ops.linear import Linear
from .base import Mixer, StepContext
from .registry import register_part
from .spec import CacheSpec, ParamSpec


@register_part("mixer", "gated_linear_recurrence")
class GatedLinearRecurrence(Mixer):
    """[y | x] = W h + b (``width`` channels each); u = conv(x) + bias, a causal convolution of ``taps`` taps a channel (no
    activation).  u is ``parts`` equal pieces; in each r = sigmoid(ra u + ra.b), i = sigmoid(ri u + ri.b) with square matrices.
    Channel by channel

      a = exp(-sharpness r softplus(lam)),      S <- a S + sqrt(1 - a^2) i u,      out = Wo (S * gelu_tanh(y))

    from S = 0.  A request's state (float32, zero for a new request) is S and the last taps - 1 inputs of the convolution,
    together [width, taps] in its state slot.  The gates behind their products, decays, the walk and the state are float32
    in both engines.  A step of single tokens makes convolution, gates, walk and output in one launch."""

    graph_safe_prompts = True

    # In the bfloat16 engine a step with a prompt portion cuts its sequences into chunks that run side by side
    # (``kernels.lru_scan``), its gates on the matrix cores; decided from the step's shape alone.  The 32-bit engine walks
    # every sequence whole, so that its sums do not depend on how a prompt was cut.
    CHUNKED_FROM = 128

    NAMES = {"y": "y", "y_bias": "y.b", "x": "x", "x_bias": "x.b", "conv": "conv", "conv_bias": "conv.b", "ra": "ra", "ra_bias": "ra.b",
             "ri": "ri", "ri_bias": "ri.b", "lam": "lam", "o": "o"}

    def __init__(self, hidden_size: int, width: int, parts: int, taps: int, sharpness: float = 8.0,
                 names: Optional[Dict[str, str]] = None, act_dtype: torch.dtype = torch.bfloat16):
        if width < 1 or parts < 1 or width % parts or width // parts > kernels.LRU_MAX_PART:
            raise ValueError(f"{width} channels are not {parts} equal parts of at most {kernels.LRU_MAX_PART}")
        if not 1 <= taps <= kernels.LRU_MAX_TAPS:
            raise ValueError(f"1 to {kernels.LRU_MAX_TAPS} taps, got {taps}")
        self.hidden_size, self.width, self.num_parts, self.taps, self.sharpness = hidden_size, width, parts, taps, float(sharpness)
        self.names = dict(self.NAMES, **(names or {}))
        self.act_dtype = act_dtype
        self.proj: Optional[Linear] = None               # rows [y | x]
        self.o: Optional[Linear] = None
        self.conv_w = self.conv_b = self.gates = self.gates_out_in = self.r_bias = self.i_bias = self.decay = None

    def cache_spec(self) -> CacheSpec:
        return CacheSpec("state", state_shape=(self.width, self.taps), state_dtype="float32")

    def flops(self, tokens: int, pairs: int) -> float:
        # the products, the two gates' products, the convolution, the update
        return super().flops(tokens, pairs) + tokens * self.width * (4.0 * (self.width // self.num_parts) + 2.0 * self.taps + 2.0)

    def weight_bytes(self) -> int:
        return super().weight_bytes() + sum(t.numel() * t.element_size() for t in self.gates)

    def param_specs(self) -> List[ParamSpec]:
        D, C, P, n = self.hidden_size, self.width, self.num_parts, self.names
        s = C // P
        return [ParamSpec(n["y"], (C, D)), ParamSpec(n["y_bias"], (C,), role="bias"), ParamSpec(n["x"], (C, D)),
                ParamSpec(n["x_bias"], (C,), role="bias"), ParamSpec(n["conv"], (C, self.taps), role="f32", std=0.3),
                ParamSpec(n["conv_bias"], (C,), role="f32"), ParamSpec(n["ra"], (P, s, s)), ParamSpec(n["ra_bias"], (P, s), role="f32"),
                ParamSpec(n["ri"], (P, s, s)), ParamSpec(n["ri_bias"], (P, s), role="f32"),
                ParamSpec(n["lam"], (C,), role="f32", std=1.0), ParamSpec(n["o"], (D, C))]

    def load(self, tensors: Dict[str, torch.Tensor], device, dtype) -> None:
        n = self.names
        ws = [tensors[n["y"]], tensors[n["x"]]]
        wdt = torch.float32 if any(w.dtype == torch.float32 for w in ws) else ws[0].dtype
        bias = torch.cat([tensors[n["y_bias"]].float(), tensors[n["x_bias"]].float()], dim=0).to(device)
        self.proj = Linear(torch.cat([t.to(wdt) for t in ws], dim=0).to(device), bias)
        self.o = Linear(tensors[n["o"]].to(device))
        f32 = lambda k: tensors[n[k]].to(device=device, dtype=torch.float32).contiguous()
        self.conv_w = f32("conv").t().contiguous()          # tap by tap, [taps, width]: neighbouring channels side by side
        self.conv_b, self.r_bias, self.i_bias = f32("conv_bias"), f32("ra_bias").view(-1), f32("ri_bias").view(-1)
        out_in = tuple(tensors[n[k]].to(device=device, dtype=self.act_dtype).contiguous() for k in ("ra", "ri"))
        self.gates = tuple(t.transpose(1, 2).contiguous() for t in out_in)        # [parts, inner, output]
        self.gates_out_in = out_in if self._matrix_cores() else None
        self.decay = (-self.sharpness * torch.nn.functional.softplus(tensors[n["lam"]].double(), threshold=1e4)).to(
            device=device, dtype=torch.float32).contiguous()

    def _matrix_cores(self) -> bool:
        return self.act_dtype == torch.bfloat16 and (self.width // self.num_parts) % 8 == 0

    def forward(self, x: torch.Tensor, ctx: StepContext, cache) -> torch.Tensor:
        return self.o.partial(self.mix(x, ctx, cache))

    def mix(self, h: torch.Tensor, ctx: StepContext, cache) -> torch.Tensor:
        """S * gelu_tanh(y) [T, width] in front of the output projection."""
        C = self.width
        yx = self.proj(h)                                                            # [T, y | x]
        y, x = yx[:, :C], yx[:, C:]
        if ctx.all_decode and ctx.num_tokens == ctx.num_seqs:
            return kernels.lru_step(x, y, self.conv_w, self.conv_b, self.gates, self.r_bias, self.i_bias, self.decay, ctx, cache.state)
        u = kernels.causal_conv(x, C, self.conv_w, self.conv_b, ctx, cache.state, 1, activation="none")
        chunked = self.gates_out_in is not None and ctx.num_tokens >= self.CHUNKED_FROM
        return kernels.lru_scan(u, y, self.gates, self.r_bias, self.i_bias, self.decay, ctx, cache.state, self.taps - 1,
                                w_out_in=self.gates_out_in, chunked=chunked)
