"""A new stream made of the stream and the layers' input."""
from __future__ import annotations

from typing import Dict, List, Optional

import torch

from ..ops import kernels
from ..ops.linear import Linear
from .base import StepContext, StreamPart
from .norm import StreamRows
from .registry import register_part
from .spec import ParamSpec


@register_part("stream", "input_mix")
class InputMix(StreamPart):
    """x <- W [x | x0], x0 the stream as it entered the first layer (``ModelSpec.input_mix``; in front of the runs that say
    ``mix_input``).  [x | x0] are the halves of one buffer a step: x0's is filled once (``enter``), x's by the launch that
    wrote the stream last where that launch can (``rows``), else here.  The product's sums stay float32: they are the new
    stream (its partial sums join it in the next norm's launch, as ``pending``)."""

    graph_safe_prompts = True

    def __init__(self, size: int, name: str = "weight", act_dtype: torch.dtype = torch.bfloat16):
        self.size, self.name, self.act_dtype = int(size), name, act_dtype
        self.proj: Optional[Linear] = None

    def param_specs(self) -> List[ParamSpec]:
        return [ParamSpec(self.name, (self.size, 2 * self.size))]

    def load(self, tensors: Dict[str, torch.Tensor], device, dtype) -> None:
        self.proj = Linear(tensors[self.name].to(device))

    def _key(self):
        return ("input_mix", id(self))

    def enter(self, resid: torch.Tensor, ctx: StepContext) -> None:
        """The stream in front of the first layer, kept for the step."""
        both = torch.empty(resid.shape[0], 2 * self.size, dtype=self.act_dtype, device=resid.device)
        kernels.store_rows(resid, both[:, self.size:])
        ctx.shared[self._key()] = (both, StreamRows(both[:, :self.size]))

    def rows(self, ctx: StepContext) -> StreamRows:
        return ctx.shared[self._key()][1]

    def mix(self, resid: torch.Tensor, pending: Optional[torch.Tensor], ctx: StepContext):
        """(the new stream, what is still to be added to it)."""
        both, left = ctx.shared[self._key()]
        if pending is not None:
            for d in (pending if pending.dim() == 3 else (pending,)):
                kernels.residual_add(resid, d)
            left.of = None
        if left.of is not resid:
            kernels.store_rows(resid, left.rows)
        left.of = None
        y = self.proj.sums(both)
        return y[0], y[1:] if y.shape[0] > 1 else None
