"""A layer's own input of the token: a row of a table that all layers share, gated by the stream."""
from __future__ import annotations

from typing import Dict, List, Optional

import torch

from ..ops.linear import Linear
from .base import Part, StepContext, StreamPart
from .registry import register_part
from .spec import ParamSpec

TOKEN_TABLE = "token_table"      # in a step's shared things: the table


@register_part("stream", "token_table")
class TokenTable(StreamPart):
    """Holds a table with a row a token, one part of the row for every layer, and hands it to the layers' token inputs; the
    stream passes unchanged.  Nothing is gathered here: a layer's launch reads the entries it needs."""
    graph_safe_prompts = True

    def __init__(self, rows: int, size: int, name: str = "weight", act_dtype: torch.dtype = torch.bfloat16):
        self.rows, self.size, self.name = int(rows), int(size), name
        self.table: Optional[torch.Tensor] = None

    def param_specs(self) -> List[ParamSpec]:
        return [ParamSpec(self.name, (self.rows, self.size))]

    def load(self, tensors: Dict[str, torch.Tensor], device, dtype) -> None:
        self.table = tensors[self.name].to(device).contiguous()

    def weight_bytes(self) -> int:
        return 0                     # a step reads one row a token, not the table

    def forward(self, resid: torch.Tensor, ctx: StepContext) -> torch.Tensor:
        ctx.shared[TOKEN_TABLE] = self.table
        return resid


@register_part("token_input", "gated_token_row")
class GatedTokenRow(Part):
    """y = Wp (gelu_tanh(Wg x) * e), e = the ``dim`` entries from ``column`` of the token's row of the shared table; y joins the
    stream as y / sqrt(mean(y^2) + eps) * weight, which the arrangement does (``norm_weight``, ``norm_eps``).
    ``names``: the tensors' names behind the part's prefix."""
    graph_safe_prompts = True

    NAMES = {"gate": "gate", "proj": "proj", "norm": "norm"}

    def __init__(self, size: int, dim: int, column: int, norm_eps: float, names: Optional[Dict[str, str]] = None,
                 act_dtype: torch.dtype = torch.bfloat16):
        self.size, self.dim, self.column, self.norm_eps = int(size), int(dim), int(column), float(norm_eps)
        self.names = dict(self.NAMES, **(names or {}))
        self.gate: Optional[Linear] = None
        self.proj: Optional[Linear] = None
        self.norm_weight: Optional[torch.Tensor] = None

    def param_specs(self) -> List[ParamSpec]:
        n = self.names
        return [ParamSpec(n["gate"], (self.dim, self.size)), ParamSpec(n["proj"], (self.size, self.dim)),
                ParamSpec(n["norm"], (self.size,), role="norm")]

    def load(self, tensors: Dict[str, torch.Tensor], device, dtype) -> None:
        n = self.names
        self.gate, self.proj = Linear(tensors[n["gate"]].to(device)), Linear(tensors[n["proj"]].to(device))
        self.norm_weight = tensors[n["norm"]].to(device=device, dtype=torch.float32).contiguous()

    def forward(self, x: torch.Tensor, ctx: StepContext) -> torch.Tensor:
        """x: the stream's rows in the activations' dtype; returns y in front of its norm, [T, H] or partial sums of it."""
        g = self.gate.gelu_token(x, ctx.token_ids[:ctx.num_tokens], ctx.shared[TOKEN_TABLE], self.column)
        return self.proj.partial(g)
