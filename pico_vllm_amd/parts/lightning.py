"""Linear attention with one fixed decay a head behind activations on q, k and v, all heads normed together."""
from __future__ import annotations

from typing import Dict, List, Optional, Sequence

import torch

from ..ops import kernels
from .base import OpenMixer, StepContext
from .gla import GatedLinearAttention
from .registry import register_part
from .spec import CacheSpec, ParamSpec


@register_part("mixer", "lightning_attention")
class LightningAttention(OpenMixer):
    """q = silu(Wq h), k = silu(Wk h) (heads x dk), v = silu(Wv h) (heads x dv), g = Wg h (heads x dv).  Per head, with the
    head's constant decay gamma_h:

      S_t = gamma_h S_(t-1) + k_t v_t^T,      o_t = S_t^T q_t

    The heads side by side are RMS-normed as one row with a weight of the row's size, multiplied by sigmoid(g), and the output
    matrix follows.  The recurrence is the one of ``parts.gla`` with a constant in place of the token's decays; the activations
    are made as the walk reads its operands.  The state [heads, dk, dv] is float32, zero for a new request, and lives in the
    request's state slot; activations, decays, recurrence, state, norm and gate are float32 in both engines."""

    graph_safe_prompts = True
    # tokens of a chunk, and of a step from which on the bfloat16 engine cuts its sequences into chunks: where the matrix cores
    # take them (``kernels.decay_chunks_ok``) and where they do not
    CHUNK, CHUNKED_FROM, WALKED_BELOW = kernels.DECAY_CHUNK, 32, GatedLinearAttention.CHUNKED_FROM

    NAMES = {"q": "q", "k": "k", "v": "v", "g": "g", "o": "o", "norm": "norm"}

    def __init__(self, hidden_size: int, num_heads: int, key_dim: int, value_dim: int, decay: Sequence[float], norm_eps: float,
                 names: Optional[Dict[str, str]] = None, act_dtype: torch.dtype = torch.bfloat16):
        if not 1 <= key_dim <= kernels.GLA_MAX_KEY_DIM:
            raise ValueError(f"key size {key_dim} outside what the recurrence kernel takes (1 to {kernels.GLA_MAX_KEY_DIM})")
        if len(decay) != num_heads or not all(0.0 < float(g) <= 1.0 for g in decay):
            raise ValueError(f"one decay in (0, 1] a head, got {len(decay)} for {num_heads} heads")
        self.hidden_size, self.heads, self.dk, self.dv = hidden_size, num_heads, key_dim, value_dim
        self.decay_values, self.norm_eps = tuple(float(g) for g in decay), float(norm_eps)
        self.names = dict(self.NAMES, **(names or {}))
        self.act_dtype = act_dtype
        self.decay = self.norm_weight = None
        hk, hv = num_heads * key_dim, num_heads * value_dim
        self.k_col, self.v_col, self.g_col = hk, 2 * hk, 2 * hk + hv

    def cache_spec(self) -> CacheSpec:
        return CacheSpec("state", state_shape=(self.heads, self.dk, self.dv), state_dtype="float32")

    def flops(self, tokens: int, pairs: int) -> float:
        return super().flops(tokens, pairs) + tokens * self.heads * self.dk * 5.0 * self.dv

    def in_matrices(self) -> List[tuple]:
        n, hk, hv = self.names, self.heads * self.dk, self.heads * self.dv
        return [(n["q"], hk), (n["k"], hk), (n["v"], hv), (n["g"], hv)]

    def out_matrix(self) -> tuple:
        return self.names["o"], self.heads * self.dv

    def core_params(self) -> List[ParamSpec]:
        return [ParamSpec(self.names["norm"], (self.heads * self.dv,), role="norm")]

    def load_core(self, tensors: Dict[str, torch.Tensor], device, dtype, scale: float = 1.0) -> None:
        self.decay = torch.tensor(self.decay_values, dtype=torch.float64).to(torch.float32).to(device)
        self.norm_weight = (tensors[self.names["norm"]].to(device=device, dtype=torch.float32) * scale).contiguous()

    def core(self, y: torch.Tensor, col: int, ctx: StepContext, cache, out: torch.Tensor) -> None:
        # the bfloat16 engine cuts long portions into chunks that run side by side (the same sums in another order);
        # the 32-bit engine walks every sequence whole
        at = (col, col + self.k_col, col + self.v_col)
        least = self.CHUNKED_FROM if kernels.decay_chunks_ok(y, *at, self.dk, self.dv) else self.WALKED_BELOW
        chunked = self.act_dtype == torch.bfloat16 and not ctx.all_decode and ctx.num_tokens >= least
        o = kernels.gla_scan(y, *at, None, ctx.cu_seqlens, ctx.state_slots, cache.state,
                             ctx.num_seqs, self.heads, self.dk, self.dv, 1.0, chunk=self.CHUNK if chunked else 0,
                             head_decay=self.decay, silu=True)
        kernels.gated_row_norm(o, y, col + self.g_col, self.norm_weight, self.norm_eps, out=out)
