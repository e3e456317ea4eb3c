"""Grouped-query attention that norms its queries and keys head by head."""
from __future__ import annotations

from typing import Dict, List, Optional

import torch

from ..ops import kernels
from ..ops.linear import Linear
from .attention_bias import kv_page_tensors
from .base import Mixer, StepContext
from .registry import register_part
from .rotary import HalvesTable
from .spec import CacheSpec, ParamSpec


@register_part("mixer", "normed_attention")
class NormedAttention(Mixer):
    """q = x Wq^T (heads x dk), k = x Wk^T (kv heads x dk), v = x Wv^T (kv heads x dv); no biases.  Every head of q and of k over
    its root mean square (eps inside) times one weight [dk] for all heads of q, one for all of k; then the first
    ``rotary_dim`` entries of every head turned (entry i with entry i + rotary_dim / 2).

      score_ij = (q_i . k_j) scale, softmax over j <= i, heads side by side, Wo

    One product makes q, k and v; one launch norms, turns and stores.  With keys and values of one size the rotary
    attention's kernels serve it (a decode step reads a group's keys once for all its heads), else those for keys and values
    of different sizes.  Norms, angles, scores and softmax are float32 in both engines."""

    graph_safe_prompts = True

    NAMES = {"q": "q", "k": "k", "v": "v", "o": "o", "q_norm": "q.norm", "k_norm": "k.norm"}

    def __init__(self, hidden_size: int, num_heads: int, num_kv_heads: int, key_dim: int, value_dim: int, scale: float,
                 norm_eps: float, rotary_dim: int = 0, base: float = 10000.0, scaling=None, names: Optional[Dict[str, str]] = None,
                 act_dtype: torch.dtype = torch.bfloat16):
        if num_heads % num_kv_heads:
            raise ValueError(f"{num_heads} query heads are not a multiple of {num_kv_heads} kv heads")
        if not (1 <= key_dim <= 1024 and 1 <= value_dim <= 256):
            raise ValueError(f"key size {key_dim} (1 to 1024) or value size {value_dim} (1 to 256) outside what the kernels take")
        if rotary_dim % 2 or not 0 <= rotary_dim <= key_dim:
            raise ValueError(f"{rotary_dim} turned entries must be even and fit a head of {key_dim}")
        self.hidden_size, self.nq, self.nkv, self.dk, self.dv = hidden_size, num_heads, num_kv_heads, key_dim, value_dim
        self.scale, self.norm_eps = float(scale), float(norm_eps)
        self.names = dict(self.NAMES, **(names or {}))
        self.act_dtype = act_dtype
        self.angles = HalvesTable(rotary_dim, base, scaling) if rotary_dim else None
        # what the attention kernels see (ops.attention_bias_fast.choose reads these)
        self.window, self.temp_coef, self.temp_every, self.slope_span = 0, 0.0, 0, 0.0
        self.k_col = self.nq * key_dim
        self.v_col = self.k_col + self.nkv * key_dim
        self.qkv: Optional[Linear] = None
        self.o: Optional[Linear] = None
        self.q_norm = self.k_norm = None
        self.fast = self.fast_two = None                 # matrix-core kernels, chosen at load: one size, two sizes

    def cache_spec(self) -> CacheSpec:
        return CacheSpec("paged_kv", page_tensors=kv_page_tensors(self.nkv, self.dk, self.dv))

    def flops(self, tokens: int, pairs: int) -> float:
        return super().flops(tokens, pairs) + 2.0 * self.nq * (self.dk + self.dv) * pairs

    def param_specs(self) -> List[ParamSpec]:
        D, n = self.hidden_size, self.names
        return [ParamSpec(n["q"], (self.nq * self.dk, D)), ParamSpec(n["k"], (self.nkv * self.dk, D)),
                ParamSpec(n["v"], (self.nkv * self.dv, D)), ParamSpec(n["o"], (D, self.nq * self.dv)),
                ParamSpec(n["q_norm"], (self.dk,), role="norm"), ParamSpec(n["k_norm"], (self.dk,), role="norm")]

    def load(self, tensors: Dict[str, torch.Tensor], device, dtype) -> None:
        n = self.names
        ws = [tensors[n[x]] for x in "qkv"]
        wdt = torch.float32 if any(w.dtype == torch.float32 for w in ws) else ws[0].dtype
        self.qkv = Linear(torch.cat([t.to(wdt) for t in ws], dim=0).to(device))
        self.o = Linear(tensors[n["o"]].to(device))
        self.q_norm = tensors[n["q_norm"]].to(device=device, dtype=torch.float32).contiguous()
        self.k_norm = tensors[n["k_norm"]].to(device=device, dtype=torch.float32).contiguous()
        if self.angles is not None:
            self.angles.load(device)
        if self.act_dtype == torch.bfloat16:
            from ..ops import attention_bias_fast, attention_fast
            if self.dk == self.dv:
                self.fast = attention_fast.choose(self.nq, self.nkv, self.dk, 0)
            if self.fast is None:
                self.fast_two = attention_bias_fast.choose(self)

    def graph_variant(self, ctx: StepContext) -> tuple:
        own = ()
        if self.fast is not None and not ctx.all_decode:
            own = (("normed_attention",) + self.fast.plan(ctx),)
        elif self.fast_two is not None:
            own = (("normed_attention",) + self.fast_two.plan(ctx),)
        return own + super().graph_variant(ctx)

    def forward(self, x: torch.Tensor, ctx: StepContext, cache) -> torch.Tensor:
        return self.o.partial(self.attend(x, ctx, cache))

    def attend(self, x: torch.Tensor, ctx: StepContext, cache) -> torch.Tensor:
        """The heads' outputs [T, H dv] in front of the output projection."""
        bt = ctx.block_tables[cache.group]
        y = self.qkv(x)                                    # [T, H dk | G dk | G dv]
        table = self.angles.table(ctx) if self.angles is not None else None
        q = kernels.qk_norm_store(y, 0, self.k_col, self.v_col, self.nq, self.nkv, self.nkv, self.dk, self.dv, 1,
                                  kernels.QK_NORM_UNIT, self.q_norm, self.k_norm, self.norm_eps, table,
                                  self.angles.rotary_dim if self.angles is not None else 0, ctx.slot_mapping[cache.group], cache.k, cache.v)
        if cache.k.dtype == torch.bfloat16 and self.fast is not None:
            return self.fast(q, cache, bt, ctx, self.scale)
        if cache.k.dtype == torch.bfloat16 and self.fast_two is not None:
            return self.fast_two(q, cache, bt, ctx)
        return kernels.attn_bias_plain(q, cache.k, cache.v, bt, ctx.positions, ctx.token_seq, self.nq, self.nkv, self.dk,
                                       self.dv, self.scale)
