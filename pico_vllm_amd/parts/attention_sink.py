"""Grouped-query attention in a sliding window with a learned sink and a gate a head, whose queries and keys have unit length."""
from __future__ import annotations

from typing import Dict, List, Optional

import torch

from ..ops import kernels
from .attention_bias import kv_page_tensors
from .base import OpenMixer, StepContext
from .lightning import LightningAttention
from .registry import register_part
from .rotary import PairsTable
from .spec import CacheSpec, ParamSpec


@register_part("mixer", "sink_attention")
class SinkAttention(OpenMixer):
    """q = Wq h (heads x dk), k = Wk h (kv heads x dk), v = Wv h (kv heads x dv), g = Wg h (one number a head); no biases.  The
    first ``rotary_dim`` entries of every head of q and k are turned (entry 2 i with entry 2 i + 1, by position
    base^(-2 i / rotary_dim)), then every head of q and k is divided by its root mean square over dk (eps inside, no weight).

      s_ij = (q_i . k_j) scale;   key j <= i is seen iff i - j < window   (window 0: every j <= i)
      p_ij = exp(s_ij) / (exp(sink_h) + sum_j exp(s_ij))                  (a learned number a head, with neither key nor value)

    Head h's output is multiplied by sigmoid(g_h); query head h reads kv head h // (H / G).  A rotation keeps a head's
    length, so one launch norms, turns and stores.  Norms, angles, scores, softmax and sink are float32 in both engines."""

    graph_safe_prompts = True

    NAMES = {"q": "q", "k": "k", "v": "v", "g": "g", "o": "o", "sink": "sink"}

    def __init__(self, hidden_size: int, num_heads: int, num_kv_heads: int, key_dim: int, value_dim: int, scale: float,
                 norm_eps: float, window: int = 0, rotary_dim: int = 0, base: float = 10000.0,
                 names: Optional[Dict[str, str]] = None, act_dtype: torch.dtype = torch.bfloat16):
        if num_heads % num_kv_heads:
            raise ValueError(f"{num_heads} query heads are not a multiple of {num_kv_heads} kv heads")
        if not (1 <= key_dim <= 1024 and 1 <= value_dim <= 256):
            raise ValueError(f"key size {key_dim} (1 to 1024) or value size {value_dim} (1 to 256) outside what the kernels take")
        if window < 0 or rotary_dim % 2 or not 0 <= rotary_dim <= key_dim:
            raise ValueError(f"window {window} must not be negative; {rotary_dim} turned entries must be even and fit a head of {key_dim}")
        self.hidden_size, self.nq, self.nkv, self.dk, self.dv = hidden_size, num_heads, num_kv_heads, key_dim, value_dim
        self.scale, self.norm_eps, self.window = float(scale), float(norm_eps), int(window)
        self.names = dict(self.NAMES, **(names or {}))
        self.act_dtype = act_dtype
        self.angles = PairsTable(rotary_dim, base) if rotary_dim else None
        # what the attention kernels see (ops.attention_bias_fast.choose reads these)
        self.temp_coef, self.temp_every, self.slope_span = 0.0, 0, 0.0
        self.sink, self.gated, self.gate_heads, self.out_scale = True, True, True, 1.0
        self.k_col = self.nq * key_dim
        self.v_col = self.k_col + self.nkv * key_dim
        self.g_col = self.v_col + self.nkv * value_dim
        self.sinks: Optional[torch.Tensor] = None
        self.fast = None                                 # matrix-core kernel, chosen at load

    def cache_spec(self) -> CacheSpec:
        return CacheSpec("paged_kv", window=self.window, page_tensors=kv_page_tensors(self.nkv, self.dk, self.dv))

    def flops(self, tokens: int, pairs: int) -> float:
        if self.window:
            pairs = min(pairs, tokens * self.window)
        return super().flops(tokens, pairs) + 2.0 * self.nq * (self.dk + self.dv) * pairs

    def in_matrices(self) -> List[tuple]:
        n = self.names
        return [(n["q"], self.nq * self.dk), (n["k"], self.nkv * self.dk), (n["v"], self.nkv * self.dv), (n["g"], self.nq)]

    def out_matrix(self) -> tuple:
        return self.names["o"], self.nq * self.dv

    def core_params(self) -> List[ParamSpec]:
        return [ParamSpec(self.names["sink"], (self.nq,), role="f32", std=1.0)]

    def load_core(self, tensors: Dict[str, torch.Tensor], device, dtype, scale: float = 1.0) -> None:
        self.sinks = tensors[self.names["sink"]].to(device=device, dtype=torch.float32).contiguous()
        self.out_scale = float(scale)
        if self.angles is not None:
            self.angles.load(device)
        if self.act_dtype == torch.bfloat16:
            from ..ops import attention_bias_fast
            self.fast = attention_bias_fast.choose(self)

    def graph_variant(self, ctx: StepContext) -> tuple:
        own = (("sink_attention",) + self.fast.plan(ctx),) if self.fast is not None else ()
        return own + super().graph_variant(ctx)

    def core(self, y: torch.Tensor, col: int, ctx: StepContext, cache, out: torch.Tensor) -> None:
        bt = ctx.block_tables[cache.group]
        table = self.angles.table(ctx) if self.angles is not None else None
        q = kernels.qk_norm_store(y, col, col + self.k_col, col + self.v_col, self.nq, self.nkv, self.nkv, self.dk, self.dv, 1,
                                  kernels.QK_NORM_UNIT, None, None, self.norm_eps, table,
                                  self.angles.rotary_dim if self.angles is not None else 0, ctx.slot_mapping[cache.group],
                                  cache.k, cache.v, pairs=True)
        gate = y[:, col + self.g_col:]
        if self.fast is not None and cache.k.dtype == torch.bfloat16 and out.stride(0) % 4 == 0 and out.data_ptr() % 8 == 0:
            self.fast(q, cache, bt, ctx, gate=gate, out=out)
            return
        kernels.attn_bias_plain(q, cache.k, cache.v, bt, ctx.positions, ctx.token_seq, self.nq, self.nkv, self.dk, self.dv, self.scale,
                                self.window, gate=gate, gate_heads=True, sinks=self.sinks, out=out, out_scale=self.out_scale)

    def core_beside(self, other: OpenMixer, y: torch.Tensor, col: int, other_col: int, ctx: StepContext, cache, other_cache,
                    out: torch.Tensor, other_out: torch.Tensor) -> bool:
        """This core and a ``LightningAttention``'s in shared launches, for a step of single tokens in bfloat16: norm, rotation
        and store beside the walk of a token; attention over cut keys; the pieces put together beside the norm over all heads.
        False: nothing was done (another mixer, another step, sizes that the launches do not take)."""
        if not (isinstance(other, LightningAttention) and self.fast is not None and cache.k.dtype == torch.bfloat16 and ctx.all_decode
                and ctx.num_tokens == ctx.num_seqs and other.heads * other.dv <= kernels.PAIR_MAX_ROW):
            return False
        split, pieces, shape = self.fast.plan(ctx)
        if shape or not split or not 2 <= pieces <= kernels.PAIR_MAX_PIECES:
            return False
        table = self.angles.table(ctx) if self.angles is not None else None
        q, o = kernels.pair_open(
            y, (col, col + self.k_col, col + self.v_col, self.nq, self.nkv, self.dk, self.dv), self.norm_eps, table,
            self.angles.rotary_dim if self.angles is not None else 0, ctx.slot_mapping[cache.group], cache.k, cache.v,
            (other_col, other_col + other.k_col, other_col + other.v_col, other.heads, other.dk, other.dv), ctx.state_slots, other.decay,
            other_cache.state)
        parts = self.fast.run(q, cache.k, cache.v, ctx.block_tables[cache.group], ctx.cu_seqlens, ctx.positions, ctx.num_seqs, split=True,
                              chunks=pieces, pieces=True)
        kernels.pair_close(*parts, self.sinks, y[:, col + self.g_col:], self.out_scale, out, o, y[:, other_col + other.g_col:],
                           other.norm_weight, other.norm_eps, other_out)
        return True
