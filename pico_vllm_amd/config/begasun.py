"""The Begasun decoder as a typed configuration and a model description.

config.json gives every size and every constant that differs between models of the design:

  architecture "Begasun", vocab, width, norm.eps, embedding.scale (or none: 1), logit_scale (or none: 1),
  loop.{start, stop, times} (or none), token_side.dim (or none),
  layers: a list; each entry has type (its mixer), mixer (the mixer's sizes) and mlp (its feed-forward, or null)
    type "latent_attention": heads, dim, rot_dim, vdim, kv_rank, scale, rot.base, rot.scaling.{factor, original, fast, slow}
    type "rglru":            width, blocks, conv
    type "attention":        heads, kv_heads, dim, vdim, scale, rot.dims / rot.base (or no rot)
    mlp kind "dense": ff, limit

The model: token rows times a constant; layers with a norm in front of and behind every sublayer (weights stored around
zero) and a stored vector on what joins the stream, and behind the sublayers a gated row of a table of tokens; layers
loop.start .. loop.stop - 1 run loop.times times in a row with the same weights and a cache or state of their own each
time, and in front of every pass a matrix makes the stream anew from the stream and the embeddings; a final norm; an
output matrix of its own, the logits times a constant.
Tensor names: embed, head, final.norm, loop.in, side.embed, l<i>.{norm1, norm1b, ls1, norm2, norm2b, ls2}, l<i>.mix.*, l<i>.mlp.*,
l<i>.side.{gate, proj, norm}.
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import Any, Dict, Optional, Tuple

from ..parts.spec import LayerSpec, ModelSpec, PartSpec, RunEntry
from .lerazen import _int, _num
from .model_config import ConfigError
from .nasedra import RotationConfig
from .registry import register_architecture

GATE_SHARPNESS = 8.0        # of the recurrence's decay
ACTIVATION_SLOPE = 1.702    # of the feed-forward's gate


@dataclass(frozen=True)
class LatentAttentionConfig:
    heads: int
    dim: int
    rot_dim: int
    vdim: int
    kv_rank: int
    scale: float
    base: float
    scaling: Optional[Tuple[float, float, float, float]]

    @classmethod
    def from_dict(cls, d: Dict[str, Any], where: str) -> "LatentAttentionConfig":
        rot_dim = _int(d, "rot_dim", where, least=0)
        base, scaling = 10000.0, None
        if rot_dim:
            if not isinstance(d.get("rot"), dict):
                raise ConfigError(f"{where}: a rotated part needs 'rot'")
            # the rotated vector is the rot_dim part, whatever rot.dims says
            r = RotationConfig.from_dict(dict(d["rot"], dims=rot_dim), where + ".rot", rot_dim)
            base, scaling = r.base, r.scaling
        return cls(heads=_int(d, "heads", where), dim=_int(d, "dim", where), rot_dim=rot_dim, vdim=_int(d, "vdim", where),
                   kv_rank=_int(d, "kv_rank", where), scale=_num(d, "scale", where), base=base, scaling=scaling)


@dataclass(frozen=True)
class RecurrenceConfig:
    width: int
    blocks: int
    conv: int

    @classmethod
    def from_dict(cls, d: Dict[str, Any], where: str) -> "RecurrenceConfig":
        cfg = cls(width=_int(d, "width", where), blocks=_int(d, "blocks", where), conv=_int(d, "conv", where))
        if cfg.width % cfg.blocks:
            raise ConfigError(f"{where}: {cfg.width} channels are not {cfg.blocks} equal blocks")
        return cfg


@dataclass(frozen=True)
class AttentionConfig:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    rot: Optional[RotationConfig]

    @classmethod
    def from_dict(cls, d: Dict[str, Any], where: str) -> "AttentionConfig":
        dim = _int(d, "dim", where)
        cfg = cls(heads=_int(d, "heads", where), kv_heads=_int(d, "kv_heads", where), dim=dim, vdim=_int(d, "vdim", where),
                  scale=_num(d, "scale", where),
                  rot=RotationConfig.from_dict(d["rot"], where + ".rot", dim) if (d.get("rot") or {}).get("dims") else None)
        if cfg.heads % cfg.kv_heads:
            raise ConfigError(f"{where}: {cfg.heads} heads are not a multiple of {cfg.kv_heads} kv_heads")
        return cfg


@dataclass(frozen=True)
class FeedForwardConfig:
    ff: int
    limit: float

    @classmethod
    def from_dict(cls, d: Dict[str, Any], where: str) -> "FeedForwardConfig":
        if d.get("kind") != "dense":
            raise ConfigError(f"{where}: mlp kind {d.get('kind')!r} is not known (dense)")
        cfg = cls(_int(d, "ff", where), _num(d, "limit", where))
        if not cfg.limit > 0:
            raise ConfigError(f"{where}: the limit must be positive")
        return cfg


@dataclass(frozen=True)
class BegasunLayer:
    type: str
    mixer: Any
    mlp: Optional[FeedForwardConfig]


_MIXERS = {"latent_attention": LatentAttentionConfig, "rglru": RecurrenceConfig, "attention": AttentionConfig}


@dataclass(frozen=True)
class BegasunConfig:
    vocab: int
    width: int
    norm_eps: float
    embed_scale: float
    logit_scale: float
    loop: Optional[Tuple[int, int, int]]         # start, stop, times; None: every layer runs once, nothing is mixed in
    side_dim: int                                # 0: no token side
    layers: Tuple[BegasunLayer, ...]
    eos_token_id: Optional[int] = None

    @classmethod
    def from_dict(cls, d: Dict[str, Any]) -> "BegasunConfig":
        raw_layers = d.get("layers")
        if not isinstance(raw_layers, list) or not raw_layers:
            raise ConfigError("config.json lacks the list 'layers'")
        layers = []
        for i, l in enumerate(raw_layers):
            where = f"layers[{i}]"
            if not isinstance(l, dict) or not isinstance(l.get("mixer"), dict):
                raise ConfigError(f"{where} lacks 'mixer'")
            if l.get("type") not in _MIXERS:
                raise ConfigError(f"{where}: mixer type {l.get('type')!r} is not known ({', '.join(sorted(_MIXERS))})")
            mlp = l.get("mlp")
            layers.append(BegasunLayer(l["type"], _MIXERS[l["type"]].from_dict(l["mixer"], where + ".mixer"),
                                       FeedForwardConfig.from_dict(mlp, where + ".mlp") if mlp else None))
        eps = _num(d.get("norm") or {}, "eps", "norm")
        if not eps > 0:
            raise ConfigError("norm.eps must be positive")
        emb, side, lp = d.get("embedding") or {}, d.get("token_side") or {}, d.get("loop")
        loop = None
        if lp:
            loop = (_int(lp, "start", "loop", least=0), _int(lp, "stop", "loop", least=0), _int(lp, "times", "loop"))
            if not loop[0] <= loop[1] <= len(layers):
                raise ConfigError(f"loop: layers {loop[0]} .. {loop[1]} - 1 of {len(layers)}")
            if loop[0] == loop[1]:
                loop = None                      # a span without layers has no passes
        eos = d.get("eos_token_id")
        return cls(vocab=_int(d, "vocab", "config.json"), width=_int(d, "width", "config.json"), norm_eps=eps,
                   embed_scale=_num(emb, "scale", "embedding") if emb.get("scale") is not None else 1.0,
                   logit_scale=_num(d, "logit_scale", "config.json") if d.get("logit_scale") is not None else 1.0, loop=loop,
                   side_dim=_int(side, "dim", "token_side") if side else 0, layers=tuple(layers),
                   eos_token_id=eos if isinstance(eos, int) and not isinstance(eos, bool) else None)


def begasun_run_order(cfg: BegasunConfig):
    """The layers in the order they run: (layer, whether a pass of the looped span starts with it)."""
    n = len(cfg.layers)
    if not cfg.loop:
        return [(i, False) for i in range(n)]
    start, stop, times = cfg.loop
    out = [(i, False) for i in range(start)]
    for _ in range(times):
        out += [(i, i == start) for i in range(start, stop)]
    return out + [(i, False) for i in range(stop, n)]


def _mixer_spec(cfg: BegasunConfig, l: BegasunLayer) -> PartSpec:
    m, D, eps = l.mixer, cfg.width, cfg.norm_eps
    if l.type == "latent_attention":
        return PartSpec("latent_attention", {
            "hidden_size": D, "num_heads": m.heads, "dim": m.dim, "rot_dim": m.rot_dim, "value_dim": m.vdim, "q_rank": 0,
            "kv_rank": m.kv_rank, "scale": m.scale, "base": m.base, "scaling": m.scaling, "norm_eps": eps, "gate_heads": True})
    if l.type == "rglru":
        return PartSpec("gated_linear_recurrence", {
            "hidden_size": D, "width": m.width, "parts": m.blocks, "taps": m.conv, "sharpness": GATE_SHARPNESS})
    return PartSpec("normed_attention", {
        "hidden_size": D, "num_heads": m.heads, "num_kv_heads": m.kv_heads, "key_dim": m.dim, "value_dim": m.vdim, "scale": m.scale,
        "norm_eps": eps, "rotary_dim": m.rot.dims if m.rot else 0, "base": m.rot.base if m.rot else 10000.0,
        "scaling": m.rot.scaling if m.rot else None})


def begasun_spec(cfg: BegasunConfig) -> ModelSpec:
    norm = PartSpec("rms_norm", {"size": cfg.width, "eps": cfg.norm_eps, "weight_name": "", "offset": 1.0})
    layers, unused = [], []
    for i, l in enumerate(cfg.layers):
        slots = {"norm1": ("norm1", norm), "mixer": ("mix", _mixer_spec(cfg, l)), "post1": ("norm1b", norm)}
        if l.mlp is not None:
            slots.update(norm2=("norm2", norm), post2=("norm2b", norm), ff=("mlp", PartSpec("clipped_glu_mlp", {
                "hidden_size": cfg.width, "intermediate_size": l.mlp.ff, "limit": l.mlp.limit, "alpha": ACTIVATION_SLOPE})))
        else:
            # a checkpoint may still hold the second norms and vector of a layer that has no feed-forward to use them
            unused += [f"l{i}.norm2", f"l{i}.norm2b", f"l{i}.ls2"]
        if cfg.side_dim:
            slots["side"] = ("side", PartSpec("gated_token_row", {"size": cfg.width, "dim": cfg.side_dim, "column": i * cfg.side_dim,
                                                                  "norm_eps": cfg.norm_eps}))
        layers.append(LayerSpec(prefix=f"l{i}", block="sandwich_scaled", slots=slots, block_params={"size": cfg.width}))
    before = ()
    if cfg.side_dim:
        before = (("side.embed", PartSpec("token_table", {"rows": cfg.vocab, "size": cfg.side_dim * len(cfg.layers), "name": ""})),)
    return ModelSpec(
        hidden_size=cfg.width, vocab_size=cfg.vocab, embed_name="embed", layers=layers,
        run_order=[RunEntry(i, mix_input=first) for i, first in begasun_run_order(cfg)],
        # the logits' constant sits on the final norm's weight (the output matrix is linear)
        final_norm=PartSpec("rms_norm", dict(norm.params, gain=cfg.logit_scale)), final_norm_name="final.norm", head_name="head",
        eos_token_id=cfg.eos_token_id, before_layers=before, embed_scale=cfg.embed_scale,
        input_mix=("loop.in", PartSpec("input_mix", {"size": cfg.width, "name": ""})) if cfg.loop else None,
        ignored_tensors=tuple(unused) + (() if cfg.loop else ("loop.in",)))


def begasun_sizes(cfg: BegasunConfig) -> dict:
    """The sizes of a configuration as a flat record (of its first layer of every kind)."""
    out = {"layers": len(cfg.layers), "runs": len(begasun_run_order(cfg)), "hidden": cfg.width, "vocab": cfg.vocab, "tied": False,
           "side_dim": cfg.side_dim}
    for l in cfg.layers:
        m = l.mixer
        if l.type == "latent_attention":
            out.setdefault("latent_heads", m.heads)
            out.setdefault("latent_head_dim", m.dim + m.rot_dim)
            out.setdefault("latent_value_dim", m.vdim)
            out.setdefault("kv_rank", m.kv_rank)
        elif l.type == "rglru":
            out.setdefault("recurrence_width", m.width)
            out.setdefault("recurrence_blocks", m.blocks)
        else:
            out.setdefault("q_heads", m.heads)
            out.setdefault("kv_heads", m.kv_heads)
            out.setdefault("head_dim", m.dim)
            out.setdefault("value_dim", m.vdim)
        if l.mlp is not None:
            out.setdefault("intermediate", l.mlp.ff)
    return out


def begasun_with_layers(raw: dict, layers: int) -> dict:
    """The same kinds of layers, ``layers`` of them (the list cut, or repeated from its start), without a loop."""
    have = raw["layers"]
    out = dict(raw, layers=[have[i % len(have)] for i in range(layers)] if have else [])
    out.pop("loop", None)
    return out


register_architecture("Begasun", BegasunConfig.from_dict, begasun_spec, begasun_sizes, begasun_with_layers)
