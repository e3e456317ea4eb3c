"""The Tubusun decoder as a typed configuration and a model description.

config.json gives every size and every constant that differs between models of the design:

  architecture "Tubusun", vocab, width, norm.eps, embedding.scale (or none: 1), logit_softcap (or none),
  loop.{start, stop, times} (or none),
  layers: a list; each entry has type, mixer (the mixer's sizes) and mlp (its feed-forward, or null)
    type "parallel": left:  heads, kv_heads, dim, vdim, scale, mask.size (or no mask), rot.dims / rot.base (or no rot)
                     right: heads, dim, vdim, decay (a list, one a head)
                     left_scale, right_scale (or none: 1)
    mlp kind "dense": ff
    mlp kind "moe":   expert.{ff, limit}, router.{experts, top}, router.groups.{count, keep} (or no groups)

The model: token rows times a constant; layers with a norm in front of and behind every sublayer; layers loop.start ..
loop.stop - 1 run loop.times times in a row with the same weights and a cache and state of their own each time, and in front
of pass t the vector loop.step[t] joins the stream; a final norm; the embedding matrix as output matrix, the logits softly
capped.
Tensor names: embed, final.norm, loop.step, l<i>.{norm1, norm1b, norm2, norm2b}, l<i>.mix.left.{q, k, v, sink, g, o},
l<i>.mix.right.{q, k, v, g, o, norm}, l<i>.mlp.{up, up.b, down, down.b}, l<i>.mlp.{router, e<j>.gate, e<j>.up, e<j>.down}.
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import Any, Dict, Optional, Tuple, Union

from ..parts.spec import LayerSpec, ModelSpec, PartSpec, RunEntry
from .lerazen import _int, _num
from .model_config import ConfigError
from .registry import register_architecture

ACTIVATION_SLOPE = 1.702    # of the experts' gate


@dataclass(frozen=True)
class SinkAttentionConfig:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    window: int         # 0: every earlier position is seen
    rot_dims: int       # 0: no rotation
    rot_base: float

    @classmethod
    def from_dict(cls, d: Dict[str, Any], where: str) -> "SinkAttentionConfig":
        mask, rot = d.get("mask") or {}, d.get("rot") or {}
        cfg = cls(heads=_int(d, "heads", where), kv_heads=_int(d, "kv_heads", where), dim=_int(d, "dim", where),
                  vdim=_int(d, "vdim", where), scale=_num(d, "scale", where),
                  window=_int(mask, "size", where + ".mask") if mask else 0,
                  rot_dims=_int(rot, "dims", where + ".rot", least=0) if rot else 0,
                  rot_base=_num(rot, "base", where + ".rot") if rot else 10000.0)
        if cfg.heads % cfg.kv_heads:
            raise ConfigError(f"{where}: {cfg.heads} heads are not a multiple of {cfg.kv_heads} kv_heads")
        if cfg.rot_dims % 2 or cfg.rot_dims > cfg.dim or not cfg.rot_base > 0:
            raise ConfigError(f"{where}.rot: an even number of at most {cfg.dim} turned entries and a positive base")
        return cfg


@dataclass(frozen=True)
class LightningConfig:
    heads: int
    dim: int
    vdim: int
    decay: Tuple[float, ...]

    @classmethod
    def from_dict(cls, d: Dict[str, Any], where: str) -> "LightningConfig":
        heads, decay = _int(d, "heads", where), d.get("decay")
        if not isinstance(decay, list) or len(decay) != heads or not all(
                isinstance(g, (int, float)) and not isinstance(g, bool) and 0 < g <= 1 for g in decay):
            raise ConfigError(f"{where}.decay: a list of {heads} numbers in (0, 1], one a head")
        return cls(heads=heads, dim=_int(d, "dim", where), vdim=_int(d, "vdim", where), decay=tuple(float(g) for g in decay))


@dataclass(frozen=True)
class ParallelConfig:
    left: SinkAttentionConfig
    right: LightningConfig
    left_scale: float
    right_scale: float

    @classmethod
    def from_dict(cls, d: Dict[str, Any], where: str) -> "ParallelConfig":
        for side in ("left", "right"):
            if not isinstance(d.get(side), dict):
                raise ConfigError(f"{where} lacks {side!r}")
        scale = lambda key: _num(d, key, where) if d.get(key) is not None else 1.0
        return cls(SinkAttentionConfig.from_dict(d["left"], where + ".left"), LightningConfig.from_dict(d["right"], where + ".right"),
                   scale("left_scale"), scale("right_scale"))


@dataclass(frozen=True)
class DenseConfig:
    ff: int


@dataclass(frozen=True)
class ExpertsConfig:
    ff: int
    limit: float
    experts: int
    top: int
    groups: int
    keep: int

    @classmethod
    def from_dict(cls, d: Dict[str, Any], where: str) -> "ExpertsConfig":
        e, r = d.get("expert"), d.get("router")
        if not isinstance(e, dict) or not isinstance(r, dict):
            raise ConfigError(f"{where} lacks 'expert' or 'router'")
        g = r.get("groups") or {}
        cfg = cls(ff=_int(e, "ff", where + ".expert"), limit=_num(e, "limit", where + ".expert"),
                  experts=_int(r, "experts", where + ".router"), top=_int(r, "top", where + ".router"),
                  groups=_int(g, "count", where + ".router.groups") if g else 1,
                  keep=_int(g, "keep", where + ".router.groups") if g else 1)
        if not cfg.limit > 0:
            raise ConfigError(f"{where}.expert: the limit must be positive")
        if cfg.experts % cfg.groups or cfg.keep > cfg.groups or cfg.top > cfg.keep * (cfg.experts // cfg.groups):
            raise ConfigError(f"{where}.router: {cfg.top} of the experts of {cfg.keep} of {cfg.groups} equal groups of {cfg.experts}")
        return cfg


def _feed_forward(d: Optional[Dict[str, Any]], where: str) -> Union[DenseConfig, ExpertsConfig, None]:
    if not d:
        return None
    if d.get("kind") == "dense":
        return DenseConfig(_int(d, "ff", where))
    if d.get("kind") == "moe":
        return ExpertsConfig.from_dict(d, where)
    raise ConfigError(f"{where}: kind {d.get('kind')!r} is not known (dense, moe)")


@dataclass(frozen=True)
class TubusunLayer:
    mixer: ParallelConfig
    mlp: Union[DenseConfig, ExpertsConfig, None]


@dataclass(frozen=True)
class TubusunConfig:
    vocab: int
    width: int
    norm_eps: float
    embed_scale: float
    logit_softcap: float                         # 0: none
    loop: Optional[Tuple[int, int, int]]         # start, stop, times; None: every layer runs once
    step_rows: int                               # of the vectors the checkpoint holds (0: none)
    layers: Tuple[TubusunLayer, ...]
    eos_token_id: Optional[int] = None

    @classmethod
    def from_dict(cls, d: Dict[str, Any]) -> "TubusunConfig":
        raw_layers = d.get("layers")
        if not isinstance(raw_layers, list) or not raw_layers:
            raise ConfigError("config.json lacks the list 'layers'")
        layers = []
        for i, l in enumerate(raw_layers):
            where = f"layers[{i}]"
            if not isinstance(l, dict) or not isinstance(l.get("mixer"), dict):
                raise ConfigError(f"{where} lacks 'mixer'")
            if l.get("type") != "parallel":
                raise ConfigError(f"{where}: mixer type {l.get('type')!r} is not known (parallel)")
            layers.append(TubusunLayer(ParallelConfig.from_dict(l["mixer"], where + ".mixer"), _feed_forward(l.get("mlp"), where + ".mlp")))
        eps = _num(d.get("norm") or {}, "eps", "norm")
        if not eps > 0:
            raise ConfigError("norm.eps must be positive")
        emb, lp, loop, rows = d.get("embedding") or {}, d.get("loop"), None, 0
        if lp:
            loop = (_int(lp, "start", "loop", least=0), _int(lp, "stop", "loop", least=0), _int(lp, "times", "loop"))
            rows = loop[2]
            if not loop[0] <= loop[1] <= len(layers):
                raise ConfigError(f"loop: layers {loop[0]} .. {loop[1]} - 1 of {len(layers)}")
            if loop[0] == loop[1]:
                loop = None                      # a span without layers has no passes
        cap = _num(d, "logit_softcap", "config.json") if d.get("logit_softcap") is not None else 0.0
        if cap < 0:
            raise ConfigError("logit_softcap must not be negative")
        eos = d.get("eos_token_id")
        return cls(vocab=_int(d, "vocab", "config.json"), width=_int(d, "width", "config.json"), norm_eps=eps,
                   embed_scale=_num(emb, "scale", "embedding") if emb.get("scale") is not None else 1.0, logit_softcap=cap,
                   loop=loop, step_rows=rows, layers=tuple(layers),
                   eos_token_id=eos if isinstance(eos, int) and not isinstance(eos, bool) else None)


def tubusun_run_order(cfg: TubusunConfig):
    """The layers in the order they run: (layer, the number of the pass of the looped span that starts with it or None)."""
    n = len(cfg.layers)
    if not cfg.loop:
        return [(i, None) for i in range(n)]
    start, stop, times = cfg.loop
    out = [(i, None) for i in range(start)]
    for t in range(times):
        out += [(i, t if i == start else None) for i in range(start, stop)]
    return out + [(i, None) for i in range(stop, n)]


def _mixer_spec(cfg: TubusunConfig, m: ParallelConfig) -> PartSpec:
    D, eps, a, r = cfg.width, cfg.norm_eps, m.left, m.right
    left = PartSpec("sink_attention", {
        "hidden_size": D, "num_heads": a.heads, "num_kv_heads": a.kv_heads, "key_dim": a.dim, "value_dim": a.vdim, "scale": a.scale,
        "norm_eps": eps, "window": a.window, "rotary_dim": a.rot_dims, "base": a.rot_base})
    right = PartSpec("lightning_attention", {
        "hidden_size": D, "num_heads": r.heads, "key_dim": r.dim, "value_dim": r.vdim, "decay": r.decay, "norm_eps": eps})
    return PartSpec("mixer_sum", {"hidden_size": D, "left": left, "right": right, "left_scale": m.left_scale, "right_scale": m.right_scale})


def _ff_spec(cfg: TubusunConfig, f: Union[DenseConfig, ExpertsConfig]) -> PartSpec:
    if isinstance(f, DenseConfig):
        return PartSpec("gelu_mlp", {"hidden_size": cfg.width, "intermediate_size": f.ff})
    return PartSpec("group_routed_experts", {
        "hidden_size": cfg.width, "expert_size": f.ff, "num_experts": f.experts, "top": f.top, "limit": f.limit,
        "act_alpha": ACTIVATION_SLOPE, "groups": f.groups, "keep": f.keep})


def tubusun_spec(cfg: TubusunConfig) -> ModelSpec:
    norm = PartSpec("rms_norm", {"size": cfg.width, "eps": cfg.norm_eps, "weight_name": ""})
    layers, unused = [], []
    for i, l in enumerate(cfg.layers):
        slots = {"norm1": ("norm1", norm), "mixer": ("mix", _mixer_spec(cfg, l.mixer)), "post1": ("norm1b", norm)}
        if l.mlp is not None:
            slots.update(norm2=("norm2", norm), post2=("norm2b", norm), ff=("mlp", _ff_spec(cfg, l.mlp)))
        else:
            # a checkpoint may still hold the second norms of a layer that has no feed-forward to use them
            unused += [f"l{i}.norm2", f"l{i}.norm2b"]
        layers.append(LayerSpec(prefix=f"l{i}", block="sandwich", slots=slots, block_params={"size": cfg.width}))
    return ModelSpec(
        hidden_size=cfg.width, vocab_size=cfg.vocab, embed_name="embed", layers=layers,
        run_order=[RunEntry(i, add_vector=t) for i, t in tubusun_run_order(cfg)],
        final_norm=norm, final_norm_name="final.norm", head_name=None, eos_token_id=cfg.eos_token_id, embed_scale=cfg.embed_scale,
        logit_softcap=cfg.logit_softcap, run_vectors=("loop.step", cfg.step_rows) if cfg.loop else None,
        ignored_tensors=tuple(unused) + (() if cfg.loop else ("loop.step",)))


def tubusun_sizes(cfg: TubusunConfig) -> dict:
    """The sizes of a configuration as a flat record (of its first layer of every kind)."""
    out = {"layers": len(cfg.layers), "runs": len(tubusun_run_order(cfg)), "hidden": cfg.width, "vocab": cfg.vocab, "tied": True}
    for l in cfg.layers:
        a, r = l.mixer.left, l.mixer.right
        for key, value in (("q_heads", a.heads), ("kv_heads", a.kv_heads), ("head_dim", a.dim), ("value_dim", a.vdim), ("window", a.window),
                           ("linear_heads", r.heads), ("linear_key_dim", r.dim), ("linear_value_dim", r.vdim)):
            out.setdefault(key, value)
        if isinstance(l.mlp, DenseConfig):
            out.setdefault("intermediate", l.mlp.ff)
        elif l.mlp is not None:
            out.setdefault("experts", l.mlp.experts)
            out.setdefault("experts_per_token", l.mlp.top)
            out.setdefault("expert_intermediate", l.mlp.ff)
    return out


def tubusun_with_layers(raw: dict, layers: int) -> dict:
    """The same kinds of layers, ``layers`` of them (the list cut, or repeated from its start), without a loop."""
    have = raw["layers"]
    out = dict(raw, layers=[have[i % len(have)] for i in range(layers)] if have else [])
    out.pop("loop", None)
    return out


register_architecture("Tubusun", TubusunConfig.from_dict, tubusun_spec, tubusun_sizes, tubusun_with_layers)
