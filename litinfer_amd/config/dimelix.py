"""Typed configuration of the Dimelix decoder, read from config.json, and the model as data.

config.json: `vocab`, `width`, `norm.eps`, `streams`, `embedding.scale` (optional, 1), `logit_softcap` (optional),
`loop` {start, stop, times} (optional: layers start..stop-1 are passed `times` times with the same weights, every pass
with a cache or state of its own) and `layers`, a list whose entries have `type` (`attention`, `latent_attention` or
`parallel`), the mixer's sizes and constants under `mixer`, and `mlp` (null or {kind: dense, ff}).

The model: the token's embedding row times a factor, in `streams` residual streams with learned mixing
(`parts/block.py`, HyperBlock); every sublayer reads a weighted sum of the streams through an RMS norm whose weight is
stored around zero (1 + w); a final norm of the same kind on the streams' sum, the embedding table as the head (without
the factor) and a tanh cap on the logits.
`attention`: an RMS norm on every query and key head, rotation of neighbouring pairs, a sink a head, a gate an element.
`latent_attention`: attention over a compressed cache without positions, a gate an element (`parts/masked_attention.py`).
`parallel`: attention with a window whose scores lose slope_h times the distance, slope_h = 2^(-8 (h + 1) / heads), and
whose values are its keys as projected, beside a delta rule with a decay and a removal rate a channel
(`parts/channel_delta.py`), added with factors.  Feed-forward: Wdown xIELU(Wup x) (`parts/mlp.py`).
Tensor names: embed, final.norm and per layer i `l<i>.norm1|norm2`, `l<i>.hc1|hc2.in|out|mix`, `l<i>.mix.*` (`.left.*`,
`.right.*` for the two mixers of a parallel layer), `l<i>.mlp.up|down|act`.
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import Any, Dict, Optional, Tuple

from .kufolorn import _obj
from .qwen2 import ConfigError
from .spec import ExecEntry, LayerSpec, ModelSpec, PartSpec
from .tovasun import DEFAULT_MAX_POSITIONS, _number, _pos_int

MIXER_TYPES = ("attention", "latent_attention", "parallel")


def _opt_int(d: Dict[str, Any], key: str, where: str, default: int) -> int:
    return _pos_int(d, key, where) if d.get(key) is not None else default


@dataclass(frozen=True)
class HeadsConfig:
    """Grouped-query attention: with `rot_dims` columns rotated, or with a window of `window` tokens (0: none)."""
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    rot_base: float = 0.0
    rot_dims: int = 0
    window: int = 0

    @classmethod
    def from_dict(cls, d: Any, where: str, rotates: bool) -> "HeadsConfig":
        d = _obj(d, where)
        heads, dim = _pos_int(d, "heads", where), _pos_int(d, "dim", where)
        kvh, vdim = _opt_int(d, "kv_heads", where, heads), _opt_int(d, "vdim", where, dim)
        if heads % kvh:
            raise ConfigError(f"config.json: {where}: {heads} heads are not a multiple of {kvh} kv heads")
        scale = _number(d, "scale", where)
        if rotates:
            rot = _obj(d.get("rot"), where + ".rot")
            base, dims = _number(rot, "base", where + ".rot"), _pos_int(rot, "dims", where + ".rot")
            if base <= 0 or dims % 2 or dims > dim:
                raise ConfigError(f"config.json: {where}.rot: base must be positive, dims even and at most the head size {dim}")
            return cls(heads, kvh, dim, vdim, scale, rot_base=base, rot_dims=dims)
        if vdim != dim:
            raise ConfigError(f"config.json: {where}: the keys are the values, vdim ({vdim}) must equal dim ({dim})")
        window = _opt_int(_obj(d["mask"], where + ".mask"), "size", where + ".mask", 0) if d.get("mask") is not None else 0
        return cls(heads, kvh, dim, vdim, scale, window=window)


@dataclass(frozen=True)
class LatentConfig:
    heads: int
    dim: int
    vdim: int
    kv_rank: int
    scale: float

    @classmethod
    def from_dict(cls, d: Any, where: str) -> "LatentConfig":
        d = _obj(d, where)
        dim = _pos_int(d, "dim", where)
        return cls(_pos_int(d, "heads", where), dim, _opt_int(d, "vdim", where, dim), _pos_int(d, "kv_rank", where), _number(d, "scale", where))


@dataclass(frozen=True)
class ChannelDeltaConfig:
    heads: int
    dim: int

    @classmethod
    def from_dict(cls, d: Any, where: str) -> "ChannelDeltaConfig":
        d = _obj(d, where)
        return cls(_pos_int(d, "heads", where), _pos_int(d, "dim", where))


@dataclass(frozen=True)
class ParallelConfig:
    left: HeadsConfig
    right: ChannelDeltaConfig
    left_scale: float
    right_scale: float

    @classmethod
    def from_dict(cls, d: Any, where: str) -> "ParallelConfig":
        d = _obj(d, where)
        return cls(HeadsConfig.from_dict(d.get("left"), where + ".left", rotates=False),
                   ChannelDeltaConfig.from_dict(d.get("right"), where + ".right"),
                   _number(d, "left_scale", where), _number(d, "right_scale", where))


@dataclass(frozen=True)
class DimelixLayer:
    type: str
    mixer: Any                   # HeadsConfig | LatentConfig | ParallelConfig
    ff: int                      # 0: the layer has no feed-forward


@dataclass(frozen=True)
class DimelixConfig:
    vocab: int
    width: int
    eps: float
    streams: int
    embedding_scale: float
    layers: Tuple[DimelixLayer, ...]
    loop: Optional[Tuple[int, int, int]]        # (start, stop, times)
    logit_softcap: float
    max_positions: int
    eos_token_ids: Tuple[int, ...]
    raw: Any = None

    architecture = "Dimelix"

    @classmethod
    def from_dict(cls, cfg: Dict[str, Any]) -> "DimelixConfig":
        vocab, width = _pos_int(cfg, "vocab", "config"), _pos_int(cfg, "width", "config")
        eps = _number(cfg.get("norm") or {}, "eps", "norm")
        if eps < 0:
            raise ConfigError("config.json: norm.eps must not be negative")
        raw_layers = cfg.get("layers")
        if not isinstance(raw_layers, list) or not raw_layers:
            raise ConfigError("config.json: 'layers' must be a list with at least one layer")
        layers = []
        for i, L in enumerate(raw_layers):
            where = f"layers[{i}]"
            L = _obj(L, where)
            kind, m = L.get("type"), L.get("mixer")
            if kind not in MIXER_TYPES:
                raise ConfigError(f"config.json: {where}: unknown mixer type {kind!r} (known: {', '.join(MIXER_TYPES)})")
            if kind == "attention":
                mixer: Any = HeadsConfig.from_dict(m, where + ".mixer", rotates=True)
            else:
                mixer = (LatentConfig if kind == "latent_attention" else ParallelConfig).from_dict(m, where + ".mixer")
            ff = 0
            if L.get("mlp") is not None:
                mlp = _obj(L["mlp"], where + ".mlp")
                if mlp.get("kind") != "dense":
                    raise ConfigError(f"config.json: {where}.mlp.kind {mlp.get('kind')!r} is not supported (only 'dense')")
                ff = _pos_int(mlp, "ff", where + ".mlp")
            layers.append(DimelixLayer(kind, mixer, ff))
        loop = cfg.get("loop")
        if loop is not None:
            loop = _obj(loop, "loop")
            start, stop = _pos_int(loop, "start", "loop", allow_zero=True), _pos_int(loop, "stop", "loop", allow_zero=True)
            times = _pos_int(loop, "times", "loop")
            if not 0 <= start <= stop <= len(layers):
                raise ConfigError(f"config.json: loop {start}..{stop} lies outside the {len(layers)} layers")
            loop = (start, stop, times) if stop > start else None
        emb = _obj(cfg.get("embedding") or {}, "embedding")
        scale = _number(emb, "scale", "embedding") if emb.get("scale") is not None else 1.0
        cap = 0.0 if cfg.get("logit_softcap") is None else _number(cfg, "logit_softcap", "config")
        if cap < 0:
            raise ConfigError("config.json: logit_softcap must not be negative")
        eos = cfg.get("eos_token_id")
        eos_ids = () if eos is None else tuple(int(e) for e in (eos if isinstance(eos, list) else [eos]))
        return cls(vocab=vocab, width=width, eps=eps, streams=_pos_int(cfg, "streams", "config"), embedding_scale=scale,
                   layers=tuple(layers), loop=loop, logit_softcap=cap,
                   max_positions=_opt_int(cfg, "max_positions", "config", DEFAULT_MAX_POSITIONS),
                   eos_token_ids=tuple(e for e in eos_ids if e >= 0), raw=cfg)


def distance_slopes(heads: int):
    """The slope of head h's distance bias: 2^(-8 (h + 1) / heads)."""
    return [2.0 ** (-8.0 * (h + 1) / heads) for h in range(heads)]


def _mixer_spec(c: DimelixConfig, L: DimelixLayer, prefix: str) -> PartSpec:
    m = L.mixer
    if L.type == "latent_attention":
        return PartSpec("latent_attention", prefix, {
            "hidden_size": c.width, "num_heads": m.heads, "head_dim": m.dim, "rot_dim": 0, "value_dim": m.vdim,
            "kv_rank": m.kv_rank, "column_gate": True, "scale": m.scale, "eps": c.eps})

    def heads(a: HeadsConfig, at: str, more: Dict[str, Any]) -> PartSpec:
        return PartSpec("masked_attention", at, {
            "hidden_size": c.width, "num_heads": a.heads, "num_kv_heads": a.kv_heads, "head_dim": a.dim, "value_dim": a.vdim,
            "scale": a.scale, "qk_norm": "heads", "eps": c.eps, "column_gate": True, **more})
    if L.type == "attention":
        return heads(m, prefix, {"sink": True, "position": PartSpec("rope_pairs", "", {
            "head_dim": m.dim, "rotary_dim": m.rot_dims, "theta": m.rot_base, "layout": "pairs"})})
    left = heads(m.left, prefix + "left.", {"keys_are_values": True, "window": m.left.window, "slopes": distance_slopes(m.left.heads)})
    right = PartSpec("channel_delta", prefix + "right.", {"hidden_size": c.width, "num_heads": m.right.heads,
                                                          "head_dim": m.right.dim, "eps": c.eps})
    return PartSpec("mixer_pair", prefix, {"left": left, "right": right, "left_scale": m.left_scale, "right_scale": m.right_scale})


def dimelix_model_spec(c: DimelixConfig) -> ModelSpec:
    n = len(c.layers)
    layers = []
    for i, L in enumerate(c.layers):
        p = f"l{i}."

        def norm(name):
            return PartSpec("rmsnorm", p, {"size": c.width, "eps": c.eps, "param": name, "offset": 1.0})
        parts: Dict[str, Optional[PartSpec]] = {"hyper": PartSpec("hyper", p, {"streams": c.streams}), "norm1": norm("norm1"),
                                                "mixer": _mixer_spec(c, L, p + "mix.")}
        if L.ff:
            parts.update({"norm2": norm("norm2"),
                          "feed_forward": PartSpec("xielu_mlp", p + "mlp.", {"hidden_size": c.width, "intermediate_size": L.ff})})
        layers.append(LayerSpec(block="hyper", parts=parts))
    order = list(range(n))
    if c.loop:
        start, stop, times = c.loop
        order = order[:start] + times * order[start:stop] + order[stop:]
    return ModelSpec(
        architecture=c.architecture, hidden_size=c.width, vocab_size=c.vocab, max_positions=c.max_positions,
        embedding=PartSpec("token_embedding", "", {"vocab_size": c.vocab, "hidden_size": c.width, "param": "embed",
                                                   "scale": c.embedding_scale}),
        layers=tuple(layers), order=tuple(ExecEntry(i) for i in order),
        final_norm=PartSpec("rmsnorm", "final.", {"size": c.width, "eps": c.eps, "param": "norm", "offset": 1.0}),
        head=PartSpec("linear_head", "", {"vocab_size": c.vocab, "hidden_size": c.width, "tied_to": "embed",
                                          "softcap": c.logit_softcap}),
        eos_token_ids=c.eos_token_ids, streams=c.streams)
