"""Typed configuration of the Besorax decoder, read from config.json, and the model as data.

config.json: `vocab`, `width`, `norm.eps`, `residual_mult` (optional, 1), `embedding.scale` (optional, 1) and `layers`, a
list whose entries have `type` (`lightning`, `attention` or `latent_attention`), the mixer's sizes and constants under
`mixer`, and `mlp`: null, {kind: dense, ff, limit} or {kind: moe, expert: {ff}, router: {experts, top}, shared: {ff}}.

The model: the token's embedding row times a factor; per layer x += m mixer(norm1(x)), then x += m ff(norm2(x)), m =
residual_mult; the norms are tanh(alpha x) w + b, element by element; a last norm of the same kind and a head of its own.
`lightning`: linear attention with a fixed decay a head, silu on q, k and v, one norm over all heads, a sigmoid gate
(`parts/retention.py`).  `attention`: grouped-query attention whose queries see only their own run of `mask.size`
positions, neighbouring columns rotated in pairs, a sink a head; with `kv_from`: j the layer reads the keys and values
that layer j keeps.  `latent_attention`: attention over a compressed cache, queries through a latent of their own, a sink
a head (`parts/masked_attention.py`).  Feed-forwards: the clamped gated one (`parts/mlp.py`), or GELU experts behind a
router with sigmoid scores whose weights multiply the experts' inputs, and a shared expert (`parts/moe.py`).
Tensor names: embed, head, final.norm and per layer i `l<i>.norm1|norm2` (each norm with `.alpha` and `.b` beside it),
`l<i>.mix.*`, `l<i>.mlp.gate|up|down` or `l<i>.mlp.router|e<j>.up|e<j>.down|shared.up|shared.down`.
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import Any, Dict, Optional, Tuple

from .dimelix import _opt_int
from .kufolorn import _obj
from .qwen2 import ConfigError
from .spec import ExecEntry, LayerSpec, ModelSpec, PartSpec
from .tovasun import DEFAULT_MAX_POSITIONS, _number, _pos_int

MIXER_TYPES = ("lightning", "attention", "latent_attention")


def _rotation(d: Any, where: str, at_most: int) -> Tuple[float, int]:
    """(base, rotated columns); (0, 0) where there is no rotation."""
    if d is None:
        return 0.0, 0
    d = _obj(d, where)
    base, dims = _number(d, "base", where), _pos_int(d, "dims", where)
    if base <= 0 or dims % 2 or dims > at_most:
        raise ConfigError(f"config.json: {where}: base must be positive, dims even and at most {at_most}")
    return base, dims


@dataclass(frozen=True)
class LightningConfig:
    heads: int
    dim: int
    vdim: int
    decay: Tuple[float, ...]

    @classmethod
    def from_dict(cls, d: Any, where: str) -> "LightningConfig":
        d = _obj(d, where)
        heads, dim = _pos_int(d, "heads", where), _pos_int(d, "dim", where)
        decay = d.get("decay")
        if not isinstance(decay, list) or len(decay) != heads or not all(isinstance(x, (int, float)) and not isinstance(x, bool) for x in decay):
            raise ConfigError(f"config.json: {where}.decay must be a list of {heads} numbers, one a head")
        return cls(heads, dim, _opt_int(d, "vdim", where, dim), tuple(float(x) for x in decay))


@dataclass(frozen=True)
class ChunkedConfig:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    rot_base: float
    rot_dims: int
    chunk: int                   # 0: no chunks
    kv_from: Optional[int]

    @classmethod
    def from_dict(cls, d: Any, where: str) -> "ChunkedConfig":
        d = _obj(d, where)
        heads, dim = _pos_int(d, "heads", where), _pos_int(d, "dim", where)
        kvh = _opt_int(d, "kv_heads", where, heads)
        if heads % kvh:
            raise ConfigError(f"config.json: {where}: {heads} heads are not a multiple of {kvh} kv heads")
        base, dims = _rotation(d.get("rot"), where + ".rot", dim)
        mask = d.get("mask")
        chunk = _pos_int(_obj(mask, where + ".mask"), "size", where + ".mask") if mask is not None else 0
        src = d.get("kv_from")
        if src is not None:
            src = _pos_int(d, "kv_from", where, allow_zero=True)
        return cls(heads, kvh, dim, _opt_int(d, "vdim", where, dim), _number(d, "scale", where), base, dims, chunk, src)

    def kept(self) -> Tuple[Any, ...]:
        """What two layers that share keys and values must agree in."""
        return (self.heads, self.kv_heads, self.dim, self.vdim, self.rot_base, self.rot_dims)


@dataclass(frozen=True)
class LatentConfig:
    heads: int
    dim: int
    rot_dim: int
    vdim: int
    kv_rank: int
    q_rank: int
    scale: float
    rot_base: float

    @classmethod
    def from_dict(cls, d: Any, where: str) -> "LatentConfig":
        d = _obj(d, where)
        dim, rot_dim = _pos_int(d, "dim", where), _pos_int(d, "rot_dim", where)
        base, dims = _rotation(_obj(d.get("rot"), where + ".rot"), where + ".rot", rot_dim)
        if dims != rot_dim:
            raise ConfigError(f"config.json: {where}: rot.dims ({dims}) must equal rot_dim ({rot_dim})")
        return cls(_pos_int(d, "heads", where), dim, rot_dim, _opt_int(d, "vdim", where, dim), _pos_int(d, "kv_rank", where),
                   _pos_int(d, "q_rank", where), _number(d, "scale", where), base)


@dataclass(frozen=True)
class FeedForwardConfig:
    kind: str                    # "dense" or "moe"
    ff: int
    limit: float = 0.0           # dense
    experts: int = 0             # moe
    top: int = 0
    shared_ff: int = 0

    @classmethod
    def from_dict(cls, d: Any, where: str) -> "FeedForwardConfig":
        d = _obj(d, where)
        kind = d.get("kind")
        if kind == "dense":
            limit = _number(d, "limit", where)
            if limit <= 0:
                raise ConfigError(f"config.json: {where}.limit must be positive")
            return cls("dense", _pos_int(d, "ff", where), limit)
        if kind != "moe":
            raise ConfigError(f"config.json: {where}.kind {kind!r} is not supported ('dense' or 'moe')")
        expert, router = _obj(d.get("expert"), where + ".expert"), _obj(d.get("router"), where + ".router")
        experts, top = _pos_int(router, "experts", where + ".router"), _pos_int(router, "top", where + ".router")
        if top > experts:
            raise ConfigError(f"config.json: {where}.router: {top} choices among {experts} experts")
        shared = d.get("shared")
        shared_ff = _pos_int(_obj(shared, where + ".shared"), "ff", where + ".shared") if shared is not None else 0
        return cls("moe", _pos_int(expert, "ff", where + ".expert"), experts=experts, top=top, shared_ff=shared_ff)


_MIXERS = {"lightning": LightningConfig, "attention": ChunkedConfig, "latent_attention": LatentConfig}


@dataclass(frozen=True)
class BesoraxLayer:
    type: str
    mixer: Any                   # LightningConfig | ChunkedConfig | LatentConfig
    mlp: Optional[FeedForwardConfig]


@dataclass(frozen=True)
class BesoraxConfig:
    vocab: int
    width: int
    eps: float
    residual_mult: float
    embedding_scale: float
    layers: Tuple[BesoraxLayer, ...]
    max_positions: int
    eos_token_ids: Tuple[int, ...]
    raw: Any = None

    architecture = "Besorax"

    @classmethod
    def from_dict(cls, cfg: Dict[str, Any]) -> "BesoraxConfig":
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
            kind = L.get("type")
            if kind not in MIXER_TYPES:
                raise ConfigError(f"config.json: {where}: unknown mixer type {kind!r} (known: {', '.join(MIXER_TYPES)})")
            mixer = _MIXERS[kind].from_dict(L.get("mixer"), where + ".mixer")
            src = getattr(mixer, "kv_from", None)
            if src is not None:
                owner = layers[src] if src < i else None
                if owner is None or owner.type != "attention" or owner.mixer.kv_from is not None or owner.mixer.kept() != mixer.kept():
                    raise ConfigError(f"config.json: {where}.mixer.kv_from {src}: that must be an earlier attention layer with "
                                      f"keys of its own and the same heads, sizes and rotation")
            mlp = FeedForwardConfig.from_dict(L["mlp"], where + ".mlp") if L.get("mlp") is not None else None
            layers.append(BesoraxLayer(kind, mixer, mlp))
        emb = _obj(cfg.get("embedding") or {}, "embedding")
        mult = 1.0 if cfg.get("residual_mult") is None else _number(cfg, "residual_mult", "config")
        if mult == 0:
            raise ConfigError("config.json: residual_mult must not be zero")
        eos = cfg.get("eos_token_id")
        eos_ids = () if eos is None else tuple(int(e) for e in (eos if isinstance(eos, list) else [eos]))
        return cls(vocab=vocab, width=width, eps=eps, residual_mult=mult,
                   embedding_scale=_number(emb, "scale", "embedding") if emb.get("scale") is not None else 1.0,
                   layers=tuple(layers), max_positions=_opt_int(cfg, "max_positions", "config", DEFAULT_MAX_POSITIONS),
                   eos_token_ids=tuple(e for e in eos_ids if e >= 0), raw=cfg)


def _mixer_spec(c: BesoraxConfig, L: BesoraxLayer, prefix: str) -> PartSpec:
    m = L.mixer
    if L.type == "lightning":
        return PartSpec("lightning", prefix, {"hidden_size": c.width, "num_heads": m.heads, "head_dim": m.dim, "value_dim": m.vdim,
                                              "decay": m.decay, "eps": c.eps})

    def pairs(head_dim: int, dims: int, base: float) -> PartSpec:
        return PartSpec("rope_pairs", "", {"head_dim": head_dim, "rotary_dim": dims, "theta": base, "layout": "pairs"})
    if L.type == "latent_attention":
        return PartSpec("latent_attention", prefix, {
            "hidden_size": c.width, "num_heads": m.heads, "head_dim": m.dim, "rot_dim": m.rot_dim, "value_dim": m.vdim,
            "kv_rank": m.kv_rank, "q_rank": m.q_rank, "sink": True, "scale": m.scale, "eps": c.eps,
            "position": pairs(m.rot_dim, m.rot_dim, m.rot_base)})
    return PartSpec("masked_attention", prefix, {
        "hidden_size": c.width, "num_heads": m.heads, "num_kv_heads": m.kv_heads, "head_dim": m.dim, "value_dim": m.vdim,
        "scale": m.scale, "sink": True, "chunk": m.chunk, "shared_keys": m.kv_from is not None,
        "position": pairs(m.dim, m.rot_dims, m.rot_base) if m.rot_dims else None})


def _mlp_spec(c: BesoraxConfig, f: FeedForwardConfig, prefix: str) -> PartSpec:
    if f.kind == "dense":
        return PartSpec("gated_mlp", prefix, {"hidden_size": c.width, "intermediate_size": f.ff, "activation": "clamped",
                                              "limit": f.limit, "names": {"gate": "gate", "up": "up", "down": "down"}})
    return PartSpec("routed_mlp", prefix, {
        "hidden_size": c.width, "intermediate_size": f.ff, "experts": f.experts, "top": f.top, "activation": "gelu",
        "scores": "sigmoid", "normalize": False, "router_bias": False, "weigh_input": True,
        "shared_intermediate_size": f.shared_ff, "shared_gate": False})


def besorax_model_spec(c: BesoraxConfig) -> ModelSpec:
    def norm(prefix: str, name: str) -> PartSpec:
        return PartSpec("dynamic_tanh", prefix, {"size": c.width, "param": name})
    layers = []
    for i, L in enumerate(c.layers):
        p = f"l{i}."
        parts: Dict[str, Optional[PartSpec]] = {"norm1": norm(p, "norm1"), "mixer": _mixer_spec(c, L, p + "mix.")}
        if L.mlp is not None:
            parts.update({"norm2": norm(p, "norm2"), "feed_forward": _mlp_spec(c, L.mlp, p + "mlp.")})
        layers.append(LayerSpec(block="prenorm", parts=parts))
    return ModelSpec(
        architecture=c.architecture, hidden_size=c.width, vocab_size=c.vocab, max_positions=c.max_positions,
        embedding=PartSpec("token_embedding", "", {"vocab_size": c.vocab, "hidden_size": c.width, "param": "embed",
                                                   "scale": c.embedding_scale}),
        layers=tuple(layers),
        order=tuple(ExecEntry(i, cache_from=getattr(L.mixer, "kv_from", None)) for i, L in enumerate(c.layers)),
        final_norm=norm("final.", "norm"),
        head=PartSpec("linear_head", "", {"vocab_size": c.vocab, "hidden_size": c.width, "param": "head"}),
        eos_token_ids=c.eos_token_ids, residual_scale=c.residual_mult)
