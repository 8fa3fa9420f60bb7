"""Typed configuration of the Netanex design, read from the keys of its ``config.json``.

Top level: ``vocab``, ``width``, ``norm.eps`` and ``layers``, a list of ``{type, mixer, mlp}`` and optionally ``weights_of: j``
(the layer uses layer j's tensors; the rest of its entry equals layer j's).  ``type`` names the mixer: ``attention``
(differential: ``heads, kv_heads, dim, vdim, scale, diff`` and optionally ``q_temp: {coef, every}``), ``latent_attention``
(``heads, dim, rot_dim, vdim, kv_rank, scale, rot: {dims, base, scaling}`` and optionally ``mask: {size}``; ``scaling`` may be
null or ``{factor, original, fast, slow}``) or ``attention_2`` (``heads, kv_heads, dim, vdim, scale``).  ``mlp`` is ``null``
(none) or ``{kind: moe, expert: {ff}, router: {experts, top}}``.  Every size is a required key."""
from __future__ import annotations

from dataclasses import dataclass
from typing import Optional, Tuple, Union

from ..errors import ConfigError

MAX_POSITIONS = 1 << 20     # the design has no limit of its own; the cache's size decides


def _get(d, key, kind, where, least=1):
    if not isinstance(d, dict) or key not in d or d[key] is None:
        raise ConfigError(f"config.json: required key '{key}' is missing in {where}")
    v = d[key]
    if isinstance(v, bool) or not isinstance(v, (int, float)):
        raise ConfigError(f"config.json: '{key}' in {where} must be a number, got {v!r}")
    if kind is int:
        if v != int(v) or v < least:
            raise ConfigError(f"config.json: '{key}' in {where} must be an integer of at least {least}, got {v!r}")
        return int(v)
    return float(v)


def _positive(d, key, where):
    v = _get(d, key, float, where)
    if v <= 0.0:
        raise ConfigError(f"config.json: '{key}' in {where} must be positive, got {v!r}")
    return v


def _heads(m, where):
    heads, kv_heads = _get(m, "heads", int, where), _get(m, "kv_heads", int, where)
    if heads % kv_heads:
        raise ConfigError(f"config.json: {where}.heads must be a multiple of kv_heads")
    return heads, kv_heads


@dataclass(frozen=True)
class DifferentialConfig:
    heads: int
    kv_heads: int
    dim: int               # of one map
    vdim: int
    scale: float
    diff: float
    growth: Optional[Tuple[float, int]]     # (coef, every) of the queries' growth with their position
    kind: str = "attention"


@dataclass(frozen=True)
class LatentConfig:
    heads: int
    dim: int
    rot_dim: int
    vdim: int
    kv_rank: int
    scale: float
    window: int            # 0: every earlier token
    rot_dims: int
    rot_base: float
    yarn: Optional[Tuple[float, float, float, float]]     # factor, original, fast, slow
    kind: str = "latent_attention"


@dataclass(frozen=True)
class GatedConfig:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    kind: str = "attention_2"


@dataclass(frozen=True)
class MoeConfig:
    experts: int
    top: int
    ff: int


@dataclass(frozen=True)
class LayerConfig:
    mixer: Union[DifferentialConfig, LatentConfig, GatedConfig]
    mlp: Optional[MoeConfig]
    owner: int             # the layer whose tensors it uses (its own number unless weights_of says otherwise)


def _differential(m, where):
    heads, kv_heads = _heads(m, where)
    growth, gw = m.get("q_temp"), where + ".q_temp"
    if growth is not None:
        growth = (_get(growth, "coef", float, gw), _get(growth, "every", int, gw))
    return DifferentialConfig(heads, kv_heads, _get(m, "dim", int, where), _get(m, "vdim", int, where), _get(m, "scale", float, where),
                              _get(m, "diff", float, where), growth)


def _latent(m, where):
    rot, mask, rw = m.get("rot"), m.get("mask"), where + ".rot"
    rot_dim, dims = _get(m, "rot_dim", int, where), _get(rot, "dims", int, rw)
    if dims % 2 or dims != rot_dim:
        raise ConfigError(f"config.json: {rw}.dims must be even and equal rot_dim = {rot_dim}, got {dims}")
    scaling, yarn = rot.get("scaling"), None
    if scaling is not None:
        yarn = tuple(_positive(scaling, k, rw + ".scaling") for k in ("factor", "original", "fast", "slow"))
    return LatentConfig(_get(m, "heads", int, where), _get(m, "dim", int, where), rot_dim, _get(m, "vdim", int, where),
                        _get(m, "kv_rank", int, where), _get(m, "scale", float, where),
                        _get(mask, "size", int, where + ".mask") if mask is not None else 0, dims, _positive(rot, "base", rw), yarn)


def _gated(m, where):
    heads, kv_heads = _heads(m, where)
    return GatedConfig(heads, kv_heads, _get(m, "dim", int, where), _get(m, "vdim", int, where), _get(m, "scale", float, where))


MIXERS = {"attention": _differential, "latent_attention": _latent, "attention_2": _gated}


def _feed_forward(mlp, where):
    if mlp is None:
        return None
    kind = mlp.get("kind") if isinstance(mlp, dict) else None
    if kind != "moe":
        raise ConfigError(f"config.json: {where}.kind is {kind!r}; known: moe")
    router = mlp.get("router")
    experts, top = _get(router, "experts", int, where + ".router"), _get(router, "top", int, where + ".router")
    if top > experts:
        raise ConfigError(f"config.json: {where}.router.top is more than its {experts} experts")
    return MoeConfig(experts, top, _get(mlp.get("expert"), "ff", int, where + ".expert"))


@dataclass(frozen=True)
class NetanexConfig:
    vocab: int
    width: int
    eps: float
    layers: Tuple[LayerConfig, ...]

    @property
    def vocab_size(self):
        return self.vocab

    @property
    def max_positions(self):
        return MAX_POSITIONS

    @classmethod
    def from_dict(cls, d: dict) -> "NetanexConfig":
        layers = d.get("layers")
        if not isinstance(layers, list) or not layers:
            raise ConfigError("config.json: 'layers' must be a non-empty list")
        out = []
        for i, entry in enumerate(layers):
            where = f"layers[{i}]"
            kind = entry.get("type") if isinstance(entry, dict) else None
            if kind not in MIXERS:
                raise ConfigError(f"config.json: {where}.type is {kind!r}; known: {', '.join(MIXERS)}")
            mixer = MIXERS[kind](entry.get("mixer") or {}, where + ".mixer")
            mlp, owner = _feed_forward(entry.get("mlp"), where + ".mlp"), i
            if entry.get("weights_of") is not None:
                owner = _get(entry, "weights_of", int, where, least=0)
                if owner >= i:
                    raise ConfigError(f"config.json: {where}.weights_of must name an earlier layer, got {owner}")
                if (mixer, mlp) != (out[owner].mixer, out[owner].mlp):
                    raise ConfigError(f"config.json: {where} differs from layer {owner}, whose weights_of it takes")
                owner = out[owner].owner
            out.append(LayerConfig(mixer, mlp, owner))
        top = "the top level"
        return cls(vocab=_get(d, "vocab", int, top), width=_get(d, "width", int, top), eps=_get(d.get("norm"), "eps", float, "norm"),
                   layers=tuple(out))
