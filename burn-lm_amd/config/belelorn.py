"""Typed configuration of the Belelorn design, read from the keys of its ``config.json``.

Top level: ``vocab``, ``width``, ``norm.eps``, ``logit_scale``, ``layers`` and optionally ``loop: {start, stop, times}``
(layers start .. stop - 1 run that many times in a row).  ``layers`` is a list of ``{type, mixer, mlp}``.  ``type`` names
the mixer: ``mlstm`` (``heads, dim, vdim, gate_cap``) or ``parallel``, two mixers side by side: ``left`` (softmax attention:
``heads, kv_heads, dim, vdim, scale, softcap, mask: {size, keep_first}``) and ``right`` (lightning attention: ``heads,
dim, vdim, decay`` with one decay per head, or one number for all).  ``mlp`` is ``null`` (none), ``{kind: dense, ff}`` or
``{kind: moe, expert: {ff, limit}, router: {experts, top}, shared: {ff, limit}}``.  Every size is a required key;
``softcap``, ``mask`` and ``shared`` may be missing or null (none)."""
from __future__ import annotations

from dataclasses import dataclass
from typing import Optional, Tuple, Union

from ..errors import ConfigError

MAX_POSITIONS = 1 << 20     # the design has no limit of its own; the cache's size decides


def _get(d, key, kind, where, least=1):
    if not isinstance(d, dict) or key not in d or d[key] is None:
        raise ConfigError(f"config.json: required key '{key}' is missing in {where}")
    v = d[key]
    if kind is int:
        if isinstance(v, bool) or not isinstance(v, int) or v < least:
            raise ConfigError(f"config.json: '{key}' in {where} must be an integer of at least {least}, got {v!r}")
        return v
    if isinstance(v, bool) or not isinstance(v, (int, float)):
        raise ConfigError(f"config.json: '{key}' in {where} must be a number, got {v!r}")
    return float(v)


def _positive(d, key, where):
    v = _get(d, key, float, where)
    if v <= 0.0:
        raise ConfigError(f"config.json: '{key}' in {where} must be positive, got {v!r}")
    return v


@dataclass(frozen=True)
class SoftmaxSide:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    softcap: float        # 0: none
    window: int           # 0: every earlier key
    keep_first: int


@dataclass(frozen=True)
class LightningSide:
    heads: int
    dim: int
    vdim: int
    decay: Tuple[float, ...]


@dataclass(frozen=True)
class PairConfig:
    left: SoftmaxSide
    right: LightningSide
    kind: str = "parallel"


@dataclass(frozen=True)
class MlstmConfig:
    heads: int
    dim: int
    vdim: int
    gate_cap: float
    kind: str = "mlstm"


@dataclass(frozen=True)
class DenseConfig:
    ff: int
    kind: str = "dense"


@dataclass(frozen=True)
class MoeConfig:
    experts: int
    top: int
    ff: int
    limit: float
    shared_ff: int        # 0: no shared expert
    shared_limit: float
    kind: str = "moe"


@dataclass(frozen=True)
class LayerConfig:
    mixer: Union[PairConfig, MlstmConfig]
    mlp: Optional[Union[DenseConfig, MoeConfig]]


@dataclass(frozen=True)
class LoopConfig:
    start: int
    stop: int
    times: int


def _softmax_side(m, where):
    heads, kv_heads = _get(m, "heads", int, where), _get(m, "kv_heads", int, where)
    if heads % kv_heads:
        raise ConfigError(f"config.json: {where}.heads must be a multiple of kv_heads")
    dim, vdim = _get(m, "dim", int, where), _get(m, "vdim", int, where)
    if vdim != dim:
        raise ConfigError(f"config.json: {where}.vdim must equal dim: the values of this attention are its keys")
    mask, mw = m.get("mask"), where + ".mask"
    window = _get(mask, "size", int, mw) if mask is not None else 0
    keep = _get(mask, "keep_first", int, mw, least=0) if mask is not None and mask.get("keep_first") is not None else 0
    cap = _positive(m, "softcap", where) if m.get("softcap") is not None else 0.0
    return SoftmaxSide(heads, kv_heads, dim, vdim, _get(m, "scale", float, where), cap, window, keep)


def _lightning_side(m, where):
    heads = _get(m, "heads", int, where)
    decay = m.get("decay")
    if isinstance(decay, (int, float)) and not isinstance(decay, bool):
        decay = [decay] * heads      # one number for all heads
    if not isinstance(decay, list) or len(decay) != heads \
            or not all(isinstance(a, (int, float)) and not isinstance(a, bool) and 0.0 < a <= 1.0 for a in decay):
        raise ConfigError(f"config.json: {where}.decay must list one number in (0, 1] for each of the {heads} heads")
    return LightningSide(heads, _get(m, "dim", int, where), _get(m, "vdim", int, where), tuple(float(a) for a in decay))


def _feed_forward(mlp, where):
    if mlp is None:
        return None
    kind = mlp.get("kind") if isinstance(mlp, dict) else None
    if kind == "dense":
        return DenseConfig(_get(mlp, "ff", int, where))
    if kind != "moe":
        raise ConfigError(f"config.json: {where}.kind is {kind!r}; known: dense, moe")
    router, expert, shared = mlp.get("router"), mlp.get("expert"), mlp.get("shared")
    experts, top = _get(router, "experts", int, where + ".router"), _get(router, "top", int, where + ".router")
    if top > experts:
        raise ConfigError(f"config.json: {where}.router.top is more than its {experts} experts")
    sw = where + ".shared"
    return MoeConfig(experts, top, _get(expert, "ff", int, where + ".expert"), _positive(expert, "limit", where + ".expert"),
                     _get(shared, "ff", int, sw) if shared is not None else 0,
                     _positive(shared, "limit", sw) if shared is not None else 0.0)


@dataclass(frozen=True)
class BelelornConfig:
    vocab: int
    width: int
    eps: float
    logit_scale: float
    layers: Tuple[LayerConfig, ...]
    loop: Optional[LoopConfig]

    @property
    def vocab_size(self):
        return self.vocab

    @property
    def max_positions(self):
        return MAX_POSITIONS

    @classmethod
    def from_dict(cls, d: dict) -> "BelelornConfig":
        layers = d.get("layers")
        if not isinstance(layers, list) or not layers:
            raise ConfigError("config.json: 'layers' must be a non-empty list")
        out = []
        for i, entry in enumerate(layers):
            where = f"layers[{i}]"
            kind = entry.get("type") if isinstance(entry, dict) else None
            m, mw = (entry.get("mixer") or {}) if isinstance(entry, dict) else {}, where + ".mixer"
            if kind == "parallel":
                mixer = PairConfig(_softmax_side(m.get("left") or {}, mw + ".left"), _lightning_side(m.get("right") or {}, mw + ".right"))
            elif kind == "mlstm":
                mixer = MlstmConfig(_get(m, "heads", int, mw), _get(m, "dim", int, mw), _get(m, "vdim", int, mw),
                                    _positive(m, "gate_cap", mw))
            else:
                raise ConfigError(f"config.json: {where}.type is {kind!r}; known: parallel, mlstm")
            out.append(LayerConfig(mixer, _feed_forward(entry.get("mlp"), where + ".mlp")))
        loop = d.get("loop")
        if loop is not None:
            loop = LoopConfig(_get(loop, "start", int, "loop", least=0), _get(loop, "stop", int, "loop"), _get(loop, "times", int, "loop"))
            if not loop.start < loop.stop <= len(out):
                raise ConfigError(f"config.json: loop: layers {loop.start} to {loop.stop - 1} are not a run of the {len(out)} layers")
        top = "the top level"
        return cls(vocab=_get(d, "vocab", int, top), width=_get(d, "width", int, top), eps=_get(d.get("norm"), "eps", float, "norm"),
                   logit_scale=_get(d, "logit_scale", float, top), layers=tuple(out), loop=loop)
