"""Typed configuration of the Zedotar decoder, read from its own config.json keys.

Its config.json is nested like Kodisun's: `layers` lists the layers (`type` names the mixer, `mixer`
holds its sizes and constants, `mlp` the feed-forward's or null), `norm.eps` is every norm's epsilon,
`logit_softcap` bends the logits. The architecture is named by the string `architecture`. No size has
a default: one that is missing is an error; what may be absent (a rotation, its scaling, a window, a
feed-forward, the logits' cap) is absent as a whole.
"""

import copy
import json
from dataclasses import dataclass

from .kodisun_config import NO_POSITION_LIMIT, _get, _positive
from .model_config import ConfigError

NAME = "Zedotar"


@dataclass(frozen=True)
class ScaledTurning:
    """A rotary encoding of the first `dims` numbers of a head, i and i + dims / 2 together, by
    base^(-2i / dims). `scaling`: None, ("bands", factor, original, low, high) or ("ramp", factor,
    original, fast, slow), which of them by the keys that config.json's `scaling` has."""

    dims: int = 0
    base: float = 1.0
    scaling: tuple = None

    @classmethod
    def read(cls, data, where, most):
        if data is None:
            return cls()
        dims, base = _positive(data, "dims", where), _get(data, "base", float, where)
        if dims % 2 or dims > most:
            raise ConfigError("config.json: %s.dims must be even and at most the head's size %d" % (where, most))
        if base <= 0:
            raise ConfigError("config.json: %s.base must be positive" % where)
        scaling = data.get("scaling")
        if scaling is not None:
            s = where + ".scaling"
            kind, keys = (("bands", ("factor", "original", "low", "high")) if "low" in scaling or "high" in scaling
                          else ("ramp", ("factor", "original", "fast", "slow")))
            numbers = tuple(_get(scaling, key, float, s) for key in keys)
            if min(numbers) <= 0:
                raise ConfigError("config.json: %s must hold positive numbers" % s)
            if kind == "bands" and numbers[2] == numbers[3]:
                raise ConfigError("config.json: %s.low and high must differ" % s)
            if kind == "ramp" and base == 1.0:
                raise ConfigError("config.json: %s.base must not be 1 with such a scaling" % where)
            scaling = (kind,) + numbers
        return cls(dims, base, scaling)


def _heads(data, where):
    heads, kv_heads = _positive(data, "heads", where), _positive(data, "kv_heads", where)
    if heads % kv_heads:
        raise ConfigError("config.json: %s.kv_heads (%d) must divide heads (%d)" % (where, kv_heads, heads))
    return heads, kv_heads


@dataclass(frozen=True)
class PooledWindowSizes:
    """Softmax attention over a sliding window of `window` tokens (0: all of them) and, as one key and
    value each, the runs of `pool` tokens that have left it (0: nothing behind the window)."""

    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    window: int
    pool: int
    rot: ScaledTurning

    @classmethod
    def read(cls, data, where):
        heads, kv_heads = _heads(data, where)
        dim = _positive(data, "dim", where)
        mask, window, pool = data.get("mask"), 0, 0
        if mask is not None:
            window = _positive(mask, "size", where + ".mask")
            pool = _positive(mask, "pool", where + ".mask") if mask.get("pool") is not None else 0
        return cls(heads=heads, kv_heads=kv_heads, dim=dim, vdim=_positive(data, "vdim", where),
                   scale=_get(data, "scale", float, where), window=window, pool=pool,
                   rot=ScaledTurning.read(data.get("rot"), where + ".rot", dim))


@dataclass(frozen=True)
class SigmoidAttentionSizes:
    """Attention whose keys count by the sigmoid of their scores; the values are the unturned keys,
    so `vdim`, where it is given, is `dim`."""

    heads: int
    kv_heads: int
    dim: int
    conv: int
    scale: float
    rot: ScaledTurning

    @classmethod
    def read(cls, data, where):
        heads, kv_heads = _heads(data, where)
        dim = _positive(data, "dim", where)
        if data.get("vdim") is not None and _positive(data, "vdim", where) != dim:
            raise ConfigError("config.json: %s.vdim must equal dim: the values are the keys" % where)
        return cls(heads=heads, kv_heads=kv_heads, dim=dim, conv=_positive(data, "conv", where),
                   scale=_get(data, "scale", float, where), rot=ScaledTurning.read(data.get("rot"), where + ".rot", dim))


@dataclass(frozen=True)
class MatrixMemorySizes:
    heads: int
    dim: int
    vdim: int
    gate_cap: float

    @classmethod
    def read(cls, data, where):
        cap = _get(data, "gate_cap", float, where)
        if not cap > 0:
            raise ConfigError("config.json: %s.gate_cap must be positive" % where)
        return cls(heads=_positive(data, "heads", where), dim=_positive(data, "dim", where),
                   vdim=_positive(data, "vdim", where), gate_cap=cap)


MIXERS = {"attention": PooledWindowSizes, "attention_2": SigmoidAttentionSizes, "mlstm": MatrixMemorySizes}


@dataclass(frozen=True)
class ZedotarLayer:
    type: str
    mixer: object
    ff: int = 0             # the dense feed-forward's inner size; 0: the layer has none


@dataclass(frozen=True)
class ZedotarConfig:
    architecture: str
    vocab: int
    width: int
    eps: float
    logit_softcap: float    # 0: the logits are not capped
    layers: tuple
    raw: str                # config.json as it was read, for `to_dict`
    eos_token_ids: tuple = ()
    max_position_embeddings: int = NO_POSITION_LIMIT

    @classmethod
    def from_dict(cls, data):
        listed = _get(data, "layers", list, "config")
        if not listed:
            raise ConfigError("config.json: 'layers' is empty")
        layers = []
        for i, entry in enumerate(listed):
            where = "layers[%d]" % i
            kind = _get(entry, "type", str, where)
            if kind not in MIXERS:
                raise ConfigError("config.json: %s.type %r is not known (one of %s)" % (where, kind, ", ".join(sorted(MIXERS))))
            mixer = MIXERS[kind].read(_get(entry, "mixer", dict, where), where + ".mixer")
            mlp, ff = entry.get("mlp"), 0
            if mlp is not None:
                if _get(mlp, "kind", str, where + ".mlp") != "dense":
                    raise ConfigError("config.json: %s.mlp.kind %r is not known (only 'dense')" % (where, mlp["kind"]))
                ff = _positive(mlp, "ff", where + ".mlp")
            layers.append(ZedotarLayer(kind, mixer, ff))
        eps = _get(_get(data, "norm", dict, "config"), "eps", float, "norm")
        if not eps >= 0.0:
            raise ConfigError("config.json: norm.eps must not be negative")
        cap = _get(data, "logit_softcap", float, "config") if data.get("logit_softcap") is not None else 0.0
        if cap < 0:
            raise ConfigError("config.json: logit_softcap must not be negative")
        return cls(architecture=NAME, vocab=_positive(data, "vocab", "config"), width=_positive(data, "width", "config"),
                   eps=eps, logit_softcap=cap, layers=tuple(layers), raw=json.dumps(data, sort_keys=True))

    def to_dict(self):
        return copy.deepcopy(json.loads(self.raw))
