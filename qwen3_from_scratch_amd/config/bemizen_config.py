"""Typed configuration of the Bemizen decoder, read from its own config.json keys.

Its config.json is nested like Kodisun's: `layers` lists the layers (`type` names the mixer, `mixer`
holds its sizes and constants, `mlp` the feed-forward's or null), `norm.eps` is every norm's epsilon.
The architecture is named by the string `architecture`. No size has a default: one that is missing
is an error; what may be absent (a mask, a rotation, first tokens that stay, groups of experts,
experts that give their input back, a feed-forward) is absent as a whole.
"""

import copy
import json
from dataclasses import dataclass

from .kodisun_config import NO_POSITION_LIMIT, _get, _positive
from .model_config import ConfigError
from .zedotar_config import ScaledTurning, _heads

NAME = "Bemizen"


def _count(data, key, where):
    """A number that may be absent or null (then 0) and must not be negative."""
    if data.get(key) is None:
        return 0
    value = _get(data, key, int, where)
    if value < 0:
        raise ConfigError("config.json: %s.%s must not be negative" % (where, key))
    return value


def _rotation(data, where, dim):
    rot = ScaledTurning.read(data, where, dim)
    if rot.scaling is not None:
        raise ConfigError("config.json: %s.scaling is not part of this architecture" % where)
    return rot


@dataclass(frozen=True)
class SpanSizes:
    """Softmax attention over a part of the tokens before: `chunk` (0: none) is the length of the stretches
    that see nothing of each other, `window` (0: all) how many of the last tokens are seen, `keep_first`
    how many of a sequence's first tokens are seen besides. `mixes_values`: the layer takes part in the
    mixing of values."""

    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    rot: ScaledTurning
    mixes_values: bool
    chunk: int = 0
    window: int = 0
    keep_first: int = 0

    @classmethod
    def read(cls, data, where, chunked):
        heads, kv_heads = _heads(data, where)
        dim = _positive(data, "dim", where)
        mask, span, mixes = data.get("mask"), {}, data.get("v_mix")
        if mixes is not None and not isinstance(mixes, bool):
            raise ConfigError("config.json: %s.v_mix must be true or false, found %r" % (where, mixes))
        if mask is not None:
            size = _positive(mask, "size", where + ".mask")
            span = dict(chunk=size) if chunked else dict(window=size, keep_first=_count(mask, "keep_first", where + ".mask"))
        return cls(heads=heads, kv_heads=kv_heads, dim=dim, vdim=_positive(data, "vdim", where),
                   scale=_get(data, "scale", float, where), rot=_rotation(data.get("rot"), where + ".rot", dim),
                   mixes_values=bool(mixes), **span)


MIXERS = {"attention": lambda data, where: SpanSizes.read(data, where, chunked=True),
          "attention_2": lambda data, where: SpanSizes.read(data, where, chunked=False)}


@dataclass(frozen=True)
class RoutedSizes:
    experts: int
    identity: int           # further choices of the router that give the input back
    top: int
    groups: int             # 1 without groups
    keep: int
    scale: float
    expert_ff: int

    @classmethod
    def read(cls, data, where):
        router = _get(data, "router", dict, where)
        r = where + ".router"
        groups, count, keep = router.get("groups"), 1, 1
        if groups is not None:
            count, keep = _positive(groups, "count", r + ".groups"), _positive(groups, "keep", r + ".groups")
        sizes = cls(experts=_positive(router, "experts", r), identity=_count(router, "identity", r),
                    top=_positive(router, "top", r), groups=count, keep=keep,
                    scale=_get(router, "scale", float, r) if router.get("scale") is not None else 1.0,
                    expert_ff=_positive(_get(data, "expert", dict, where), "ff", where + ".expert"))
        choices = sizes.experts + sizes.identity
        if sizes.top > choices:
            raise ConfigError("config.json: %s.top exceeds the number of experts" % r)
        if choices % sizes.groups:
            raise ConfigError("config.json: %s.groups.count (%d) must divide the experts, those that give their input back "
                              "included (%d)" % (r, sizes.groups, choices))
        if sizes.keep > sizes.groups:
            raise ConfigError("config.json: %s.groups.keep exceeds groups.count" % r)
        if sizes.top > sizes.keep * (choices // sizes.groups):
            raise ConfigError("config.json: %s.top (%d) exceeds the experts of the %d groups that are kept"
                              % (r, sizes.top, sizes.keep))
        return sizes


@dataclass(frozen=True)
class BemizenLayer:
    type: str
    mixer: SpanSizes
    mlp: RoutedSizes = None


@dataclass(frozen=True)
class BemizenConfig:
    architecture: str
    vocab: int
    width: int
    eps: float
    layers: tuple
    raw: str                    # config.json as it was read, for `to_dict`
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
            mixer = MIXERS[kind](_get(entry, "mixer", dict, where), where + ".mixer")
            mlp = entry.get("mlp")
            if mlp is not None:
                if _get(mlp, "kind", str, where + ".mlp") != "moe":
                    raise ConfigError("config.json: %s.mlp.kind %r is not known (only 'moe')" % (where, mlp["kind"]))
                mlp = RoutedSizes.read(mlp, where + ".mlp")
            layers.append(BemizenLayer(kind, mixer, mlp))
        mixing = [(i, layer.mixer.kv_heads * layer.mixer.vdim) for i, layer in enumerate(layers) if layer.mixer.mixes_values]
        for i, numbers in mixing:
            if numbers != mixing[0][1]:
                raise ConfigError("config.json: layers[%d].mixer has %d numbers of values a token, layers[%d].mixer, whose values "
                                  "it mixes in, %d" % (i, numbers, mixing[0][0], mixing[0][1]))
        eps = _get(_get(data, "norm", dict, "config"), "eps", float, "norm")
        if not eps >= 0.0:
            raise ConfigError("config.json: norm.eps must not be negative")
        return cls(architecture=NAME, vocab=_positive(data, "vocab", "config"), width=_positive(data, "width", "config"),
                   eps=eps, layers=tuple(layers), raw=json.dumps(data, sort_keys=True))

    def to_dict(self):
        return copy.deepcopy(json.loads(self.raw))
