"""The Bemizen decoder as a ModelSpec: a token embedding; pre-norm layers in the order the
configuration lists them, each a mixer behind a root-mean-square norm and, where the layer has one, a
choice among many small gated units behind another; the mixers are softmax attention within chunks
of the sequence, with a norm without weight on queries and keys, and softmax attention over a sliding
window and the sequence's first tokens, with a weighted norm and a gate per head; layers after the
first that says so mix that layer's values into their own. The model's norm and an untied head end
it. Every size and constant is the configuration's."""

from ..config.bemizen_config import NAME, BemizenConfig
from ..config.registry import register_architecture
from ..parts.base import PartSpec
from .spec import LayerSpec, ModelSpec, RunStep, Slot

EXPERT_ACTIVATION = "silu"          # fixed by the design


def _mixer(kind, m, width, eps, values):
    return PartSpec.of("mixer", "span_attention", hidden_size=width, heads=m.heads, kv_heads=m.kv_heads, dim=m.dim, vdim=m.vdim,
                       scale=m.scale, eps=eps, qk_norm="weighted" if kind == "attention_2" else "plain", chunk=m.chunk,
                       window=m.window, keep_first=m.keep_first, rot_dims=m.rot.dims, rot_base=m.rot.base, values=values,
                       gated=kind == "attention_2")


def _feed_forward(f, width):
    return PartSpec.of("feed_forward", "grouped_experts", hidden_size=width, experts=f.experts, top=f.top, expert_ff=f.expert_ff,
                       groups=f.groups, keep=f.keep, activation=EXPERT_ACTIVATION, scoring="softmax", identity=f.identity,
                       scale=f.scale)


def bemizen_spec(config):
    width = config.width
    norm = PartSpec.of("norm", "rms", size=width, eps=config.eps, leaf="")
    layers, first = [], True
    for i, layer in enumerate(config.layers):
        values = "own"
        if layer.mixer.mixes_values:
            values, first = ("first" if first else "mixed"), False
        slots = [Slot("mixer", _mixer(layer.type, layer.mixer, width, config.eps, values), "mix"),
                 Slot("mixer_norm", norm, "norm1")]
        if layer.mlp is not None:
            slots += [Slot("feed_forward", _feed_forward(layer.mlp, width), "mlp"), Slot("feed_forward_norm", norm, "norm2")]
        layers.append(LayerSpec(prefix="l%d" % i, slots=tuple(slots), block=PartSpec.of("block", "pre_norm")))
    return ModelSpec(
        hidden_size=width, vocab_size=config.vocab,
        embedding=PartSpec.of("embedding", "token", vocab_size=config.vocab, hidden_size=width, leaf=""),
        embedding_prefix="embed",
        position=PartSpec.of("position", "none"),
        layers=tuple(layers), order=tuple(RunStep(i) for i in range(len(layers))),
        final_norm=norm, final_norm_prefix="final.norm",
        head=PartSpec.of("head", "linear", hidden_size=width, vocab_size=config.vocab, weight_name="head"),
        # the first layer that mixes has a share of its own in the file, which nothing reads
        ignorable_tensors=tuple("l%d.mix.vmix" % i for i in range(len(layers))))


register_architecture(NAME, BemizenConfig, bemizen_spec)
