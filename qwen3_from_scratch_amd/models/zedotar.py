"""The Zedotar decoder as a ModelSpec: a token embedding; pre-norm layers in the order the
configuration lists them, each a mixer behind a root-mean-square norm whose weight is stored around
zero and, where the layer has one, a dense gated feed-forward behind another; the mixers are softmax
attention over a sliding window and the means of what has left it, attention whose keys count by the
sigmoid of their scores and serve as values too, and the matrix memory of mLSTM. The model's norm, an
untied head and a cap on the logits end it. Every size and constant is the configuration's."""

from ..config.registry import register_architecture
from ..config.zedotar_config import NAME, ZedotarConfig
from ..parts.base import PartSpec
from .spec import LayerSpec, ModelSpec, RunStep, Slot

ACTIVATION = "gelu_tanh"            # the feed-forward's gate, fixed by the design
NORM_OFFSET = 1.0                   # a norm's multiplier is one more than its stored weight
DENOMINATOR_EPS = 1e-6              # joins the matrix memory's denominator


def _mixer(kind, m, width, eps):
    if kind == "attention":
        return PartSpec.of("mixer", "pooled_window_attention", hidden_size=width, heads=m.heads, kv_heads=m.kv_heads,
                           dim=m.dim, vdim=m.vdim, scale=m.scale, window=m.window, pool=m.pool, rot_dims=m.rot.dims,
                           rot_base=m.rot.base, rot_scaling=m.rot.scaling)
    if kind == "attention_2":
        return PartSpec.of("mixer", "sigmoid_attention", hidden_size=width, heads=m.heads, kv_heads=m.kv_heads, dim=m.dim,
                           conv=m.conv, scale=m.scale, rot_dims=m.rot.dims, rot_base=m.rot.base, rot_scaling=m.rot.scaling)
    return PartSpec.of("mixer", "mlstm", hidden_size=width, heads=m.heads, dim=m.dim, vdim=m.vdim, gate_cap=m.gate_cap,
                       eps=eps, denominator_eps=DENOMINATOR_EPS)


def zedotar_spec(config):
    width = config.width
    norm = PartSpec.of("norm", "rms", size=width, eps=config.eps, leaf="", offset=NORM_OFFSET)
    layers = []
    for i, layer in enumerate(config.layers):
        slots = [Slot("mixer", _mixer(layer.type, layer.mixer, width, config.eps), "mix"), Slot("mixer_norm", norm, "norm1")]
        if layer.ff:
            slots += [Slot("feed_forward", PartSpec.of("feed_forward", "swiglu", hidden_size=width,
                                                       intermediate_size=layer.ff, names=("gate", "up", "down"),
                                                       activation=ACTIVATION), "mlp"),
                      Slot("feed_forward_norm", norm, "norm2")]
        layers.append(LayerSpec(prefix="l%d" % i, slots=tuple(slots), block=PartSpec.of("block", "pre_norm")))
    return ModelSpec(
        hidden_size=width, vocab_size=config.vocab,
        embedding=PartSpec.of("embedding", "token", vocab_size=config.vocab, hidden_size=width, leaf=""),
        embedding_prefix="embed",
        position=PartSpec.of("position", "none"),
        layers=tuple(layers), order=tuple(RunStep(i) for i in range(len(layers))),
        final_norm=norm, final_norm_prefix="final.norm",
        head=PartSpec.of("head", "linear", hidden_size=width, vocab_size=config.vocab, weight_name="head",
                         softcap=config.logit_softcap))


register_architecture(NAME, ZedotarConfig, zedotar_spec)
