"""Kelutar: a decoder whose config.json lists its layers, each a post-norm block behind a convolution
over the stream.

    x = embed[token] * embedding.scale + pos[position]
    x += Norm1(Mixer(x + Conv(x)));  x += Norm2(FeedForward(x))        (RMS norms with plain gains)
    logits = head Norm(x)

Conv is a causal convolution over time on each channel of the stream (``parts/stream_conv.py``).  The
mixer is a softmax attention over a window whose values are the keys as projected, with a norm and a
factor per head and a gate on every output channel (``ProjectionNormAttention``), or a linear
attention whose forget gate also writes (``BoundedForgetAttention``).  The feed-forward is
down(relu(up)^2) (``PlainMLP``) or absent.  A layer with ``weights_of: j`` is a second call of block j
in the run list, with cache streams of its own.  Checkpoint names: ``embed``, ``pos``,
``l<i>.canon1``, ``l<i>.norm1``, ``l<i>.norm2``, ``l<i>.mix.*``, ``l<i>.mlp.*``, ``final.norm``,
``head``.
"""
from ..config import KelutarConfig, register_architecture
from ..parts.attention import ProjectionNormAttention
from ..parts.block import PostNormBlock
from ..parts.embedding import OutputHead, TokenEmbedding
from ..parts.feedforward import PlainMLP
from ..parts.model import LayerCall, ModelSpec
from ..parts.norm import PostRMSNorm, RMSNorm
from ..parts.position import NoPosition
from ..parts.recurrent import BoundedForgetAttention
from ..parts.stream_conv import StreamConvolution


def _mixer(cfg: KelutarConfig, layer):
    m = layer.mixer
    if layer.kind == "hgrn2":
        return BoundedForgetAttention(cfg.width, m.heads, m.dim, m.vdim, cfg.norm_eps)
    return ProjectionNormAttention(cfg.width, m.heads, m.kv_heads, m.dim, m.dim, m.scale, NoPosition(), cfg.norm_eps,
                                   bias=True, out_bias=False, window=m.window or None, projection_norm="head",
                                   values="keys", temperature=True, gate="channel")


def build_kelutar(cfg: KelutarConfig) -> ModelSpec:
    embedding = TokenEmbedding(cfg.vocab, cfg.width, name="embed", scale=cfg.embedding_scale,
                               positions=cfg.max_positions, position_name="pos")

    def norm(name):
        return PostRMSNorm(cfg.width, cfg.norm_eps, name=name)
    layers, block_of, run, streams = [], {}, [], 0
    for i, layer in enumerate(cfg.layers):
        if layer.weights_of is None:
            mlp = PlainMLP(cfg.width, layer.mlp.ff, "relu2") if layer.mlp is not None else None
            conv = StreamConvolution(cfg.width, cfg.taps, name="canon1") if cfg.taps else None
            block_of[i] = len(layers)
            layers.append((f"l{i}.", PostNormBlock(norm("norm1"), _mixer(cfg, layer), norm("norm2"), mlp,
                                                   names=("", "mix.", "", "mlp."), input_conv=conv)))
    for i, layer in enumerate(cfg.layers):
        b = block_of[i if layer.weights_of is None else layer.weights_of]
        n = len(layers[b][1].cache_specs())
        run.append(LayerCall(b, tuple(range(streams, streams + n))))
        streams += n
    return ModelSpec(
        embedding=("", embedding),
        layers=layers,
        run=run,
        final_norm=("final.", RMSNorm(cfg.width, cfg.norm_eps, name="norm")),
        head=("", OutputHead(cfg.vocab, cfg.width, name="head")),
        vocab_size=cfg.vocab,
        hidden_size=cfg.width,
        eos_token_id=-1,
        max_position_embeddings=cfg.max_positions,
    )


register_architecture("Kelutar", KelutarConfig.from_hf, build_kelutar, model_type="kelutar")
