"""Lotinex: a decoder whose stream is kept in several copies and whose config.json lists its layers.

    x_1 = .. = x_s = embed[token] * embedding.scale
    u = sum_s in_s x_s;  y = Sublayer(Norm(u));  x_t <- sum_s mix[s, t] x_s + out_t y     (each sublayer)
    logits = embed Norm(sum_s x_s)                                  (layer norms with gain and bias)

Mixers: grouped-query attention within chunks of positions, with a norm per head, whose keys and
values may be those of an earlier layer (``ProjectionNormAttention``: the run list then hands it that
layer's pages to read); the gated delta rule with one decay a head (``GatedDeltaRule``); and two mixers
side by side with a norm on each output (``SideBySide``): attention over a window behind a short
convolution, with a norm over the projection, blended frequencies, capped scores and a sink of score 0
(``ShortConvAttention``), and a selective scan (``SelectiveStateMixer``).  Feed-forward: gated by silu
and dense (``GatedMLP``), or experts chosen by their logits and weighted, on their inputs, by the
sigmoid (``RoutedExperts``), or absent.  Checkpoint names: ``embed``, ``l<i>.norm1[.b]``,
``l<i>.norm2[.b]``, ``l<i>.hc1.*``, ``l<i>.hc2.*``, ``l<i>.mix.*``, ``l<i>.mlp.*``, ``final.norm[.b]``.
"""
from ..config import LotinexConfig, register_architecture
from ..config.lotinex import DenseGatedConfig
from ..parts.attention import ProjectionNormAttention, ShortConvAttention
from ..parts.block import StreamsBlock
from ..parts.embedding import OutputHead, TokenEmbedding
from ..parts.feedforward import GatedMLP
from ..parts.model import LayerCall, ModelSpec
from ..parts.norm import LayerNorm
from ..parts.position import NoPosition, RotaryPosition, blended_frequencies, blended_magnitude, plain_frequencies
from ..parts.recurrent import GatedDeltaRule, SelectiveStateMixer, SideBySide
from ..parts.routed import RoutedExperts
from ..parts.streams import StreamLink


def _position(rot, head_dim):
    if not rot.dims:
        return NoPosition()
    frequencies, magnitude = plain_frequencies(rot.dims, rot.base), 1.0
    if rot.scaling is not None:
        _, factor, original, fast, slow = rot.scaling
        frequencies = blended_frequencies(rot.dims, rot.base, factor, original, fast, slow)
        magnitude = blended_magnitude(factor)
    return RotaryPosition(head_dim, rot.base, rotary_dim=rot.dims, frequencies=frequencies, magnitude=magnitude)


def _mixer(cfg: LotinexConfig, layer):
    m, w, eps = layer.mixer, cfg.width, cfg.norm_eps
    if layer.kind == "attention":
        return ProjectionNormAttention(w, m.heads, m.kv_heads, m.dim, m.vdim, m.scale, _position(m.rot, m.dim), eps,
                                       bias=False, projection_norm="head", chunk=m.reach or None,
                                       shared_keys=m.kv_from is not None)
    if layer.kind == "delta":
        return GatedDeltaRule(w, m.heads, m.kv_heads, m.dim, m.vdim, m.conv, 0, 0, eps, decay="head", gate="silu")
    l, r = m.left, m.right
    args = (w, l.heads, l.kv_heads, l.dim, l.vdim, l.scale, _position(l.rot, l.dim), eps)
    options = dict(bias=False, projection_norm=True, window=l.reach or None, softcap=l.softcap or None, sink=0.0)
    left = ShortConvAttention(*args, conv=l.conv, **options) if l.conv else ProjectionNormAttention(*args, **options)
    return SideBySide(left, SelectiveStateMixer(w, r.inner, r.state, r.dt_rank, r.conv), 0.5, 0.5,
                      out_norms=("left.out", "right.out"), hidden_size=w, norm_eps=eps)


def _feedforward(cfg: LotinexConfig, c):
    if c is None:
        return None
    if isinstance(c, DenseGatedConfig):
        return GatedMLP(cfg.width, c.ff, "silu", names=("gate", "up", "down"))
    return RoutedExperts(cfg.width, c.experts, c.top, c.ff, routing="sigmoid", weigh="input")


def build_lotinex(cfg: LotinexConfig) -> ModelSpec:
    embedding = TokenEmbedding(cfg.vocab, cfg.width, name="embed", scale=cfg.embedding_scale, copies=cfg.streams)

    def norm(name):
        return LayerNorm(cfg.width, cfg.norm_eps, name=name, bias_name=name + ".b")
    layers, run, streams_of, streams = [], [], {}, 0
    for i, layer in enumerate(cfg.layers):
        block = StreamsBlock(StreamLink(cfg.streams), norm("norm1"), _mixer(cfg, layer), StreamLink(cfg.streams),
                             norm("norm2"), _feedforward(cfg, layer.mlp))
        layers.append((f"l{i}.", block))
        owner = layer.mixer.kv_from if layer.kind == "attention" else None
        if owner is not None:                       # another layer's pages, read and not written
            run.append(LayerCall(i, streams_of[owner], write=False))
            continue
        n = len(block.cache_specs())
        streams_of[i] = tuple(range(streams, streams + n))
        run.append(LayerCall(i, streams_of[i]))
        streams += n
    return ModelSpec(
        embedding=("", embedding),
        layers=layers,
        run=run,
        final_norm=("final.", norm("norm")),
        head=("", OutputHead(cfg.vocab, cfg.width, tied_to=embedding)),
        vocab_size=cfg.vocab,
        hidden_size=cfg.width,
        eos_token_id=-1,
    )


register_architecture("Lotinex", LotinexConfig.from_hf, build_lotinex, model_type="lotinex")
