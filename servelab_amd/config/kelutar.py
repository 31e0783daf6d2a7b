"""Configuration of the Kelutar design: a decoder whose config.json lists its layers, each a softmax
attention over a window or a linear attention with a bounded forget gate, behind a convolution over
the stream, with the norms on the sublayers' outputs.

    {"architecture": "Kelutar", "width", "vocab", "max_positions", "norm": {"eps"},
     "embedding": {"scale"}, "canon": {"taps"} | absent,
     "layers": [{"type", "mixer": {...}, "mlp": {"kind": "dense", "ff"} | null, "weights_of"?}]}

Mixers:
  ``attention``  heads, kv_heads, dim (= vdim: the values are the keys as projected), scale, mask
                 ({size}: a window; absent: every earlier key)
  ``hgrn2``      heads, dim, vdim
``max_positions`` is the length of the learned table of positions and so the longest sequence;
``canon.taps`` the length of the convolution in front of every mixer (absent or 0: none).  A layer
with ``weights_of: j`` runs layer j's tensors against a cache of its own.  Nothing here is a default
for a size or a constant of the model.
"""
from dataclasses import dataclass, field
from typing import Any, Dict, List, Optional

from .layered import _section, weights_owner
from .model import ConfigError, read_key


@dataclass(frozen=True)
class TemperedAttentionConfig:
    heads: int
    kv_heads: int
    dim: int                     # query, key and value channels of a head
    scale: float
    window: int = 0              # 0: every earlier key


@dataclass(frozen=True)
class BoundedForgetConfig:
    heads: int
    dim: int
    vdim: int


@dataclass(frozen=True)
class PlainMlpConfig:
    ff: int


@dataclass(frozen=True)
class KelutarLayer:
    kind: str                    # "attention" | "hgrn2"
    mixer: Any
    mlp: Optional[PlainMlpConfig]
    weights_of: Optional[int] = None


def _read_mixer(kind: str, m: Dict[str, Any], where: str):
    if kind == "attention":
        mask = _section(m, "mask", where, required=False)
        c = TemperedAttentionConfig(
            heads=read_key(m, "heads", kind=int), kv_heads=read_key(m, "kv_heads", kind=int),
            dim=read_key(m, "dim", kind=int), scale=read_key(m, "scale", kind=float),
            window=read_key(mask, "size", 0, kind=int) if mask is not None else 0)
        if min(c.heads, c.kv_heads, c.dim) < 1 or c.heads % c.kv_heads or c.window < 0 \
                or read_key(m, "vdim", c.dim, kind=int) != c.dim:
            raise ConfigError(f"config.json: {where}: heads must be a positive multiple of kv_heads, dim positive and "
                              "equal to vdim (the values are the keys), mask.size not negative")
        return c
    if kind == "hgrn2":
        c = BoundedForgetConfig(read_key(m, "heads", kind=int), read_key(m, "dim", kind=int),
                                read_key(m, "vdim", kind=int))
        if min(c.heads, c.dim, c.vdim) < 1:
            raise ConfigError(f"config.json: {where}: heads, dim and vdim must be positive")
        return c
    raise ConfigError(f"config.json: {where}: type {kind!r} is not one of attention, hgrn2")


def _read_mlp(raw, where: str) -> Optional[PlainMlpConfig]:
    if raw is None:
        return None
    if not isinstance(raw, dict):
        raise ConfigError(f"config.json: {where}: 'mlp' must be an object or null")
    kind = read_key(raw, "kind", kind=str)
    if kind != "dense":
        raise ConfigError(f"config.json: {where}: mlp.kind {kind!r} is not supported (dense)")
    c = PlainMlpConfig(read_key(raw, "ff", kind=int))
    if c.ff < 1:
        raise ConfigError(f"config.json: {where}: mlp.ff must be positive")
    return c


@dataclass
class KelutarConfig:
    width: int
    vocab: int
    max_positions: int
    norm_eps: float
    embedding_scale: float
    taps: int                    # of the convolution in front of every mixer; 0: none
    layers: List[KelutarLayer]
    architecture: str = "Kelutar"
    dtype: str = "bfloat16"
    path: str = ""
    raw: Dict[str, Any] = field(default_factory=dict, repr=False, compare=False)

    @property
    def vocab_size(self) -> int:
        return self.vocab

    @property
    def hidden_size(self) -> int:
        return self.width

    @property
    def num_layers(self) -> int:
        return len(self.layers)

    @classmethod
    def from_hf(cls, cfg: Dict[str, Any], path: str = "") -> "KelutarConfig":
        norm, embedding = _section(cfg, "norm", "model"), _section(cfg, "embedding", "model")
        canon = _section(cfg, "canon", "model", required=False)
        entries = cfg.get("layers")
        if not isinstance(entries, list) or not entries:
            raise ConfigError("config.json: 'layers' must be a non-empty list")
        layers = []
        for i in range(len(entries)):
            where = f"layers[{i}]"
            owner, entry = weights_owner(entries, i)
            kind = read_key(entry, "type", kind=str)
            layers.append(KelutarLayer(kind, _read_mixer(kind, _section(entry, "mixer", where), where),
                                       _read_mlp(entry.get("mlp"), where), owner))
        out = cls(width=read_key(cfg, "width", kind=int), vocab=read_key(cfg, "vocab", kind=int),
                  max_positions=read_key(cfg, "max_positions", kind=int), norm_eps=read_key(norm, "eps", kind=float),
                  embedding_scale=read_key(embedding, "scale", kind=float),
                  taps=read_key(canon, "taps", kind=int) if canon is not None else 0, layers=layers,
                  architecture=str(cfg.get("architecture") or "Kelutar"),
                  dtype=str(cfg.get("torch_dtype") or "bfloat16"), path=path, raw=dict(cfg))
        out.validate()
        return out

    def validate(self) -> None:
        if min(self.width, self.vocab, self.max_positions) < 1 or not self.norm_eps > 0:
            raise ConfigError("config.json: width, vocab and max_positions must be positive, norm.eps > 0")
        if not 0 <= self.taps <= 64:
            raise ConfigError("config.json: canon.taps must be in 0..64")
        for i, l in enumerate(self.layers):
            if l.weights_of is not None:
                o = self.layers[l.weights_of]
                if (o.kind, o.mixer, o.mlp) != (l.kind, l.mixer, l.mlp):
                    raise ConfigError(f"config.json: layers[{i}] uses the tensors of layer {l.weights_of} but "
                                      "describes another layer")

    def to_hf(self) -> Dict[str, Any]:
        layers = []
        for l in self.layers:
            m = l.mixer
            if l.kind == "attention":
                mixer = {"heads": m.heads, "kv_heads": m.kv_heads, "dim": m.dim, "vdim": m.dim, "scale": m.scale}
                if m.window:
                    mixer["mask"] = {"size": m.window}
            else:
                mixer = {"heads": m.heads, "dim": m.dim, "vdim": m.vdim}
            entry = {"type": l.kind, "mixer": mixer, "mlp": {"kind": "dense", "ff": l.mlp.ff} if l.mlp else None}
            if l.weights_of is not None:
                entry["weights_of"] = l.weights_of
            layers.append(entry)
        out = {"architecture": self.architecture, "width": self.width, "vocab": self.vocab,
               "max_positions": self.max_positions, "norm": {"eps": self.norm_eps},
               "embedding": {"scale": self.embedding_scale}, "layers": layers, "torch_dtype": self.dtype}
        if self.taps:
            out["canon"] = {"taps": self.taps}
        return out
