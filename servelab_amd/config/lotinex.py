"""Configuration of the Lotinex design: a decoder whose residual stream is kept in several copies and
whose config.json lists its layers, each with one of three mixers and a dense or routed feed-forward.

    {"architecture": "Lotinex", "width", "vocab", "streams", "norm": {"eps"}, "embedding": {"scale"},
     "layers": [{"type", "mixer": {...}, "mlp": {...} | null}]}

Mixers (``rot`` = {base, dims[, scaling: {factor, original, fast, slow}]}: the leading ``dims``
channels of a head turn in halves; absent: none turn):
  ``attention``  heads, kv_heads, dim, vdim, scale, rot, mask {size} (chunks of so many positions;
                 absent: every earlier key), kv_from (an earlier attention whose keys and values are
                 read; absent: own ones)
  ``delta``      heads, kv_heads, dim, vdim, conv
  ``parallel``   left: heads, kv_heads, dim, vdim, scale, softcap (absent: scores are not capped), conv
                 (absent: none), rot, mask {size} (a window; absent: every earlier key); right: inner,
                 state, dt_rank, conv
Feed-forward: ``{"kind": "dense", "ff"}`` or ``{"kind": "moe", "router": {"experts", "top"},
"expert": {"ff"}}``.  Nothing here is a default for a size or a constant of the model.
"""
from dataclasses import dataclass, field
from typing import Any, Dict, List, Optional

from .layered import _section
from .model import ConfigError, read_key
from .vunadra import RotationConfig, _rotation, _window


@dataclass(frozen=True)
class SoftmaxAttentionConfig:
    """``attention`` (``reach``: the size of its chunks) and the left side of ``parallel`` (``reach``: its
    window); reach 0: every earlier key."""
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    rot: RotationConfig
    reach: int = 0
    softcap: float = 0.0         # 0: scores are not capped
    conv: int = 0                # taps; 0: no convolution
    kv_from: Optional[int] = None


@dataclass(frozen=True)
class HeadDeltaConfig:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    conv: int


@dataclass(frozen=True)
class SelectiveConfig:
    inner: int
    state: int
    dt_rank: int
    conv: int


@dataclass(frozen=True)
class SidesConfig:
    left: SoftmaxAttentionConfig
    right: SelectiveConfig


@dataclass(frozen=True)
class DenseGatedConfig:
    ff: int


@dataclass(frozen=True)
class SigmoidExpertsConfig:
    experts: int
    top: int
    ff: int


@dataclass(frozen=True)
class LotinexLayer:
    kind: str                    # "attention" | "delta" | "parallel"
    mixer: Any
    mlp: Any                     # DenseGatedConfig | SigmoidExpertsConfig | None


def _read_softmax(m: Dict[str, Any], where: str, left: bool) -> SoftmaxAttentionConfig:
    kv_from = None if left or m.get("kv_from") is None else read_key(m, "kv_from", kind=int)
    c = SoftmaxAttentionConfig(
        heads=read_key(m, "heads", kind=int), kv_heads=read_key(m, "kv_heads", kind=int),
        dim=read_key(m, "dim", kind=int), vdim=read_key(m, "vdim", kind=int), scale=read_key(m, "scale", kind=float),
        rot=_rotation(m, where), reach=_window(m, where),
        softcap=(read_key(m, "softcap", 0.0, kind=float) or 0.0) if left else 0.0,
        conv=(read_key(m, "conv", 0, kind=int) or 0) if left else 0, kv_from=kv_from)
    if c.rot.scaling is not None and c.rot.scaling[0] != "blended":
        raise ConfigError(f"config.json: {where}: rot.scaling needs factor, original, fast and slow")
    if min(c.heads, c.kv_heads, c.dim, c.vdim) < 1 or c.heads % c.kv_heads or c.rot.dims > c.dim \
            or c.conv < 0 or c.softcap < 0:
        raise ConfigError(f"config.json: {where}: heads must be a positive multiple of kv_heads, dim and vdim "
                          "positive, rot.dims within dim, conv and softcap not negative")
    return c


def _read_mixer(kind: str, m: Dict[str, Any], where: str):
    if kind == "attention":
        return _read_softmax(m, where, left=False)
    if kind == "delta":
        c = HeadDeltaConfig(*(read_key(m, k, kind=int) for k in ("heads", "kv_heads", "dim", "vdim", "conv")))
        if min(c.heads, c.kv_heads, c.dim, c.vdim, c.conv) < 1 or c.heads % c.kv_heads:
            raise ConfigError(f"config.json: {where}: heads must be a positive multiple of kv_heads, dim, vdim and "
                              "conv positive")
        return c
    if kind == "parallel":
        left, right = _section(m, "left", where), _section(m, "right", where)
        r = SelectiveConfig(*(read_key(right, k, kind=int) for k in ("inner", "state", "dt_rank", "conv")))
        if min(r.inner, r.state, r.dt_rank, r.conv) < 1:
            raise ConfigError(f"config.json: {where}.right: inner, state, dt_rank and conv must be positive")
        return SidesConfig(_read_softmax(left, where + ".left", left=True), r)
    raise ConfigError(f"config.json: {where}: type {kind!r} is not one of attention, delta, parallel")


def _read_mlp(raw: Optional[Dict[str, Any]], where: str):
    if raw is None:
        return None
    kind = read_key(raw, "kind", kind=str)
    if kind == "dense":
        c = DenseGatedConfig(read_key(raw, "ff", kind=int))
        if c.ff < 1:
            raise ConfigError(f"config.json: {where}: mlp.ff must be positive")
        return c
    if kind == "moe":
        router, expert = _section(raw, "router", where), _section(raw, "expert", where)
        c = SigmoidExpertsConfig(read_key(router, "experts", kind=int), read_key(router, "top", kind=int),
                                 read_key(expert, "ff", kind=int))
        if c.ff < 1 or not 1 <= c.top <= c.experts:
            raise ConfigError(f"config.json: {where}: mlp needs 1 <= router.top <= router.experts and a positive width")
        return c
    raise ConfigError(f"config.json: {where}: mlp.kind {kind!r} is not one of dense, moe")


def _read_layer(i: int, entry: Dict[str, Any]) -> LotinexLayer:
    where = f"layers[{i}]"
    if not isinstance(entry, dict):
        raise ConfigError(f"config.json: {where} must be an object")
    kind = read_key(entry, "type", kind=str)
    mixer = _read_mixer(kind, _section(entry, "mixer", where), where)
    return LotinexLayer(kind, mixer, _read_mlp(_section(entry, "mlp", where, required=False), where))


@dataclass
class LotinexConfig:
    width: int
    vocab: int
    streams: int
    norm_eps: float
    embedding_scale: float
    layers: List[LotinexLayer]
    architecture: str = "Lotinex"
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
    def from_hf(cls, cfg: Dict[str, Any], path: str = "") -> "LotinexConfig":
        norm = _section(cfg, "norm", "model")
        embedding = _section(cfg, "embedding", "model")
        layers = cfg.get("layers")
        if not isinstance(layers, list) or not layers:
            raise ConfigError("config.json: 'layers' must be a non-empty list")
        out = cls(width=read_key(cfg, "width", kind=int), vocab=read_key(cfg, "vocab", kind=int),
                  streams=read_key(cfg, "streams", kind=int), norm_eps=read_key(norm, "eps", kind=float),
                  embedding_scale=read_key(embedding, "scale", kind=float),
                  layers=[_read_layer(i, e) for i, e in enumerate(layers)],
                  architecture=str(cfg.get("architecture") or "Lotinex"),
                  dtype=str(cfg.get("torch_dtype") or "bfloat16"), path=path, raw=dict(cfg))
        out.validate()
        return out

    def validate(self) -> None:
        if self.width < 1 or self.vocab < 1 or not self.norm_eps > 0:
            raise ConfigError("config.json: width and vocab must be positive, norm.eps > 0")
        if not 1 <= self.streams <= 16:
            raise ConfigError("config.json: streams must be between 1 and 16")
        for i, l in enumerate(self.layers):
            if l.kind != "attention" or l.mixer.kv_from is None:
                continue
            j, m = l.mixer.kv_from, l.mixer
            owner = self.layers[j].mixer if 0 <= j < i and self.layers[j].kind == "attention" else None
            if owner is None or owner.kv_from is not None:
                raise ConfigError(f"config.json: layers[{i}]: kv_from must name an earlier attention layer with keys "
                                  "and values of its own")
            if (owner.kv_heads, owner.dim, owner.vdim, owner.rot) != (m.kv_heads, m.dim, m.vdim, m.rot):
                raise ConfigError(f"config.json: layers[{i}]: kv_heads, dim, vdim and rot must be those of layer {j}, "
                                  "whose keys and values it reads")

    def to_hf(self) -> Dict[str, Any]:
        def softmax(m):
            out = {"heads": m.heads, "kv_heads": m.kv_heads, "dim": m.dim, "vdim": m.vdim, "scale": m.scale}
            if m.rot.dims:
                out["rot"] = m.rot.to_hf()
            if m.reach:
                out["mask"] = {"size": m.reach}
            for key, value in (("softcap", m.softcap), ("conv", m.conv)):
                if value:
                    out[key] = value
            if m.kv_from is not None:
                out["kv_from"] = m.kv_from
            return out
        layers = []
        for l in self.layers:
            m = l.mixer
            if l.kind == "attention":
                mixer = softmax(m)
            elif l.kind == "delta":
                mixer = {"heads": m.heads, "kv_heads": m.kv_heads, "dim": m.dim, "vdim": m.vdim, "conv": m.conv}
            else:
                r = m.right
                mixer = {"left": softmax(m.left),
                         "right": {"inner": r.inner, "state": r.state, "dt_rank": r.dt_rank, "conv": r.conv}}
            if l.mlp is None:
                mlp = None
            elif isinstance(l.mlp, DenseGatedConfig):
                mlp = {"kind": "dense", "ff": l.mlp.ff}
            else:
                mlp = {"kind": "moe", "router": {"experts": l.mlp.experts, "top": l.mlp.top},
                       "expert": {"ff": l.mlp.ff}}
            layers.append({"type": l.kind, "mixer": mixer, "mlp": mlp})
        return {"architecture": self.architecture, "width": self.width, "vocab": self.vocab, "streams": self.streams,
                "norm": {"eps": self.norm_eps}, "embedding": {"scale": self.embedding_scale}, "layers": layers,
                "torch_dtype": self.dtype}
