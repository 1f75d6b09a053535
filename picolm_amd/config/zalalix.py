"""Typed configuration of the Zalalix decoder, read from the keys of its config.json.

    architecture        "Zalalix"
    vocab, width        sizes of the embedding table and of the head
    embedding.scale     the embedding's rows are multiplied by it
    norm.eps            eps of every RMS norm
    layers[i]           {"type": "lightning" | "retention" | "parallel", "mixer": {...}, "mlp": {"kind": "dense", "ff": F} | null}
        lightning       mixer {heads, dim, vdim, decay: [one per head]}
        retention       mixer {heads, dim, vdim, decay: [one per head]}
        parallel        mixer {left, left_scale, right, right_scale}
            left        {heads, kv_heads, dim, vdim, scale, softcap, mask: {size, keep_first},
                         rot: {base, dims, scaling: {factor, low, high, original} | absent}}
            right       {heads, dim, vdim, tau}

The rows of the right mixer's first decay matrix are a tensor's shape, not a key; a configuration
that is written out for random weights names them in `rank`, which a reader takes if it is there.
Every size the model uses comes from an instance of `ZalalixConfig` or from a tensor's shape.
"""
from __future__ import annotations

from dataclasses import dataclass, field

from .begopel import MAX_HEAD_DIM, MAX_STATE_KEY_DIM, _integer, _number, _object
from .llama import ConfigError, RopeScaling

MIXER_TYPES = ("lightning", "retention", "parallel")


def _optional_object(d: dict, where: str, key: str):
    v = d.get(key)
    if v is not None and not isinstance(v, dict):
        raise ConfigError(f"{where}{key}: expected an object or null")
    return v


@dataclass(frozen=True)
class RotationConfig:
    base: float
    dims: int
    scaling: RopeScaling | None = None       # wavelength-dependent slowing-down of the frequencies

    @staticmethod
    def from_dict(d: dict, where: str) -> "RotationConfig":
        s = _optional_object(d, where, "scaling")
        scaling = None
        if s:
            w = where + "scaling."
            scaling = RopeScaling("llama3", _number(s, w, "factor"), _number(s, w, "low"), _number(s, w, "high"), _number(s, w, "original"))
            for key, v in (("factor", scaling.factor), ("low", scaling.low_freq_factor), ("original", scaling.original_max_position_embeddings)):
                if not v > 0:
                    raise ConfigError(f"{w}{key}: must be positive")
            if scaling.high_freq_factor < scaling.low_freq_factor:
                raise ConfigError(f"{w}high: {scaling.high_freq_factor} is below low = {scaling.low_freq_factor}")
        c = RotationConfig(_number(d, where, "base"), _integer(d, where, "dims"), scaling)
        if c.dims % 2:
            raise ConfigError(f"{where}dims: {c.dims} is odd, the rotation pairs entries")
        if not c.base > 0:
            raise ConfigError(f"{where}base: must be positive")
        return c

    def to_dict(self) -> dict:
        d = {"base": self.base, "dims": self.dims}
        if self.scaling is not None:
            s = self.scaling
            d["scaling"] = {"factor": s.factor, "low": s.low_freq_factor, "high": s.high_freq_factor,
                            "original": s.original_max_position_embeddings}
        return d


@dataclass(frozen=True)
class WindowedAttentionConfig:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    softcap: float = 0.0             # 0: none
    window: int = 0                  # 0: every key is seen
    keep_first: int = 0
    rot: RotationConfig | None = None

    @staticmethod
    def from_dict(d: dict, where: str) -> "WindowedAttentionConfig":
        heads, dim = _integer(d, where, "heads"), _integer(d, where, "dim")
        mask, rot = _optional_object(d, where, "mask"), _optional_object(d, where, "rot")
        c = WindowedAttentionConfig(
            heads, _integer(d, where, "kv_heads", heads), dim, _integer(d, where, "vdim", dim), _number(d, where, "scale", dim ** -0.5),
            _number(d, where, "softcap", 0.0) if d.get("softcap") is not None else 0.0,
            _integer(mask, where + "mask.", "size") if mask else 0,
            _integer(mask, where + "mask.", "keep_first", 0, least=0) if mask else 0,
            RotationConfig.from_dict(rot, where + "rot.") if rot else None)
        if c.heads % c.kv_heads:
            raise ConfigError(f"{where}kv_heads: {c.kv_heads} does not divide heads = {c.heads}")
        for key in ("dim", "vdim"):
            if getattr(c, key) > MAX_HEAD_DIM:
                raise ConfigError(f"{where}{key}: {getattr(c, key)} exceeds {MAX_HEAD_DIM}, the largest head the attention kernels take")
        if not c.scale > 0:
            raise ConfigError(f"{where}scale: must be positive")
        if c.softcap < 0:
            raise ConfigError(f"{where}softcap: must be positive")
        if rot and c.rot.dims > c.dim:
            raise ConfigError(f"{where}rot.dims: {c.rot.dims} entries of a head of {c.dim}")
        return c

    def to_dict(self) -> dict:
        d = {"heads": self.heads, "kv_heads": self.kv_heads, "dim": self.dim, "vdim": self.vdim, "scale": self.scale}
        if self.softcap:
            d["softcap"] = self.softcap
        if self.window:
            d["mask"] = {"size": self.window, "keep_first": self.keep_first}
        if self.rot is not None:
            d["rot"] = self.rot.to_dict()
        return d


@dataclass(frozen=True)
class LinearAttentionConfig:
    """A mixer with a matrix state per head: with fixed decays, or with decays of the token's own."""
    heads: int
    dim: int
    vdim: int
    decay: tuple | None = None
    tau: float | None = None
    rank: int | None = None          # rows of the first decay matrix; None: the tensor's shape says

    @staticmethod
    def from_dict(d: dict, where: str, fixed: bool) -> "LinearAttentionConfig":
        heads, dim = _integer(d, where, "heads"), _integer(d, where, "dim")
        vdim = _integer(d, where, "vdim", dim)
        if dim > MAX_STATE_KEY_DIM:
            raise ConfigError(f"{where}dim: {dim} exceeds {MAX_STATE_KEY_DIM}, the largest key of a matrix state")
        if not fixed:
            tau = _number(d, where, "tau")
            if not tau > 0:
                raise ConfigError(f"{where}tau: must be positive")
            return LinearAttentionConfig(heads, dim, vdim, None, tau, _integer(d, where, "rank") if d.get("rank") is not None else None)
        decay = d.get("decay")
        if not isinstance(decay, (list, tuple)) or any(isinstance(x, bool) or not isinstance(x, (int, float)) for x in decay):
            raise ConfigError(f"{where}decay: expected a list of numbers")
        if len(decay) != heads:
            raise ConfigError(f"{where}decay: {len(decay)} decays for {heads} heads")
        if not all(0.0 <= x <= 1.0 for x in decay):
            raise ConfigError(f"{where}decay: a decay lies between 0 and 1")
        return LinearAttentionConfig(heads, dim, vdim, tuple(float(x) for x in decay))

    def to_dict(self) -> dict:
        d = {"heads": self.heads, "dim": self.dim, "vdim": self.vdim}
        if self.decay is not None:
            d["decay"] = list(self.decay)
        else:
            d["tau"] = self.tau
        if self.rank is not None:
            d["rank"] = self.rank
        return d


@dataclass(frozen=True)
class ParallelMixerConfig:
    left: WindowedAttentionConfig
    left_scale: float
    right: LinearAttentionConfig
    right_scale: float

    @staticmethod
    def from_dict(d: dict, where: str) -> "ParallelMixerConfig":
        return ParallelMixerConfig(WindowedAttentionConfig.from_dict(_object(d, where, "left"), where + "left."),
                                   _number(d, where, "left_scale", 1.0),
                                   LinearAttentionConfig.from_dict(_object(d, where, "right"), where + "right.", fixed=False),
                                   _number(d, where, "right_scale", 1.0))

    def to_dict(self) -> dict:
        return {"left": self.left.to_dict(), "left_scale": self.left_scale, "right": self.right.to_dict(), "right_scale": self.right_scale}


@dataclass(frozen=True)
class ZalalixLayer:
    kind: str                        # one of MIXER_TYPES
    mixer: object                    # LinearAttentionConfig, or ParallelMixerConfig
    ff: int | None                   # inner width of the dense feed-forward; None: the layer has none

    @staticmethod
    def from_dict(d: dict, where: str) -> "ZalalixLayer":
        if not isinstance(d, dict):
            raise ConfigError(f"{where[:-1]}: expected an object")
        kind = d.get("type")
        if kind not in MIXER_TYPES:
            raise ConfigError(f"{where}type: '{kind}' is not a known mixer (known: {', '.join(MIXER_TYPES)})")
        m, w = _object(d, where, "mixer"), where + "mixer."
        mixer = ParallelMixerConfig.from_dict(m, w) if kind == "parallel" else LinearAttentionConfig.from_dict(m, w, fixed=True)
        mlp = _optional_object(d, where, "mlp")
        if mlp is not None and mlp.get("kind") != "dense":
            raise ConfigError(f"{where}mlp.kind: '{mlp.get('kind')}' is not supported (known: dense)")
        return ZalalixLayer(kind, mixer, _integer(mlp, where + "mlp.", "ff") if mlp is not None else None)

    def to_dict(self) -> dict:
        return {"type": self.kind, "mixer": self.mixer.to_dict(), "mlp": None if self.ff is None else {"kind": "dense", "ff": self.ff}}


@dataclass(frozen=True)
class ZalalixConfig:
    vocab: int
    width: int
    layers: tuple
    embedding_scale: float = 1.0
    norm_eps: float = 1e-6
    torch_dtype: str = "bfloat16"
    max_position_embeddings: int | None = None       # rotary tables are laid out for what the cache holds
    bos_token_id: int | None = None
    eos_token_ids: tuple = field(default=())

    @staticmethod
    def from_dict(root: dict) -> "ZalalixConfig":
        if not isinstance(root, dict):
            raise ConfigError("config.json: expected an object")
        layers = root.get("layers")
        if not isinstance(layers, (list, tuple)) or not layers:
            raise ConfigError("layers: expected a list of at least one layer")
        eos = root.get("eos_token_id")
        cfg = ZalalixConfig(
            vocab=_integer(root, "", "vocab"), width=_integer(root, "", "width"),
            layers=tuple(ZalalixLayer.from_dict(l, f"layers[{i}].") for i, l in enumerate(layers)),
            embedding_scale=_number(_optional_object(root, "", "embedding") or {}, "embedding.", "scale", 1.0),
            norm_eps=_number(_optional_object(root, "", "norm") or {}, "norm.", "eps", 1e-6),
            torch_dtype=str(root.get("torch_dtype", "bfloat16")),
            max_position_embeddings=(_integer(root, "", "max_position_embeddings")
                                     if root.get("max_position_embeddings") is not None else None),
            bos_token_id=None if root.get("bos_token_id") is None else int(root["bos_token_id"]),
            eos_token_ids=() if eos is None else tuple(int(e) for e in (eos if isinstance(eos, (list, tuple)) else [eos])))
        cfg.validate()
        return cfg

    def validate(self) -> None:
        if not self.norm_eps > 0:
            raise ConfigError("norm.eps: must be positive")
        if self.torch_dtype not in ("bfloat16", "float32", "float16"):
            raise ConfigError(f"torch_dtype: '{self.torch_dtype}' is not one of bfloat16, float32, float16")
        for e in self.eos_token_ids:
            if not 0 <= e < self.vocab:
                raise ConfigError(f"eos_token_id: {e} is outside the vocabulary of {self.vocab}")

    def to_dict(self) -> dict:
        d = {"architecture": "Zalalix", "vocab": self.vocab, "width": self.width, "embedding": {"scale": self.embedding_scale},
             "norm": {"eps": self.norm_eps}, "layers": [l.to_dict() for l in self.layers], "torch_dtype": self.torch_dtype}
        if self.max_position_embeddings is not None:
            d["max_position_embeddings"] = self.max_position_embeddings
        if self.bos_token_id is not None:
            d["bos_token_id"] = self.bos_token_id
        if self.eos_token_ids:
            d["eos_token_id"] = list(self.eos_token_ids)
        return d

    # -- derived ---------------------------------------------------------------------------
    @property
    def vocab_size(self) -> int:
        return self.vocab

    @property
    def hidden_size(self) -> int:
        return self.width
