"""Typed configuration of the Belorax decoder, read from the keys of its config.json.

    architecture        "Belorax"
    vocab, width        sizes of the embedding table and of the head
    embedding.scale     the embedding's rows are multiplied by it
    residual_mult       what a sublayer adds to the residual rows is multiplied by it, behind its norm
    norm.eps            eps of every RMS norm
    layers[i]           {"type": "retention" | "attention" | "latent_attention", "mixer": {...}, "mlp": {...} | null}
        retention       mixer {heads, dim, vdim, decay: [one per head], rot: {base, dims}}
        attention       mixer {heads, kv_heads, dim, vdim, scale, q_temp: {coef, every}, kv_from: j}     kv_from: the layer
                        reads layer j's keys and values instead of making its own
        latent_attention  mixer {heads, dim, rot_dim, vdim, kv_rank, scale, rot: {base, dims, scaling: {factor, original,
                        fast, slow} | null}}
        mlp             {"kind": "dense", "ff"} or {"kind": "moe", "router": {experts, top}, "expert": {ff}}

Every size the model uses comes from an instance of `BeloraxConfig`.
"""
from __future__ import annotations

from dataclasses import dataclass, field

from .begopel import MAX_HEAD_DIM, MAX_STATE_KEY_DIM, _integer, _number, _object
from .llama import ConfigError
from .satedra import YarnScaling
from .zalalix import _optional_object

MIXER_TYPES = ("retention", "attention", "latent_attention")


@dataclass(frozen=True)
class RotationConfig:
    base: float
    dims: int
    scaling: YarnScaling | None = None

    @staticmethod
    def from_dict(d: dict, where: str) -> "RotationConfig":
        scaling = _optional_object(d, where, "scaling")
        c = RotationConfig(_number(d, where, "base"), _integer(d, where, "dims"),
                           YarnScaling.from_dict(scaling, where + "scaling.") if scaling else None)
        if c.dims % 2:
            raise ConfigError(f"{where}dims: {c.dims} is odd, the rotation pairs entries")
        if not c.base > 0:
            raise ConfigError(f"{where}base: must be positive")
        if c.scaling is not None and c.base == 1.0:
            raise ConfigError(f"{where}base: a base of one has no wavelengths to scale")
        return c

    def to_dict(self) -> dict:
        d = {"base": self.base, "dims": self.dims}
        if self.scaling is not None:
            d["scaling"] = self.scaling.to_dict()
        return d


@dataclass(frozen=True)
class RetentionConfig:
    heads: int
    dim: int
    vdim: int
    decay: tuple
    rot: RotationConfig | None = None

    kv_from = None

    @staticmethod
    def from_dict(d: dict, where: str) -> "RetentionConfig":
        heads, dim, rot = _integer(d, where, "heads"), _integer(d, where, "dim"), _optional_object(d, where, "rot")
        if dim > MAX_STATE_KEY_DIM:
            raise ConfigError(f"{where}dim: {dim} exceeds {MAX_STATE_KEY_DIM}, the largest key of a matrix state")
        decay = d.get("decay")
        if not isinstance(decay, (list, tuple)) or any(isinstance(x, bool) or not isinstance(x, (int, float)) for x in decay):
            raise ConfigError(f"{where}decay: expected a list of numbers")
        if len(decay) != heads:
            raise ConfigError(f"{where}decay: {len(decay)} decays for {heads} heads")
        if not all(0.0 <= x <= 1.0 for x in decay):
            raise ConfigError(f"{where}decay: a decay lies between 0 and 1")
        c = RetentionConfig(heads, dim, _integer(d, where, "vdim", dim), tuple(float(x) for x in decay),
                            RotationConfig.from_dict(rot, where + "rot.") if rot else None)
        if c.rot is not None and c.rot.dims > dim:
            raise ConfigError(f"{where}rot.dims: {c.rot.dims} entries of a head of {dim}")
        return c

    def to_dict(self) -> dict:
        d = {"heads": self.heads, "dim": self.dim, "vdim": self.vdim, "decay": list(self.decay)}
        if self.rot is not None:
            d["rot"] = self.rot.to_dict()
        return d


@dataclass(frozen=True)
class AttentionConfig:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    q_temp: tuple | None = None      # (coef, every)
    kv_from: int | None = None

    @staticmethod
    def from_dict(d: dict, where: str) -> "AttentionConfig":
        heads, dim, temp = _integer(d, where, "heads"), _integer(d, where, "dim"), _optional_object(d, where, "q_temp")
        c = AttentionConfig(heads, _integer(d, where, "kv_heads", heads), dim, _integer(d, where, "vdim", dim),
                            _number(d, where, "scale", dim ** -0.5),
                            (_number(temp, where + "q_temp.", "coef"), _number(temp, where + "q_temp.", "every")) if temp else None,
                            None if d.get("kv_from") is None else _integer(d, where, "kv_from", least=0))
        if c.heads % c.kv_heads:
            raise ConfigError(f"{where}kv_heads: {c.kv_heads} does not divide heads = {c.heads}")
        for key in ("dim", "vdim"):
            if getattr(c, key) > MAX_HEAD_DIM:
                raise ConfigError(f"{where}{key}: {getattr(c, key)} exceeds {MAX_HEAD_DIM}, the largest head the attention kernels take")
        if not c.scale > 0:
            raise ConfigError(f"{where}scale: must be positive")
        if temp and not c.q_temp[1] > 0:
            raise ConfigError(f"{where}q_temp.every: must be positive")
        return c

    def to_dict(self) -> dict:
        d = {"heads": self.heads, "kv_heads": self.kv_heads, "dim": self.dim, "vdim": self.vdim, "scale": self.scale}
        if self.q_temp is not None:
            d["q_temp"] = {"coef": self.q_temp[0], "every": self.q_temp[1]}
        if self.kv_from is not None:
            d["kv_from"] = self.kv_from
        return d

    def cached_like(self, other) -> bool:
        """Whether what this layer reads is what `other` caches."""
        return isinstance(other, AttentionConfig) and (self.kv_heads, self.dim, self.vdim) == (other.kv_heads, other.dim, other.vdim)


@dataclass(frozen=True)
class LatentConfig:
    heads: int
    dim: int                         # unrotated query/key entries a head
    rot_dim: int                     # rotated ones; the rotated key part is shared by the heads
    vdim: int
    kv_rank: int
    scale: float
    rot: RotationConfig

    kv_from = None

    @staticmethod
    def from_dict(d: dict, where: str) -> "LatentConfig":
        c = LatentConfig(_integer(d, where, "heads"), _integer(d, where, "dim"), _integer(d, where, "rot_dim"), _integer(d, where, "vdim"),
                         _integer(d, where, "kv_rank"), _number(d, where, "scale"),
                         RotationConfig.from_dict(_object(d, where, "rot"), where + "rot."))
        if c.rot.dims != c.rot_dim:
            raise ConfigError(f"{where}rot.dims: {c.rot.dims} is not rot_dim = {c.rot_dim}, the part of a head that is rotated")
        if not c.scale > 0:
            raise ConfigError(f"{where}scale: must be positive")
        if c.kv_rank + c.rot_dim > MAX_HEAD_DIM:        # the attention runs over [latent | rotated part]: that is its key
            raise ConfigError(f"{where}kv_rank: {c.kv_rank} + rot_dim = {c.rot_dim} exceed {MAX_HEAD_DIM}, the largest key the "
                              "attention kernels take")
        return c

    def to_dict(self) -> dict:
        return {"heads": self.heads, "dim": self.dim, "rot_dim": self.rot_dim, "vdim": self.vdim, "kv_rank": self.kv_rank,
                "scale": self.scale, "rot": self.rot.to_dict()}


_MIXERS = {"retention": RetentionConfig, "attention": AttentionConfig, "latent_attention": LatentConfig}


@dataclass(frozen=True)
class BeloraxMLP:
    kind: str                        # "dense" | "moe"
    ff: int                          # inner width of the dense layer, or of one expert
    experts: int = 0
    top: int = 0

    @staticmethod
    def from_dict(d: dict, where: str) -> "BeloraxMLP":
        kind = d.get("kind")
        if kind == "dense":
            return BeloraxMLP("dense", _integer(d, where, "ff"))
        if kind != "moe":
            raise ConfigError(f"{where}kind: '{kind}' is not supported (known: dense, moe)")
        router = _object(d, where, "router")
        c = BeloraxMLP("moe", _integer(_object(d, where, "expert"), where + "expert.", "ff"), _integer(router, where + "router.", "experts"),
                       _integer(router, where + "router.", "top"))
        if c.top > c.experts:
            raise ConfigError(f"{where}router.top: {c.top} exceeds the {c.experts} experts")
        return c

    def to_dict(self) -> dict:
        if self.kind == "dense":
            return {"kind": "dense", "ff": self.ff}
        return {"kind": "moe", "router": {"experts": self.experts, "top": self.top}, "expert": {"ff": self.ff}}


@dataclass(frozen=True)
class BeloraxLayer:
    kind: str                        # one of MIXER_TYPES
    mixer: object                    # RetentionConfig, AttentionConfig or LatentConfig
    mlp: BeloraxMLP | None           # None: the layer has no feed-forward

    @staticmethod
    def from_dict(d: dict, where: str) -> "BeloraxLayer":
        if not isinstance(d, dict):
            raise ConfigError(f"{where[:-1]}: expected an object")
        kind = d.get("type")
        if kind not in MIXER_TYPES:
            raise ConfigError(f"{where}type: '{kind}' is not a known mixer (known: {', '.join(MIXER_TYPES)})")
        mlp = _optional_object(d, where, "mlp")
        return BeloraxLayer(kind, _MIXERS[kind].from_dict(_object(d, where, "mixer"), where + "mixer."),
                            BeloraxMLP.from_dict(mlp, where + "mlp.") if mlp is not None else None)

    def to_dict(self) -> dict:
        return {"type": self.kind, "mixer": self.mixer.to_dict(), "mlp": self.mlp.to_dict() if self.mlp is not None else None}


@dataclass(frozen=True)
class BeloraxConfig:
    vocab: int
    width: int
    layers: tuple
    embedding_scale: float = 1.0
    residual_mult: float = 1.0
    norm_eps: float = 1e-6
    torch_dtype: str = "bfloat16"
    max_position_embeddings: int | None = None       # rotary tables are laid out for what the cache holds
    bos_token_id: int | None = None
    eos_token_ids: tuple = field(default=())

    @staticmethod
    def from_dict(root: dict) -> "BeloraxConfig":
        if not isinstance(root, dict):
            raise ConfigError("config.json: expected an object")
        layers = root.get("layers")
        if not isinstance(layers, (list, tuple)) or not layers:
            raise ConfigError("layers: expected a list of at least one layer")
        eos = root.get("eos_token_id")
        cfg = BeloraxConfig(
            vocab=_integer(root, "", "vocab"), width=_integer(root, "", "width"),
            layers=tuple(BeloraxLayer.from_dict(l, f"layers[{i}].") for i, l in enumerate(layers)),
            embedding_scale=_number(_optional_object(root, "", "embedding") or {}, "embedding.", "scale", 1.0),
            residual_mult=_number(root, "", "residual_mult", 1.0),
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
        if self.residual_mult == 0:
            raise ConfigError("residual_mult: nought leaves the layers without effect")
        if self.torch_dtype not in ("bfloat16", "float32", "float16"):
            raise ConfigError(f"torch_dtype: '{self.torch_dtype}' is not one of bfloat16, float32, float16")
        for e in self.eos_token_ids:
            if not 0 <= e < self.vocab:
                raise ConfigError(f"eos_token_id: {e} is outside the vocabulary of {self.vocab}")
        for i, layer in enumerate(self.layers):
            j = layer.mixer.kv_from
            if j is None:
                continue
            where = f"layers[{i}].mixer.kv_from: "
            if j >= i:
                raise ConfigError(f"{where}{j} is not an earlier layer")
            if self.layers[j].mixer.kv_from is not None:
                raise ConfigError(f"{where}layer {j} has no keys of its own")
            if not layer.mixer.cached_like(self.layers[j].mixer):
                raise ConfigError(f"{where}layer {j} does not keep the keys and values that this layer reads")

    def to_dict(self) -> dict:
        d = {"architecture": "Belorax", "vocab": self.vocab, "width": self.width, "embedding": {"scale": self.embedding_scale},
             "residual_mult": self.residual_mult, "norm": {"eps": self.norm_eps}, "layers": [l.to_dict() for l in self.layers],
             "torch_dtype": self.torch_dtype}
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
