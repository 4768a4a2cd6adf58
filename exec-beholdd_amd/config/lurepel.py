"""Lurepel: the typed configuration read from config.json.

A config.json of this design lists its layers one by one, each with the kind of its mixer ("attention": grouped softmax
attention within chunks of positions whose values are its keys), the mixer's sizes and constants, and its feed-forward
("dense", "moe" or none).  Every layer norms what its sublayers give: x <- x + norm(sublayer(x)).  Every size and constant
comes from the file; a key that a formula needs and the file does not give is an error.  A block that the file does not have
stands for a mechanism the model does not have (no `mask`: every earlier key is seen; no `rot`: no rotation; no `scaling`:
the rotation's plain frequencies; no `identity`: no expert that hands its input through).  The file gives no longest
position: a sequence may be as long as the cache it runs in.
"""

from __future__ import annotations

from dataclasses import dataclass

from .base import ConfigError, ConfigReader, LayerKinds


@dataclass(frozen=True)
class KeyValueAttentionSizes:
    heads: int
    kv_heads: int
    dim: int              # of a head's queries and keys, and of its values, which are the keys
    scale: float
    rot_dims: int         # how many of a head's first dimensions the rotation turns, 2i with 2i + 1 (0: none)
    rot_base: float
    rot_slowed: tuple | None      # (factor, low, high, original) or None
    chunk: int            # keys are seen within the query's chunk of that many positions, counted from 0 (0: all earlier keys)


@dataclass(frozen=True)
class LurepelDense:
    ff: int


@dataclass(frozen=True)
class LurepelExperts:
    experts: int          # with matrices of their own
    identity: int         # more of them, numbered behind, whose output is their input
    top: int
    expert_ff: int


@dataclass(frozen=True)
class LurepelLayer:
    kind: str             # "attention"
    mixer: KeyValueAttentionSizes
    mlp: object           # LurepelDense, LurepelExperts or None


MIXER_KINDS = {"attention": "keyed_value_attention"}


def _block(reader: ConfigReader, key: str, origin: str) -> ConfigReader:
    value = reader.raw(key)
    if not isinstance(value, dict):
        raise ConfigError(f"{origin}: {key!r} must be an object")
    return ConfigReader(value, f"{origin}: {key}")


def _rotation(mixer: ConfigReader, origin: str, most: int):
    """(dims, base, slowed) of a mixer's `rot` block; (0, 1.0, None) without one."""
    if not mixer.has("rot"):
        return 0, 1.0, None
    rot = _block(mixer, "rot", origin)
    dims = rot.integer("dims", minimum=0, maximum=most)
    if dims % 2:
        raise ConfigError(f"{origin}: rot.dims turns pairs of dimensions, got {dims}")
    base = rot.number("base")
    if base <= 0.0:
        raise ConfigError(f"{origin}: rot.base must be positive, got {base}")
    slowed = None
    if rot.has("scaling"):
        scaling = _block(rot, "scaling", origin + ": rot")
        slowed = tuple(scaling.number(key) for key in ("factor", "low", "high", "original"))
        if slowed[0] <= 0.0 or slowed[3] <= 0.0 or not 0.0 <= slowed[1] <= slowed[2]:
            raise ConfigError(f"{origin}: rot.scaling needs a positive factor and length and 0 <= low <= high, got {slowed}")
    return dims, base, slowed


@dataclass(frozen=True)
class LurepelConfig:
    architecture: str
    vocab: int
    hidden: int
    layers: tuple
    rms_eps: float        # the one eps of every norm of the model

    max_position = None   # the file sets no limit: the cache's capacity is the limit
    tie_word_embeddings = False

    @property
    def n_layers(self) -> int:
        return len(self.layers)

    def layer_kinds(self) -> list:
        def feed_forward(layer):
            if layer.mlp is None:
                return "none"
            return "geglu_tanh" if isinstance(layer.mlp, LurepelDense) else "routed_identity_experts"

        return [LayerKinds(mixer=MIXER_KINDS[layer.kind], feed_forward=feed_forward(layer), norm="rmsnorm", block="output_norm")
                for layer in self.layers]

    def schedule(self) -> list:
        return [(layer, layer) for layer in range(self.n_layers)]

    # ---- reading ----
    @classmethod
    def from_dict(cls, data: dict, origin: str = "config.json") -> "LurepelConfig":
        r = ConfigReader(data, origin)
        architecture = r.string("architecture") if r.has("architecture") else str((data.get("architectures") or ["Lurepel"])[0])
        vocab = r.integer("vocab", minimum=1)
        hidden = r.integer("width", minimum=1)
        rms_eps = _block(r, "norm", origin).number("eps")
        if rms_eps <= 0.0:
            raise ConfigError(f"{origin}: norm.eps must be positive, got {rms_eps}")
        listed = r.raw("layers")
        if not isinstance(listed, list) or not listed:
            raise ConfigError(f"{origin}: 'layers' must be a list with at least one layer")
        layers = tuple(cls._layer(item, f"{origin}: layers[{index}]") for index, item in enumerate(listed))
        return cls(architecture=architecture, vocab=vocab, hidden=hidden, layers=layers, rms_eps=rms_eps)

    @staticmethod
    def _layer(item, origin: str) -> LurepelLayer:
        r = ConfigReader(item, origin)
        kind = r.string("type")
        if kind not in MIXER_KINDS:
            raise ConfigError(f"{origin}: layer type {kind!r} is not implemented; only {sorted(MIXER_KINDS)}")
        m = _block(r, "mixer", origin)
        heads, kv_heads, dim = m.integer("heads", minimum=1), m.integer("kv_heads", minimum=1), m.integer("dim", minimum=1)
        if heads % kv_heads:
            raise ConfigError(f"{origin}: {heads} query heads do not group evenly into {kv_heads} kv_heads")
        if m.integer("vdim", default=dim) != dim:
            raise ConfigError(f"{origin}: the values are the keys, so vdim {m.raw('vdim')} must be dim {dim}")
        rot_dims, rot_base, rot_slowed = _rotation(m, origin + ": mixer", dim)
        chunk = _block(m, "mask", origin + ": mixer").integer("size", minimum=1) if m.has("mask") else 0
        mixer = KeyValueAttentionSizes(heads=heads, kv_heads=kv_heads, dim=dim, scale=m.number("scale"), rot_dims=rot_dims,
                                       rot_base=rot_base, rot_slowed=rot_slowed, chunk=chunk)
        mlp = None
        if r.has("mlp"):
            f = _block(r, "mlp", origin)
            form = f.string("kind")
            if form == "dense":
                mlp = LurepelDense(ff=f.integer("ff", minimum=1))
            elif form == "moe":
                router = _block(f, "router", origin + ": mlp")
                experts = router.integer("experts", minimum=1)
                identity = router.integer("identity", default=0, minimum=0)
                top = router.integer("top", minimum=1)
                if top > experts + identity:
                    raise ConfigError(f"{origin}: mlp.router.top {top} is more than the {experts + identity} experts")
                mlp = LurepelExperts(experts=experts, identity=identity, top=top,
                                     expert_ff=_block(f, "expert", origin + ": mlp").integer("ff", minimum=1))
            else:
                raise ConfigError(f"{origin}: mlp.kind {form!r} is not implemented; only 'dense' and 'moe'")
        return LurepelLayer(kind=kind, mixer=mixer, mlp=mlp)
