"""The Gabelorn decoder as a recipe of parts.

config.json: {"architecture": "Gabelorn", "vocab", "width", "norm": {"eps"}, "logit_softcap", "layers": [...]}. Every entry
of ``layers`` has a ``type``, the sizes of its mixer (``mixer``) and its feed-forward (``mlp``, or null):

* ``latent_attention``: attention over a cached latent: ``heads``, ``dim`` (unrotated entries of a query/key head),
  ``rot_dim`` (rotated entries, one key part for all heads; ``rot``: {"base", "dims" = rot_dim}, pairs (i, i + dims / 2)),
  ``vdim``, ``kv_rank``, ``scale``, a window of ``mask.size`` positions, a sink per head, a gate per entry of the result.
* ``attention``: grouped-head attention over all earlier positions: ``heads``, ``kv_heads``, ``dim``, ``vdim``, ``scale``, no
  rotation but a bias by distance with a slope per head, queries scaled by their position (``q_temp``: {"coef", "every"}), a
  sink per head; with ``v_mix`` the first such layer's values are mixed into the layer's own.
* ``mlp``: {"kind": "dense", "ff", "limit"}: a gated feed-forward with biases whose gate and up values are clamped.

Every layer is pre-norm on one float32 stream (RMS norms with a weight vector); the head is a matrix of its own and the
logits are capped: c tanh(logits / c) with c = ``logit_softcap``.

Nothing here computes: ``parse_config`` checks and types the keys, ``build_spec`` turns them into a ``ModelSpec``,
``checkpoint_names`` places the stored tensors in the model's (packed) parameters.
"""
from __future__ import annotations

from dataclasses import dataclass, field

from ..config.model_config import ConfigError, require
from ..config.registry import Architecture, WeightSource, register_architecture
from ..parts.model import LayerSpec, ModelSpec

# positions are int32 in a step; distances between them are taken in float32, in which every integer up to here is exact
MAX_POSITION = 1 << 24
# the feed-forward's gate: g sigmoid(GATE_SLOPE g) (u + UP_OFFSET)
GATE_SLOPE = 1.702
UP_OFFSET = 1.0
# a cached latent's row is filled up to a multiple of what a step of the matrix cores takes
ROW_MULTIPLE = 16


@dataclass(frozen=True)
class LatentSizes:
    heads: int
    dim: int
    rot_dim: int
    vdim: int
    kv_rank: int
    scale: float
    window: int | None
    rot_base: float


@dataclass(frozen=True)
class AttentionSizes:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    temperature: tuple | None               # (coef, every)
    v_mix: bool


@dataclass(frozen=True)
class FeedForwardSizes:
    ff: int
    limit: float


@dataclass(frozen=True)
class LayerSizes:
    type: str
    mixer: LatentSizes | AttentionSizes
    mlp: FeedForwardSizes | None
    spare_norm: bool = False                # a layer without feed-forward whose checkpoint stores a second norm all the same


@dataclass(frozen=True)
class GabelornConfig:
    vocab: int
    width: int
    eps: float
    layers: tuple
    logit_softcap: float | None = None
    max_position: int = MAX_POSITION
    raw: dict = field(default_factory=dict, compare=False, repr=False)

    def first_mixing(self) -> int | None:
        """The first layer that mixes values: the one whose values the later ones mix in."""
        return next((i for i, layer in enumerate(self.layers) if layer.type == "attention" and layer.mixer.v_mix), None)


def _where(i: int, key: str) -> str:
    return f"config.json: layers[{i}].{key}"


def _latent(i: int, m: dict) -> LatentSizes:
    mask, rot = m.get("mask") or {}, m.get("rot") or {}
    rot_dim = require(m, "rot_dim") if m.get("rot_dim") is not None else 0
    a = LatentSizes(heads=require(m, "heads"), dim=require(m, "dim"), rot_dim=rot_dim, vdim=require(m, "vdim"),
                    kv_rank=require(m, "kv_rank"), scale=require(m, "scale", float),
                    window=require(mask, "size") if mask else None, rot_base=require(rot, "base", float) if rot_dim else 1.0)
    if min(a.heads, a.dim, a.vdim, a.kv_rank) <= 0:
        raise ConfigError(f"{_where(i, 'mixer')}: sizes must be positive")
    if a.rot_dim and (a.rot_dim < 0 or a.rot_dim % 2 or require(rot, "dims") != a.rot_dim):
        raise ConfigError(f"{_where(i, 'mixer.rot.dims')}: must be even, positive and equal to rot_dim {a.rot_dim}")
    if not a.rot_base > 0:
        raise ConfigError(f"{_where(i, 'mixer.rot.base')} must be positive")
    if a.window is not None and a.window <= 0:
        raise ConfigError(f"{_where(i, 'mixer.mask.size')} must be positive")
    return a


def _attention(i: int, m: dict) -> AttentionSizes:
    temp = m.get("q_temp")
    a = AttentionSizes(heads=require(m, "heads"), kv_heads=require(m, "kv_heads"), dim=require(m, "dim"),
                       vdim=require(m, "vdim"), scale=require(m, "scale", float),
                       temperature=(require(temp, "coef", float), require(temp, "every", float)) if temp else None,
                       v_mix=bool(m.get("v_mix", False)))
    if min(a.heads, a.kv_heads, a.dim, a.vdim) <= 0 or a.heads % a.kv_heads:
        raise ConfigError(f"{_where(i, 'mixer')}: sizes must be positive and heads a multiple of kv_heads")
    if a.temperature is not None and not a.temperature[1] > 0:
        raise ConfigError(f"{_where(i, 'mixer.q_temp.every')} must be positive")
    return a


def _feed_forward(i: int, mlp) -> FeedForwardSizes | None:
    if mlp is None:
        return None
    if not isinstance(mlp, dict) or mlp.get("kind") != "dense":
        raise ConfigError(f"{_where(i, 'mlp')}: an object of kind 'dense' or null, got {mlp!r}")
    f = FeedForwardSizes(require(mlp, "ff"), require(mlp, "limit", float))
    if f.ff <= 0 or not f.limit > 0:
        raise ConfigError(f"{_where(i, 'mlp')}: ff and limit must be positive")
    return f


def parse_config(raw: dict, shapes: dict | None = None) -> GabelornConfig:
    """``shapes``: {stored tensor name: shape} of the checkpoint where there is one: a layer without feed-forward may
    or may not store its second norm, and only the stored names tell."""
    eps = require(raw.get("norm") or {}, "eps", float)
    if not eps > 0:
        raise ConfigError("config.json: norm.eps must be positive")
    entries = raw.get("layers")
    if not isinstance(entries, list) or not entries:
        raise ConfigError("config.json: 'layers' must be a list with at least one layer")
    readers = {"latent_attention": _latent, "attention": _attention}
    layers = []
    for i, entry in enumerate(entries):
        kind, m = entry.get("type"), entry.get("mixer")
        if kind not in readers:
            raise ConfigError(f"{_where(i, 'type')}: {kind!r} is not known ({sorted(readers)} are)")
        if not isinstance(m, dict):
            raise ConfigError(f"{_where(i, 'mixer')} is missing")
        mlp = _feed_forward(i, entry.get("mlp"))
        layers.append(LayerSizes(kind, readers[kind](i, m), mlp, mlp is None and shapes is not None and f"l{i}.norm2" in shapes))
    cap = raw.get("logit_softcap")
    cfg = GabelornConfig(vocab=require(raw, "vocab"), width=require(raw, "width"), eps=eps, layers=tuple(layers),
                         logit_softcap=None if cap is None else require(raw, "logit_softcap", float),
                         max_position=min(int(raw.get("max_position") or MAX_POSITION), MAX_POSITION), raw=dict(raw))
    if cfg.vocab <= 0 or cfg.width <= 0:
        raise ConfigError("config.json: 'vocab' and 'width' must be positive")
    if cfg.logit_softcap is not None and not cfg.logit_softcap > 0:
        raise ConfigError("config.json: logit_softcap must be positive")
    first = cfg.first_mixing()
    for i, layer in enumerate(cfg.layers):
        if layer.type == "attention" and layer.mixer.v_mix:
            mine, theirs = layer.mixer, cfg.layers[first].mixer
            if (mine.kv_heads, mine.vdim) != (theirs.kv_heads, theirs.vdim):
                raise ConfigError(f"{_where(i, 'mixer')}: kv_heads and vdim must equal those of layer {first}, whose values it mixes in")
    return cfg


def build_spec(cfg: GabelornConfig) -> ModelSpec:
    # the stream is float32 and the norms are rounded once, whatever the engine's options say
    norm = {"kind": "rmsnorm", "size": cfg.width, "eps": cfg.eps, "residual_float32": True, "rounds_between": False}
    first = cfg.first_mixing()
    layers, positions = [], {}
    for i, layer in enumerate(cfg.layers):
        a = layer.mixer
        position = None
        if layer.type == "latent_attention":
            if a.rot_dim:
                position = f"l{i}"
                positions[position] = {"kind": "yarn_frequencies", "rotary_dim": a.rot_dim, "base": a.rot_base}
            mixer = {"kind": "latent_attention", "hidden_size": cfg.width, "num_heads": a.heads, "head_dim": a.dim,
                     "rot_dim": a.rot_dim, "value_dim": a.vdim, "q_rank": None, "kv_rank": a.kv_rank, "scale": a.scale,
                     "eps": cfg.eps, "window": a.window, "learned_sink": True, "element_gate": True, "rotation": "halves",
                     "row_multiple": ROW_MULTIPLE}
        else:
            mix = None if not a.v_mix else ("first" if i == first else "later")
            mixer = {"kind": "rotary_attention", "hidden_size": cfg.width, "num_heads": a.heads, "num_kv_heads": a.kv_heads,
                     "head_dim": a.dim, "value_dim": a.vdim, "scale": a.scale, "bias": False, "position": None,
                     "learned_sink": True, "distance_bias": True, "temperature": a.temperature, "mix_values": mix}
        ff = None
        if layer.mlp is not None:
            ff = {"kind": "swiglu", "hidden_size": cfg.width, "intermediate_size": layer.mlp.ff, "activation": "clamped_swish",
                  "bias": True, "limit": layer.mlp.limit, "alpha": GATE_SLOPE, "offset": UP_OFFSET}
        layers.append(LayerSpec(mixer=mixer, feed_forward=ff, norm=norm, position=position,
                                block={"kind": "prenorm", "keeps_unused_norm": layer.spare_norm}))
    return ModelSpec(vocab_size=cfg.vocab, hidden_size=cfg.width, layers=layers, final_norm=norm, positions=positions,
                     max_position=cfg.max_position, tie_embeddings=False, logit_cap=cfg.logit_softcap)


def checkpoint_names(cfg: GabelornConfig) -> dict[str, WeightSource]:
    names = {"embed": WeightSource("embed.weight"), "head": WeightSource("head.weight"),
             "final.norm": WeightSource("final_norm.weight")}
    for i, layer in enumerate(cfg.layers):
        src, dst = f"l{i}.", f"layers.{i}."
        names[src + "norm1"] = WeightSource(dst + "mixer_norm.weight")
        a = layer.mixer
        ms, md = src + "mix.", dst + "mixer."
        if layer.type == "latent_attention":
            packed, parts = "down.weight", (("q", a.heads * (a.dim + a.rot_dim)), ("dkv", a.kv_rank + a.rot_dim),
                                            ("g", a.heads * a.vdim))
            names[ms + "dkv.norm"] = WeightSource(md + "kv_norm.weight")
            names[ms + "uk"] = WeightSource(md + "uk.weight")
            names[ms + "uv"] = WeightSource(md + "uv.weight")
        else:
            packed, parts = "qkv.weight", (("q", a.heads * a.dim), ("k", a.kv_heads * a.dim), ("v", a.kv_heads * a.vdim))
            if a.v_mix:
                names[ms + "vmix"] = WeightSource(md + "vmix")
        row = 0
        for name, rows in parts:
            names[ms + name] = WeightSource(md + packed, row, rows)
            row += rows
        names[ms + "sink"] = WeightSource(md + "sink")
        names[ms + "o"] = WeightSource(md + "o.weight")
        if layer.mlp is not None or layer.spare_norm:
            names[src + "norm2"] = WeightSource(dst + "feed_forward_norm.weight")
        if layer.mlp is not None:
            fs, fd, ff = src + "mlp.", dst + "feed_forward.", layer.mlp.ff
            for name, start in (("gate", 0), ("up", ff)):
                names[fs + name] = WeightSource(fd + "gate_up.weight", start, ff)
                names[fs + name + ".b"] = WeightSource(fd + "gate_up.bias", start, ff)
            names[fs + "down"] = WeightSource(fd + "down.weight")
            names[fs + "down.b"] = WeightSource(fd + "down.bias")
    return names


def _shape(layers: int, width: int, ff: int, vocab: int, heads: int, dim: int, rot_dim: int, vdim: int, kv_rank: int, window: int,
           kv_heads: int, head_dim: int, limit: float, cap: float, coef: float, every: int) -> dict:
    """The two kinds of layer in turn, a latent one first; every attention layer but each third one mixes values."""
    entries = []
    for i in range(layers):
        mlp = {"kind": "dense", "ff": ff, "limit": limit}
        if i % 2 == 0:
            entries.append({"type": "latent_attention", "mlp": mlp,
                            "mixer": {"dim": dim, "heads": heads, "kv_rank": kv_rank, "mask": {"size": window},
                                      "rot": {"base": 10000.0, "dims": rot_dim}, "rot_dim": rot_dim,
                                      "scale": (dim + rot_dim) ** -0.5, "vdim": vdim}})
        else:
            entries.append({"type": "attention", "mlp": mlp,
                            "mixer": {"dim": head_dim, "heads": heads, "kv_heads": kv_heads,
                                      "q_temp": {"coef": coef, "every": every}, "scale": head_dim ** -0.5,
                                      "v_mix": i % 6 != 5, "vdim": head_dim}})
    return {"architecture": "Gabelorn", "layers": entries, "logit_softcap": cap, "norm": {"eps": 1e-6}, "vocab": vocab, "width": width}


# config.json contents of sizes that measurements and examples name; the engine takes every size from a config.json
SHAPES = {
    "gabelorn-tiny": _shape(6, 48, 80, 149, 3, 12, 4, 10, 20, 17, 1, 16, 1.5, 9.0, 0.25, 11),
    "gabelorn-1b": _shape(16, 2048, 6144, 32768, 16, 128, 64, 128, 192, 1024, 4, 128, 7.0, 30.0, 0.1, 4096),
    "gabelorn-8b": _shape(36, 4096, 12288, 151936, 32, 128, 64, 128, 192, 2048, 8, 128, 7.0, 30.0, 0.1, 4096),
}


GABELORN = Architecture(
    name="Gabelorn",
    model_types=("gabelorn",),
    parse_config=parse_config,
    build_spec=build_spec,
    checkpoint_names=checkpoint_names,
    named_shapes=SHAPES,
    reads_checkpoint_shapes=True,
)
register_architecture(GABELORN, replace=True)
