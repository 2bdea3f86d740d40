"""The Zigelorn decoder as a recipe of parts.

config.json: {"architecture": "Zigelorn", "vocab", "width", "norm": {"eps"}, "layers": [...]}. Every entry of ``layers`` has
``type`` ("attention", "retention" or "wkv"), the sizes of its mixer (``mixer``) and its feed-forward (``mlp``, or null for
none). An entry with ``weights_of: j`` has no tensors: it runs layer j's weights (mixer, feed-forward, norms) with a cache or
a state of its own.

* a layer norms both sides of each sublayer on a float32 stream: x += norm1b(mixer(norm1(x))), then
  x += norm2b(mlp(norm2(x))); these norms and the last one are RMS norms whose weights are stored as distances from one.
* "attention": ``rotary_attention`` whose values are its keys as projected (bias included); biases on q and k; all of q and
  all of k are RMS-normed over the whole projection; the first ``rot.dims`` coordinates of a head are turned (pairs
  (i, i + dims / 2), ``rot.base``, frequencies scaled part by part by ``rot.scaling``); ``scale``; a window of ``mask.size``
  positions; a sigmoid gate per head on the result.
* "retention": a recurrence with the fixed decays ``decay``, queries and keys turned over ``rot.dims`` coordinates.
* "wkv": a recurrence whose decays the token sets, with token shift and a bonus for the token itself. The inner size of its
  low-rank decays stands in no key of config.json and is read from the shape of the stored ``l<i>.mix.w1``; a config.json
  written for random weights names it itself (``decay_rank`` beside the mixer's other sizes).
* ``mlp.kind`` "dense": down(gelu(up(x))) of inner size ``ff``. "moe": ``router.experts`` experts down(relu(up(x))^2) of inner
  size ``expert.ff``, of which a token uses the ``router.top`` with the largest softmax score plus correction among the best
  ``router.groups.keep`` of ``router.groups.count`` groups; ``router.identity`` further outputs of the router hand their
  input on; the scores weigh the outputs and are not renormalised.

The head is the embedding table.

Nothing here computes: ``parse_config`` checks and types the keys, ``build_spec`` turns them into a ``ModelSpec``,
``checkpoint_names`` places the stored tensors in the model's (packed) parameters.
"""
from __future__ import annotations

from dataclasses import dataclass, field

from ..config.model_config import ConfigError, require
from ..config.registry import Architecture, WeightSource, register_architecture
from ..parts.model import LayerSpec, ModelSpec, RunEntry

# positions are counted in int32; far below that they are exact in every product with a frequency
MAX_POSITION = 1 << 24


@dataclass(frozen=True)
class Rotation:
    dims: int = 0
    base: float = 1.0
    scaling: tuple | None = None            # (factor, original, fast, slow)


@dataclass(frozen=True)
class AttentionSizes:
    heads: int
    kv_heads: int
    dim: int
    scale: float
    window: int | None
    rot: Rotation


@dataclass(frozen=True)
class RetentionSizes:
    heads: int
    dim: int
    vdim: int
    decay: tuple
    rot: Rotation


@dataclass(frozen=True)
class WKVSizes:
    heads: int
    dim: int
    decay_rank: int


@dataclass(frozen=True)
class MlpSizes:
    kind: str                               # "dense" | "moe"
    ff: int                                 # inner size of the dense feed-forward, or of one expert
    experts: int = 0
    top: int = 0
    groups: tuple = (1, 1)                  # (count, keep)
    identity: int = 0


@dataclass(frozen=True)
class LayerSizes:
    type: str
    mixer: object
    mlp: MlpSizes | None
    weights_of: int | None = None           # the layer (index in config.json) whose weights this one runs
    spare_norms: tuple = ()                 # norms that the checkpoint stores for a feed-forward that the layer does not have


@dataclass(frozen=True)
class ZigelornConfig:
    vocab: int
    width: int
    eps: float
    layers: tuple
    max_position: int = MAX_POSITION
    raw: dict = field(default_factory=dict, compare=False, repr=False)

    def owners(self) -> list[int]:
        """Config indices of the layers that have tensors of their own, in order."""
        return [i for i, layer in enumerate(self.layers) if layer.weights_of is None]


def _where(i: int, key: str) -> str:
    return f"config.json: layers[{i}].{key}"


def _rotation(i: int, m: dict, dim: int, may_scale: bool) -> Rotation:
    rot = m.get("rot") or {}
    if not rot:
        return Rotation()
    scaling = rot.get("scaling")
    if scaling and not may_scale:
        raise ConfigError(f"{_where(i, 'mixer.rot.scaling')}: this mixer's rotation is not scaled")
    r = Rotation(require(rot, "dims"), require(rot, "base", float),
                 tuple(require(scaling, key, float) for key in ("factor", "original", "fast", "slow")) if scaling else None)
    if r.dims < 0 or r.dims % 2 or r.dims > dim:
        raise ConfigError(f"{_where(i, 'mixer')}: rot.dims {r.dims} must be even and at most dim {dim}")
    if not r.base > 0 or (r.scaling is not None and (min(r.scaling) <= 0 or r.base == 1.0)):
        raise ConfigError(f"{_where(i, 'mixer.rot')}: base and the constants of the scaling must be positive")
    return r


def _attention(i: int, m: dict, shapes) -> AttentionSizes:
    mask = m.get("mask") or {}
    dim = require(m, "dim")
    a = AttentionSizes(require(m, "heads"), require(m, "kv_heads"), dim, require(m, "scale", float),
                       require(mask, "size") if mask else None, _rotation(i, m, dim, True))
    if min(a.heads, a.kv_heads, a.dim) <= 0 or a.heads % a.kv_heads:
        raise ConfigError(f"{_where(i, 'mixer')}: sizes must be positive and heads a multiple of kv_heads")
    if m.get("vdim", dim) != dim:
        raise ConfigError(f"{_where(i, 'mixer')}: the values are the keys, so vdim {m['vdim']} must equal dim {dim}")
    if a.window is not None and a.window <= 0:
        raise ConfigError(f"{_where(i, 'mixer.mask.size')} must be positive")
    return a


def _retention(i: int, m: dict, shapes) -> RetentionSizes:
    dim, decay = require(m, "dim"), m.get("decay")
    r = RetentionSizes(require(m, "heads"), dim, require(m, "vdim"), tuple(float(g) for g in decay or ()), _rotation(i, m, dim, False))
    if min(r.heads, r.dim, r.vdim) <= 0:
        raise ConfigError(f"{_where(i, 'mixer')}: sizes must be positive")
    if len(r.decay) != r.heads or min(r.decay) < 0 or max(r.decay) > 1:
        raise ConfigError(f"{_where(i, 'mixer.decay')}: one number from 0 to 1 for each of {r.heads} heads, got {decay!r}")
    return r


def _wkv(i: int, m: dict, shapes) -> WKVSizes:
    name = f"l{i}.mix.w1"
    if "decay_rank" in m:
        rank = require(m, "decay_rank")
    elif shapes is not None and len(shapes.get(name, ())) == 2:
        rank = int(shapes[name][0])
    else:
        raise ConfigError(f"{_where(i, 'mixer')}: the inner size of the decays stands neither in 'decay_rank' nor in a stored "
                          f"tensor '{name}'")
    w = WKVSizes(require(m, "heads"), require(m, "dim"), rank)
    if min(w.heads, w.dim, w.decay_rank) <= 0:
        raise ConfigError(f"{_where(i, 'mixer')}: sizes must be positive")
    return w


_MIXERS = {"attention": _attention, "retention": _retention, "wkv": _wkv}


def _mlp(i: int, mlp) -> MlpSizes | None:
    if mlp is None:
        return None
    where = _where(i, "mlp")
    kind = mlp.get("kind") if isinstance(mlp, dict) else None
    if kind == "dense":
        out = MlpSizes("dense", require(mlp, "ff"))
    elif kind == "moe":
        router = mlp.get("router") or {}
        groups = router.get("groups")
        out = MlpSizes("moe", require(mlp.get("expert") or {}, "ff"), experts=require(router, "experts"), top=require(router, "top"),
                       groups=(require(groups, "count"), require(groups, "keep")) if groups else (1, 1),
                       identity=require(router, "identity") if router.get("identity") else 0)
        total, (count, keep) = out.experts + out.identity, out.groups
        if out.experts <= 0 or out.identity < 0 or not 0 < keep <= count or total % count or not 0 < out.top <= keep * (total // count):
            raise ConfigError(f"{where}.router: {out.top} of {out.experts} experts and {out.identity} identities, {keep} of {count} groups")
    else:
        raise ConfigError(f"{where}.kind: {kind!r} is not known ('dense' and 'moe' are)")
    if out.ff <= 0:
        raise ConfigError(f"{where}: the inner size must be positive")
    return out


def parse_config(raw: dict, shapes: dict | None = None) -> ZigelornConfig:
    """``shapes``: {stored tensor name: shape} of the checkpoint where there is one: the inner sizes of the decays, and whether
    a layer without feed-forward stores that feed-forward's norms all the same."""
    eps = require(raw.get("norm") or {}, "eps", float)
    if not eps > 0:
        raise ConfigError("config.json: norm.eps must be positive")
    entries = raw.get("layers")
    if not isinstance(entries, list) or not entries:
        raise ConfigError("config.json: 'layers' must be a list with at least one layer")
    layers = []
    for i, entry in enumerate(entries):
        kind, m, j = entry.get("type"), entry.get("mixer"), entry.get("weights_of")
        if kind not in _MIXERS:
            raise ConfigError(f"{_where(i, 'type')}: {kind!r} is not known ({sorted(_MIXERS)} are)")
        if not isinstance(m, dict):
            raise ConfigError(f"{_where(i, 'mixer')} is missing")
        if j is not None and (not isinstance(j, int) or isinstance(j, bool) or not 0 <= j < i):
            raise ConfigError(f"{_where(i, 'weights_of')}: {j!r} must name an earlier layer")
        if j is not None and layers[j].weights_of is not None:
            j = layers[j].weights_of                         # (a layer that itself runs another one's weights: that one's)
        mlp, same = _mlp(i, entry.get("mlp")), j is None or kind == layers[j].type
        mixer = _MIXERS[kind](i if j is None else j, m, shapes) if same else None
        if j is not None and (not same or (mixer, mlp) != (layers[j].mixer, layers[j].mlp)):
            raise ConfigError(f"{_where(i, 'weights_of')}: the entry must equal layer {j}'s, whose weights it runs")
        spare = tuple(n for n in ("norm2", "norm2b") if mlp is None and j is None and shapes is not None and f"l{i}.{n}" in shapes)
        layers.append(LayerSizes(kind, mixer, mlp, j, spare))
    cfg = ZigelornConfig(vocab=require(raw, "vocab"), width=require(raw, "width"), eps=eps, layers=tuple(layers),
                         max_position=min(int(raw.get("max_position") or MAX_POSITION), MAX_POSITION), raw=dict(raw))
    if cfg.vocab <= 0 or cfg.width <= 0:
        raise ConfigError("config.json: 'vocab' and 'width' must be positive")
    return cfg


def build_spec(cfg: ZigelornConfig) -> ModelSpec:
    W = cfg.width
    norm = {"kind": "stream_rmsnorm", "size": W, "eps": cfg.eps, "zero_centred": True}
    layers, positions, index = [], {}, {}
    for i in cfg.owners():
        layer, m, position = cfg.layers[i], cfg.layers[i].mixer, None
        if layer.type != "wkv" and m.rot.dims:
            position = f"l{i}"
            factor, original, fast, slow = m.rot.scaling or (None,) * 4
            positions[position] = {"kind": "yarn_frequencies", "rotary_dim": m.rot.dims, "base": m.rot.base, "factor": factor,
                                   "original": original, "fast": fast, "slow": slow}
        if layer.type == "attention":
            mixer = {"kind": "rotary_attention", "num_kv_heads": m.kv_heads, "head_dim": m.dim, "value_dim": m.dim,
                     "scale": m.scale, "bias": True, "window": m.window, "head_gate": True, "values_are_keys": True,
                     "projection_norm_eps": cfg.eps}
            if position is None:
                mixer["position"] = None
        elif layer.type == "retention":
            mixer = {"kind": "retention", "head_dim": m.dim, "value_dim": m.vdim, "decay": m.decay, "eps": cfg.eps}
        else:
            mixer = {"kind": "wkv", "head_dim": m.dim, "decay_rank": m.decay_rank, "eps": cfg.eps}
        mixer.update(hidden_size=W, num_heads=m.heads)
        p, ff = layer.mlp, None
        if p is not None and p.kind == "dense":
            ff = {"kind": "plain_mlp", "hidden_size": W, "intermediate_size": p.ff, "activation": "gelu_tanh"}
        elif p is not None:
            ff = {"kind": "routed_experts", "hidden_size": W, "num_experts": p.experts, "top": p.top, "expert_size": p.ff,
                  "activation": "relu2", "gated": False, "scoring": "softmax", "scores_on": "output", "correction": True,
                  "groups": p.groups, "identity": p.identity}
        index[i] = len(layers)
        layers.append(LayerSpec(mixer=mixer, feed_forward=ff, norm=norm, position=position,
                                block={"kind": "sandwich_norms", "keeps_unused_norms": [_NORMS[n] for n in layer.spare_norms]}))
    order = [RunEntry(index[i if layer.weights_of is None else layer.weights_of]) for i, layer in enumerate(cfg.layers)]
    return ModelSpec(vocab_size=cfg.vocab, hidden_size=W, layers=layers, final_norm=norm, positions=positions,
                     max_position=cfg.max_position, tie_embeddings=True, run_order=order, embedding={"kind": "scaled_float", "scale": 1.0})


# a layer's stored norms, and the block's slots for them
_NORMS = {"norm1": "mixer_norm", "norm1b": "mixer_out_norm", "norm2": "feed_forward_norm", "norm2b": "feed_forward_out_norm"}


def checkpoint_names(cfg: ZigelornConfig) -> dict[str, WeightSource]:
    W = cfg.width
    names = {"embed": WeightSource("embed.weight"), "final.norm": WeightSource("final_norm.weight")}
    for at, i in enumerate(cfg.owners()):
        layer, m = cfg.layers[i], cfg.layers[i].mixer
        src, dst = f"l{i}.", f"layers.{at}."
        for name, slot in _NORMS.items():
            if name in ("norm1", "norm1b") or layer.mlp is not None or name in layer.spare_norms:
                names[src + name] = WeightSource(f"{dst}{slot}.weight")
        ms, md = src + "mix.", dst + "mixer."

        def packed(param: str, bands) -> None:
            row = 0
            for name, rows in bands:
                names[ms + name] = WeightSource(md + param, row, rows)
                row += rows

        if layer.type == "attention":
            q, k = m.heads * m.dim, m.kv_heads * m.dim
            packed("qkv.weight", (("q", q), ("k", k), ("g", m.heads)))
            packed("qkv.bias", (("q.b", q), ("k.b", k)))
            names[ms + "q.norm"] = WeightSource(md + "q_norm.weight")
            names[ms + "k.norm"] = WeightSource(md + "k_norm.weight")
        elif layer.type == "retention":
            q, v = m.heads * m.dim, m.heads * m.vdim
            packed("in.weight", (("q", q), ("k", q), ("v", v), ("g", v)))
        else:
            n = m.heads * m.dim
            packed("in.weight", (("r", n), ("k", n), ("v", n), ("g", n), ("w1", m.decay_rank)))
            packed("mu", tuple((f"mu.{x}", W) for x in "rkvgw"))
            for name, param in (("w2", "w2.weight"), ("w0", "w0"), ("u", "u"), ("norm", "norm.weight")):
                names[ms + name] = WeightSource(md + param)
        names[ms + "o"] = WeightSource(md + "o.weight")
        p = layer.mlp
        if p is None:
            continue
        fs, fd = src + "mlp.", dst + "feed_forward."
        if p.kind == "dense":
            names[fs + "up"] = WeightSource(fd + "up.weight")
            names[fs + "down"] = WeightSource(fd + "down.weight")
            continue
        names[fs + "router"] = WeightSource(fd + "router.weight")
        names[fs + "correction"] = WeightSource(fd + "router.correction")
        for e in range(p.experts):
            names[f"{fs}e{e}.up"] = WeightSource(fd + "up.weight", e * p.ff, p.ff)
            names[f"{fs}e{e}.down"] = WeightSource(fd + "down.weight", e * W, W)
    return names


def _shape(layers: int, width: int, ff: int, vocab: int, heads: int, kv_heads: int, dim: int, window: int, rank: int,
           experts: int, top: int, groups: tuple, identity: int, expert_ff: int, rot_dims: int, repeat: bool = True) -> dict:
    """Groups of four layers: two wkv, one attention, one retention; feed-forwards dense and routed in turn. With ``repeat``
    the last attention layer runs the first one's weights."""
    moe = {"kind": "moe", "expert": {"ff": expert_ff},
           "router": {"experts": experts, "groups": {"count": groups[0], "keep": groups[1]}, "identity": identity, "top": top}}
    entries, first, last = [], None, None
    for i in range(layers):
        mlp = moe if i % 2 else {"kind": "dense", "ff": ff}
        if i % 4 == 2:
            entry = {"type": "attention",
                     "mixer": {"dim": dim, "heads": heads, "kv_heads": kv_heads, "mask": {"size": window},
                               "rot": {"base": 500000.0, "dims": rot_dims,
                                       "scaling": {"factor": 8.0, "fast": 32.0, "original": 4096, "slow": 1.0}},
                               "scale": dim ** -0.5, "vdim": dim}}
            first, last = (i if first is None else first), i
        elif i % 4 == 3:
            entry = {"type": "retention",
                     "mixer": {"decay": [1.0 - 2.0 ** -(5.0 + 7.0 * h / max(heads - 1, 1)) for h in range(heads)], "dim": dim,
                               "heads": heads, "rot": {"base": 10000.0, "dims": dim}, "vdim": dim}}
        else:
            entry = {"type": "wkv", "mixer": {"decay_rank": rank, "dim": dim, "heads": heads}}
        entry["mlp"] = mlp
        entries.append(entry)
    if repeat and last is not None and last != first:
        entries[last]["weights_of"] = first
    return {"architecture": "Zigelorn", "layers": entries, "norm": {"eps": 1e-6}, "vocab": vocab, "width": width}


# config.json contents of sizes that measurements and examples name; the engine itself takes every size from a config.json
SHAPES = {
    "zigelorn-tiny": _shape(7, 72, 88, 173, 3, 1, 20, 13, 6, 7, 3, (3, 2), 2, 24, 12),
    "zigelorn-1b": _shape(8, 2048, 6144, 32768, 16, 8, 128, 1024, 64, 16, 2, (2, 1), 2, 1536, 128, repeat=False),
    "zigelorn-8b": _shape(4, 4096, 12288, 151936, 32, 8, 128, 4096, 128, 32, 4, (4, 2), 4, 1536, 128, repeat=False),
}


ZIGELORN = Architecture(
    name="Zigelorn",
    model_types=("zigelorn",),
    parse_config=parse_config,
    build_spec=build_spec,
    checkpoint_names=checkpoint_names,
    named_shapes=SHAPES,
    reads_checkpoint_shapes=True,
)
register_architecture(ZIGELORN, replace=True)
