"""Small Zigelorn configurations, random weights for them and ways of cutting requests into steps, for the tests.

The configurations differ from each other in every size and option; among them are values that make two sizes equal
or 1 (one head, one expert, one group, all experts chosen, a window of one position and one longer than any request, a rank
of one), layers without feed-forward, no rotation, a partial and a whole one with and without scaling, no identity experts
and more of them than others, layers that run another layer's weights. Weights are drawn wide enough that attention is far
from uniform and the router's choices are clear; they are stored in bfloat16, so runs in both element types read the
same numbers.
"""
from __future__ import annotations

import json
import os

import torch

from pevazen_cases import in_portions, interleaved, peak_tokens, tokens, whole  # noqa: F401  (ways of cutting, shared)


def attention(heads, kv_heads, dim, window, scale, rot_dims=0, base=1.0, scaling=None):
    m = {"dim": dim, "heads": heads, "kv_heads": kv_heads, "scale": scale, "vdim": dim}
    if window is not None:
        m["mask"] = {"size": window}
    if rot_dims:
        m["rot"] = {"base": base, "dims": rot_dims}
        if scaling is not None:
            m["rot"]["scaling"] = dict(zip(("factor", "original", "fast", "slow"), scaling))
    return {"type": "attention", "mixer": m}


def retention(decay, dim, vdim, rot_dims=0, base=1.0):
    m = {"decay": list(decay), "dim": dim, "heads": len(decay), "vdim": vdim}
    if rot_dims:
        m["rot"] = {"base": base, "dims": rot_dims}
    return {"type": "retention", "mixer": m}


def wkv(heads, dim):
    return {"type": "wkv", "mixer": {"dim": dim, "heads": heads}}


def dense(ff):
    return {"kind": "dense", "ff": ff}


def moe(experts, top, ff, groups=None, identity=0):
    router = {"experts": experts, "identity": identity, "top": top}
    if groups is not None:
        router["groups"] = {"count": groups[0], "keep": groups[1]}
    return {"kind": "moe", "expert": {"ff": ff}, "router": router}


def with_mlp(entry, mlp, weights_of=None):
    return dict(entry, mlp=mlp, **({} if weights_of is None else {"weights_of": weights_of}))


def model(vocab, width, eps, layers):
    return {"architecture": "Zigelorn", "layers": layers, "norm": {"eps": eps}, "vocab": vocab, "width": width}


_ATT_A = with_mlp(attention(4, 2, 8, 6, 0.5, 4, 100.0, (2.0, 40, 8.0, 0.5)), dense(24))
_WKV_A = with_mlp(wkv(3, 8), moe(5, 2, 12, (2, 1), 1))
# width a multiple of 8; layers that run another layer's weights; a layer without feed-forward; groups; one identity expert
CONFIG_A = model(67, 40, 1e-5, [
    _WKV_A,
    _ATT_A,
    with_mlp(retention([0.9, 0.99], 12, 10, 6, 50.0), None),
    with_mlp(_ATT_A, _ATT_A["mlp"], 1),
    with_mlp(retention([0.97, 0.5, 0.999], 4, 6, 4, 1000.0), moe(6, 3, 8, (4, 3), 2)),
    with_mlp(_WKV_A, _WKV_A["mlp"], 0),
])
# a width that is no multiple of 8, one head, one expert, all experts chosen, a window of one position and one longer than any
# request, no rotation, odd head sizes
CONFIG_B = model(50, 36, 1e-3, [
    with_mlp(wkv(1, 5), moe(1, 1, 10)),
    with_mlp(attention(1, 1, 10, 1, 0.3, 10, 20.0), moe(2, 3, 6, (1, 1), 1)),
    with_mlp(retention([1.0], 7, 3), dense(20)),
    with_mlp(attention(3, 1, 6, 1000, 0.6), moe(2, 4, 6, (3, 2), 4)),
    with_mlp(wkv(2, 18), None),
])
# head sizes that the kernels on the matrix cores take, rotations whole and partial
_RET_C = with_mlp(retention([0.95, 0.998], 32, 16, 32, 10000.0), moe(6, 2, 16, (2, 2), 2))
CONFIG_C = model(90, 64, 2e-6, [
    _RET_C,
    with_mlp(wkv(4, 16), dense(40)),
    with_mlp(attention(4, 1, 32, 20, 0.2, 16, 300.0, (4.0, 64, 16.0, 1.0)), moe(8, 2, 8, (4, 1), 0)),
    with_mlp(attention(2, 2, 16, 11, 0.25, 16, 10000.0), dense(48)),
    with_mlp(_RET_C, _RET_C["mlp"], 0),
])
# recorded steps
CONFIG_R = model(40, 32, 1e-5, [
    with_mlp(wkv(2, 16), moe(4, 2, 8, (3, 2), 2)),
    with_mlp(attention(2, 1, 16, 12, 0.3, 16, 1000.0, (2.0, 32, 8.0, 1.0)), dense(16)),
    with_mlp(retention([0.9, 0.99], 16, 24, 8, 100.0), dense(24)),
])
# windows longer than a page of 64 tokens, one of them no multiple of it
CONFIG_S = model(120, 64, 1e-6, [
    with_mlp(attention(4, 2, 32, 150, 0.18, 32, 20000.0, (4.0, 128, 16.0, 1.0)), moe(6, 2, 16, (2, 1), 2)),
    with_mlp(wkv(2, 32), dense(48)),
    with_mlp(retention([0.99, 0.999], 48, 32, 16, 300000.0), moe(4, 2, 16, (1, 1), 1)),
    with_mlp(attention(2, 2, 16, 80, 0.25, 8, 300000.0), dense(32)),
])
# the sizes of a real model's layers in small number: heads of 128 and 64, a width of 1,024
CONFIG_W = model(500, 1024, 1e-6, [
    with_mlp(wkv(8, 128), moe(8, 2, 256, (2, 1), 2)),
    with_mlp(attention(8, 2, 128, 256, 0.09, 128, 20000.0, (4.0, 512, 32.0, 1.0)), dense(2048)),
    with_mlp(retention([0.97, 0.99, 0.998, 0.9995], 128, 256, 128, 300000.0), moe(6, 3, 512, (4, 2), 2)),
    with_mlp(wkv(16, 64), dense(1024)),
])

CASES = {"A": (CONFIG_A, 31), "B": (CONFIG_B, 42), "C": (CONFIG_C, 33), "R": (CONFIG_R, 34), "S": (CONFIG_S, 35)}
RANKS = (3, 1, 8, 5, 20)      # the inner sizes of the decays, by the layer's number


def random_tensors(config: dict, seed: int) -> dict[str, torch.Tensor]:
    g = torch.Generator().manual_seed(seed)
    W = config["width"]
    out = {}

    def normal(shape, std, mean=0.0):
        return mean + std * torch.randn(shape, generator=g)

    def matrix(rows, cols, gain=1.0):
        return normal((rows, cols), gain / cols ** 0.5)

    out["embed"] = normal((config["vocab"], W), 1.0)
    out["final.norm"] = normal((W,), 0.1)
    for i, layer in enumerate(config["layers"]):
        if layer.get("weights_of") is not None:
            continue
        p, m = f"l{i}.", layer["mixer"]
        out[p + "norm1"] = normal((W,), 0.1, 0.1)
        out[p + "norm1b"] = normal((W,), 0.1, -0.3)
        q = p + "mix."
        if layer["type"] == "attention":
            H, G, D = m["heads"], m["kv_heads"], m["dim"]
            for name, n in (("q", H * D), ("k", G * D)):
                out[q + name] = matrix(n, W)
                out[q + name + ".b"] = normal((n,), 0.4)
                out[q + name + ".norm"] = normal((n,), 0.3, 1.6)
            out[q + "g"] = matrix(H, W, 2.0)
            out[q + "o"] = matrix(W, H * D)
        elif layer["type"] == "retention":
            H, D, E = m["heads"], m["dim"], m["vdim"]
            for name, n in (("q", H * D), ("k", H * D), ("v", H * E), ("g", H * E)):
                out[q + name] = matrix(n, W)
            out[q + "o"] = matrix(W, H * E)
        else:
            H, D = m["heads"], m["dim"]
            R = RANKS[i % len(RANKS)]
            for x in "rkvgw":
                out[q + "mu." + x] = normal((W,), 0.3, 0.5)
            for x in "rkvg":
                out[q + x] = matrix(H * D, W)
            out[q + "w1"] = matrix(R, W, 1.5)
            out[q + "w2"] = matrix(H * D, R, 1.5)
            out[q + "w0"] = normal((H * D,), 1.5, -2.0)
            out[q + "u"] = normal((H, D), 0.5, 0.5)
            out[q + "norm"] = normal((H * D,), 0.2, 1.0)
            out[q + "o"] = matrix(W, H * D)
        mlp = layer.get("mlp")
        if mlp is None:
            continue
        out[p + "norm2"] = normal((W,), 0.1)
        out[p + "norm2b"] = normal((W,), 0.1, -0.2)
        f = p + "mlp."
        if mlp["kind"] == "dense":
            out[f + "up"] = matrix(mlp["ff"], W, 1.5)
            out[f + "down"] = matrix(W, mlp["ff"])
            continue
        n, ff = mlp["router"]["experts"], mlp["expert"]["ff"]
        total = n + mlp["router"].get("identity", 0)
        out[f + "router"] = matrix(total, W, 3.0)
        out[f + "correction"] = normal((total,), 0.2)
        for e in range(n):
            out[f + f"e{e}.up"] = matrix(ff, W, 1.5)
            out[f + f"e{e}.down"] = matrix(W, ff)
    return {k: v.to(torch.bfloat16) for k, v in out.items()}


def write_model(folder: str, config: dict, seed: int, tensors: dict | None = None) -> str:
    from safetensors.torch import save_file

    os.makedirs(folder, exist_ok=True)
    with open(os.path.join(folder, "config.json"), "w") as f:
        json.dump(config, f)
    tensors = random_tensors(config, seed) if tensors is None else tensors
    save_file({k: v.contiguous() for k, v in tensors.items()}, os.path.join(folder, "model.safetensors"))
    return folder


def random_config(seed: int) -> dict:
    """A configuration drawn at random (seeded): head sizes that the matrix-core kernels take and sizes that they do
    not, 1 to 6 query heads per key/value head, widths and vocabularies that are no multiple of 8, windows around the
    sizes of pages and tiles, any order of the three kinds of layer, weights run again."""
    import random
    r = random.Random(seed)
    layers = []
    for i in range(r.randint(3, 6)):
        again = [j for j, layer in enumerate(layers) if "weights_of" not in layer]
        if again and r.random() < 0.25:
            j = r.choice(again)
            layers.append(dict(layers[j], weights_of=j))
            continue
        kind, dim = r.choice(["attention", "retention", "wkv"]), r.choice([4, 6, 8, 16, 20, 32, 48, 64])
        rot = r.choice([0, 2, dim // 2 // 2 * 2, dim])
        if kind == "attention":
            kv = r.choice([1, 2, 3])
            scaling = r.choice([None, (4.0, 64, 16.0, 0.5), (16.0, 500, 32.0, 1.0)])
            entry = attention(kv * r.choice([1, 2, 3, 6]), kv, dim, r.choice([None, 1, 3, 15, 16, 17, 33, 63, 64, 65, 100, 500]),
                              r.choice([0.5, 1.0]) * dim ** -0.5, rot, r.choice([10.0, 1000.0, 300000.0]), scaling)
        elif kind == "retention":
            entry = retention([r.choice([0.0, 0.5, 0.9, 0.99, 0.999, 1.0]) for _ in range(r.choice([1, 2, 3]))], dim,
                              r.choice([3, 8, 16, 24, 40]), rot, r.choice([10.0, 10000.0]))
        else:
            entry = wkv(r.choice([1, 2, 3]), dim)
        what = r.choice(["none", "dense", "moe", "moe"])
        mlp = None
        if what == "dense":
            mlp = dense(r.choice([16, 24, 50]))
        elif what == "moe":
            size, count = r.choice([1, 2, 3]), r.choice([1, 2, 4])
            identity = r.randint(0, max(0, size * count - 1))
            keep = r.randint(1, count)
            mlp = moe(size * count - identity, r.randint(1, min(4, keep * size)), r.choice([6, 8, 16, 24]), (count, keep), identity)
        layers.append(with_mlp(entry, mlp))
    return model(r.choice([33, 64, 90, 131]), r.choice([24, 40, 52, 64, 72, 100]), r.choice([1e-6, 1e-5, 1e-3]), layers)
