"""Small Gabelorn configurations, random weights for them and ways of cutting requests into steps, for the tests.

The configurations differ from each other in every size and option; among them are values that make two sizes equal
or 1 (one head, a window of one position, a window longer than any request, value heads of the key heads' size and of
another, one key/value head for all heads), numbers of heads that are no power of two, layers without feed-forward,
layers that mix values and layers that do not, stored rows that are a multiple of 16 and rows that are not. Weights are
drawn wide enough that attention is far from uniform, sinks and slopes matter and the feed-forward's clamps bind; they
are stored in bfloat16, so runs in both element types read the same numbers.
"""
from __future__ import annotations

import json
import os

import torch

from pevazen_cases import in_portions, interleaved, peak_tokens, tokens, whole  # noqa: F401  (ways of cutting, shared)


def latent(heads, dim, rot_dim, vdim, kv_rank, window, base, scale):
    m = {"dim": dim, "heads": heads, "kv_rank": kv_rank, "mask": {"size": window}, "rot": {"base": base, "dims": rot_dim},
         "rot_dim": rot_dim, "scale": scale, "vdim": vdim}
    return {"type": "latent_attention", "mixer": m}


def biased(heads, kv_heads, dim, vdim, scale, coef, every, v_mix):
    m = {"dim": dim, "heads": heads, "kv_heads": kv_heads, "q_temp": {"coef": coef, "every": every}, "scale": scale,
         "v_mix": v_mix, "vdim": vdim}
    return {"type": "attention", "mixer": m}


def model(vocab, width, eps, cap, layers):
    return {"architecture": "Gabelorn", "layers": layers, "logit_softcap": cap, "norm": {"eps": eps}, "vocab": vocab, "width": width}


def _with(entry, ff=None, limit=None):
    return dict(entry, mlp=None if ff is None else {"kind": "dense", "ff": ff, "limit": limit})


# width a multiple of 8; a layer without feed-forward; mixing layers of different head sizes, and one that does not mix between
CONFIG_A = model(67, 40, 1e-4, 6.0, [
    _with(latent(3, 8, 4, 6, 10, 6, 100.0, 0.6), 24, 1.0),
    _with(biased(4, 2, 6, 10, 0.5, 0.2, 5, True), 18, 0.5),
    _with(latent(2, 6, 2, 12, 7, 9, 1000.0, 0.5)),
    _with(biased(3, 1, 12, 4, 0.3, 0.0, 3, False), 24, 3.0),
    _with(biased(6, 2, 4, 10, 0.6, 0.25, 1, True), 20, 0.8),
    _with(biased(2, 2, 8, 10, 0.4, 0.2, 8, True)),
])
# a width that is no multiple of 8, one head, a window of one position and one longer than any request, sizes of 1
CONFIG_B = model(50, 36, 1e-2, 2.0, [
    _with(biased(1, 1, 8, 1, 0.35, 0.4, 7, False), 10, 0.7),
    _with(latent(1, 10, 10, 10, 6, 1, 20.0, 0.3), 36, 2.0),
    _with(latent(5, 1, 2, 3, 36, 1000, 5.0, 0.9), 9, 0.4),
    _with(biased(5, 5, 3, 3, 0.5, 0.3, 2, True), 20, 1.0),
])
# head sizes and rows that the kernels on the matrix cores take (and rows that are filled up to such a size)
CONFIG_C = model(90, 64, 2e-6, 8.0, [
    _with(latent(4, 16, 8, 16, 24, 11, 10000.0, 0.25), 40, 1.2),
    _with(biased(6, 2, 16, 16, 0.25, 0.4, 9, True), 48, 0.9),
    _with(latent(20, 8, 16, 8, 37, 20, 300.0, 0.2), 40, 1.0),
    _with(biased(18, 1, 32, 32, 0.2, 0.3, 16, False), 24, 0.6),
    _with(biased(2, 2, 32, 16, 0.18, 0.4, 30, True)),
])
# recorded steps
CONFIG_R = model(40, 32, 1e-5, 5.0, [
    _with(biased(2, 1, 16, 16, 0.3, 0.5, 6, True), 16, 1.0),
    _with(latent(2, 16, 16, 16, 16, 12, 1000.0, 0.25), 24, 1.5),
    _with(biased(4, 1, 16, 16, 0.3, 0.2, 10, True), 16, 0.8),
])
# windows around and beyond a page of 64 tokens, none of them a multiple of it but one
CONFIG_S = model(120, 64, 1e-6, 10.0, [
    _with(latent(4, 32, 16, 32, 48, 150, 20000.0, 0.15), 32, 1.0),
    _with(biased(8, 2, 32, 32, 0.18, 0.3, 50, True), 48, 0.7),
    _with(latent(2, 16, 32, 48, 32, 65, 300000.0, 0.2), 40, 2.0),
    _with(biased(4, 2, 64, 32, 0.12, 0.6, 33, True), 24, 1.0),
    _with(latent(3, 16, 8, 16, 24, 128, 500.0, 0.2), 40, 1.4),
])
# the sizes of a real model's layers in small number: heads of 128, rows of 256, more than 16 heads on a row, a width of 1,024
CONFIG_W = model(500, 1024, 1e-6, 20.0, [
    _with(latent(20, 128, 64, 128, 192, 190, 20000.0, 0.07), 1536, 2.0),
    _with(biased(8, 2, 128, 128, 0.09, 0.25, 70, True), 2048, 1.0),
    _with(biased(16, 2, 64, 128, 0.12, 0.25, 128, True), 1024, 3.0),
])

CASES = {"A": (CONFIG_A, 31), "B": (CONFIG_B, 42), "C": (CONFIG_C, 33), "R": (CONFIG_R, 34), "S": (CONFIG_S, 35)}


def random_tensors(config: dict, seed: int) -> dict[str, torch.Tensor]:
    g = torch.Generator().manual_seed(seed)
    W = config["width"]
    out = {}

    def normal(shape, std, mean=0.0):
        return mean + std * torch.randn(shape, generator=g)

    def matrix(rows, cols, gain=1.0):
        return normal((rows, cols), gain / cols ** 0.5)

    out["embed"] = normal((config["vocab"], W), 1.0)
    out["head"] = matrix(config["vocab"], W, 3.0)
    out["final.norm"] = normal((W,), 0.1, 1.0)
    for i, layer in enumerate(config["layers"]):
        p, m = f"l{i}.", layer["mixer"]
        H, D, E = m["heads"], m["dim"], m["vdim"]
        out[p + "norm1"] = normal((W,), 0.1, 1.1)
        if layer["type"] == "latent_attention":
            R, C = m["rot_dim"], m["kv_rank"]
            out[p + "mix.q"] = matrix(H * (D + R), W, 1.4)
            out[p + "mix.dkv"] = matrix(C + R, W, 1.5)
            out[p + "mix.dkv.norm"] = normal((C,), 0.2, 1.0)
            out[p + "mix.uk"] = matrix(H * D, C, 1.4)
            out[p + "mix.uv"] = matrix(H * E, C, 1.5)
            out[p + "mix.g"] = matrix(H * E, W, 2.0)
        else:
            G = m["kv_heads"]
            out[p + "mix.q"] = matrix(H * D, W, 1.4)
            out[p + "mix.k"] = matrix(G * D, W, 1.4)
            out[p + "mix.v"] = matrix(G * E, W, 1.5)
            if m.get("v_mix"):
                out[p + "mix.vmix"] = normal((), 0.2, 0.45)
        out[p + "mix.sink"] = normal((H,), 1.0, 1.0)
        out[p + "mix.o"] = matrix(W, H * E)
        mlp = layer.get("mlp")
        if mlp is not None:
            F = mlp["ff"]
            out[p + "norm2"] = normal((W,), 0.1, 0.9)
            for name in ("gate", "up"):
                out[p + f"mlp.{name}"] = matrix(F, W, 1.5)
                out[p + f"mlp.{name}.b"] = normal((F,), 0.5)
            out[p + "mlp.down"] = matrix(W, F)
            out[p + "mlp.down.b"] = normal((W,), 0.3)
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
    """A configuration drawn at random (seeded): head sizes and rows that the matrix-core kernels take and sizes that they do
    not, 1 to 17 query heads per key/value head, widths and vocabularies that are no multiple of 8, windows around the
    sizes of pages and tiles, any order of the two kinds of layer."""
    import random
    r = random.Random(seed)
    kv, vdim = r.choice([1, 2, 3]), r.choice([4, 12, 16, 32])          # shared by the layers that mix values
    layers = []
    for _ in range(r.randint(2, 5)):
        if r.random() < 0.5:
            dim, rot = r.choice([4, 8, 12, 16, 32]), r.choice([2, 4, 8, 16])
            entry = latent(r.choice([1, 2, 3, 6, 17]), dim, rot, r.choice([4, 5, 8, 16, 24]),
                           r.choice([6, 8, 16, 24, 40]), r.choice([1, 2, 3, 15, 16, 17, 31, 33, 63, 64, 65, 100, 500]),
                           r.choice([10.0, 1000.0, 300000.0]), r.choice([0.5, 1.0, 1.5]) * (dim + rot) ** -0.5)
        else:
            mixes = r.random() < 0.7
            g = kv if mixes else r.choice([1, 2])
            dim, size = r.choice([4, 8, 16, 20, 32, 48]), vdim if mixes else r.choice([4, 6, 16])
            dim = size if r.random() < 0.4 else dim                # (equal sizes: the kernels on the matrix cores)
            entry = biased(g * r.choice([1, 2, 3, 5, 17]), g, dim, size, r.choice([0.5, 1.0, 1.5]) * dim ** -0.5, r.choice([0.0, 0.1, 0.3]), r.choice([1, 2, 7, 16, 50]), mixes)
        layers.append(_with(entry, *((r.choice([16, 24, 50]), r.choice([0.5, 1.0, 4.0])) if r.random() < 0.8 else ())))
    return model(r.choice([33, 64, 90, 131]), r.choice([24, 40, 52, 64, 72, 100]), r.choice([1e-6, 1e-5, 1e-3]),
                 r.choice([2.0, 8.0, 30.0]), layers)
