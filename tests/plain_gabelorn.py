"""The Gabelorn decoder, plain and slow: whole sequences, no cache, no batch, one function per mechanism.

Written from the design's equations alone and sharing no code with the engine: its own reader of the model folder,
its own rotation, masks, biases. ``dtype`` is the float type everything is computed in (float64 by default).

The design in this file's notation (x the stream, h a sublayer's input, p a position counted from 0):

* x0 = E[token]; a layer: x += mixer(N1(x)); x += ff(N2(x)), the second only where the layer has a feed-forward;
  N(v) = v / sqrt(mean(v^2) + eps) * w.
* mixer "latent_attention": [c' | r'] = D h, c = N(c'), r = r' turned; k_h = [K_h c | r], v_h = V_h c, q_h = Q_h h with its
  last ``rot_dim`` entries turned; pairs (i, i + dims/2), angle p * base^(-2i / dims). Position i reads the last
  ``mask.size`` positions up to itself. The concatenated heads are multiplied entry by entry with sigmoid(G h).
* mixer "attention": grouped key/value heads, no rotation; q at position p times 1 + coef ln(floor((p + 1) / every) + 1);
  score q . k * scale - 2^(-8 (h + 1) / H) (i - j) over all j <= i. Where the layer mixes values: the first such layer's
  values v1 of the same token join, v <- (1 - lambda) v + lambda v1 (in all such layers but the first).
* both: the softmax of head h has one more term exp(z_h) in its denominator.
* feed-forward: g = min(G h + b, limit), u = clamp(U h + b', +-limit), D (g sigmoid(1.702 g) (u + 1)) + b''.
* logits = c tanh(A N_f(x) / c).
"""
from __future__ import annotations

import json
import math
import os
import struct

import torch


def read_folder(folder: str) -> tuple[dict, dict]:
    """config.json and every tensor of model.safetensors (read by hand: 8 bytes of length, a JSON header, the data)."""
    with open(os.path.join(folder, "config.json")) as f:
        config = json.load(f)
    with open(os.path.join(folder, "model.safetensors"), "rb") as f:
        (n,) = struct.unpack("<Q", f.read(8))
        header = json.loads(f.read(n))
        data = f.read()
    kinds = {"BF16": torch.bfloat16, "F32": torch.float32, "I32": torch.int32, "F16": torch.float16}
    tensors = {}
    for name, entry in header.items():
        if name == "__metadata__":
            continue
        lo, hi = entry["data_offsets"]
        t = torch.frombuffer(bytearray(data[lo:hi]), dtype=kinds[entry["dtype"]])
        tensors[name] = t.reshape(entry["shape"]).clone()
    return config, tensors


def rms_norm(v: torch.Tensor, w: torch.Tensor, eps: float) -> torch.Tensor:
    return v / torch.sqrt((v * v).mean(-1, keepdim=True) + eps) * w


def turn_halves(t: torch.Tensor, dims: int, base: float, positions: torch.Tensor) -> torch.Tensor:
    """t [n, heads, size]: pairs (i, i + dims / 2) of the first ``dims`` entries turn by position * base^(-2i / dims)."""
    half = dims // 2
    f = base ** (-2.0 * torch.arange(half, dtype=t.dtype) / dims)
    angle = positions.to(t.dtype)[:, None] * f[None, :]
    c, s = angle.cos()[:, None, :], angle.sin()[:, None, :]
    u, v = t[..., :half], t[..., half:dims]
    return torch.cat((u * c - v * s, v * c + u * s, t[..., dims:]), dim=-1)


def window_mask(n: int, size: int | None) -> torch.Tensor:
    """[n, n] True where query i reads key j: 0 <= i - j, and i - j < size where there is a window."""
    d = torch.arange(n)[:, None] - torch.arange(n)[None, :]
    return (d >= 0) & (d < size) if size is not None else d >= 0


def slopes(heads: int, dtype=torch.float64) -> torch.Tensor:
    return torch.tensor([2.0 ** (-8.0 * (h + 1) / heads) for h in range(heads)], dtype=dtype)


def distance_bias(n: int, heads: int, dtype=torch.float64) -> torch.Tensor:
    """[heads, n, n]: what is taken off the score of query i and key j."""
    d = (torch.arange(n)[:, None] - torch.arange(n)[None, :]).to(dtype)
    return slopes(heads, dtype)[:, None, None] * d[None]


def softmax_with_sink(s: torch.Tensor, sink: torch.Tensor, mask: torch.Tensor) -> torch.Tensor:
    """Weights over the last axis; the denominator also holds exp(sink)."""
    s = s.masked_fill(~mask, -math.inf)
    m = torch.maximum(s.max(dim=-1, keepdim=True).values, sink)
    e = torch.exp(s - m)
    return e / (e.sum(-1, keepdim=True) + torch.exp(sink - m))


def query_temperature(positions: torch.Tensor, coef: float, every: float, dtype=torch.float64) -> torch.Tensor:
    return torch.tensor([1.0 + coef * math.log(math.floor((int(p) + 1) / every) + 1) for p in positions], dtype=dtype)


def mixed_values(v: torch.Tensor, first: torch.Tensor, lam: torch.Tensor) -> torch.Tensor:
    return (1 - lam) * v + lam * first


def read_heads(q, k, v, scale, sink, mask, bias=None):
    """q [n, H, d], k [n, G, d], v [n, G, e] -> [n, H, e]; query head h reads key/value head h // (H / G)."""
    H, G = q.shape[1], k.shape[1]
    out = []
    for h in range(H):
        g = h // (H // G)
        s = (q[:, h] @ k[:, g].T) * scale
        if bias is not None:
            s = s - bias[h]
        out.append(softmax_with_sink(s, sink[h], mask) @ v[:, g])
    return torch.stack(out, dim=1)


def latent_attention(h: torch.Tensor, w: dict, m: dict, eps: float) -> torch.Tensor:
    n, H, D, R, E, C = h.shape[0], m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    pos = torch.arange(n)
    rot = m.get("rot") or {}
    q = (h @ w["q"].T).view(n, H, D + R)
    down = h @ w["dkv"].T
    c = rms_norm(down[:, :C], w["dkv.norm"], eps)
    q2, r = q[..., D:], down[:, None, C:]
    if R:
        q2, r = turn_halves(q2, rot["dims"], rot["base"], pos), turn_halves(r, rot["dims"], rot["base"], pos)
    k = torch.cat(((c @ w["uk"].T).view(n, H, D), r.expand(n, H, R)), dim=-1)
    v = (c @ w["uv"].T).view(n, H, E)
    mask = window_mask(n, (m.get("mask") or {}).get("size"))
    o = read_heads(torch.cat((q[..., :D], q2), dim=-1), k, v, m["scale"], w["sink"], mask).reshape(n, H * E)
    return (o * torch.sigmoid(h @ w["g"].T)) @ w["o"].T


def attention(h: torch.Tensor, w: dict, m: dict, kept: dict) -> torch.Tensor:
    """``kept``: where the first layer that mixes values leaves its own for the later ones."""
    n, H, G, D, E = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = (h @ w["q"].T).view(n, H, D)
    if m.get("q_temp"):
        q = q * query_temperature(torch.arange(n), m["q_temp"]["coef"], m["q_temp"]["every"], h.dtype)[:, None, None]
    k = (h @ w["k"].T).view(n, G, D)
    v = (h @ w["v"].T).view(n, G, E)
    if m.get("v_mix"):
        if "v" in kept:
            v = mixed_values(v, kept["v"], w["vmix"])
        else:
            kept["v"] = v
    o = read_heads(q, k, v, m["scale"], w["sink"], window_mask(n, None), distance_bias(n, H, h.dtype))
    return o.reshape(n, H * E) @ w["o"].T


def clamped_gate(g: torch.Tensor, u: torch.Tensor, limit: float) -> torch.Tensor:
    g, u = torch.clamp(g, max=limit), torch.clamp(u, -limit, limit)
    return g * torch.sigmoid(1.702 * g) * (u + 1)


def feed_forward(h: torch.Tensor, w: dict, limit: float) -> torch.Tensor:
    y = clamped_gate(h @ w["gate"].T + w["gate.b"], h @ w["up"].T + w["up.b"], limit)
    return y @ w["down"].T + w["down.b"]


def forward(config: dict, tensors: dict, tokens, dtype=torch.float64, streams: list | None = None) -> torch.Tensor:
    """Logits [len(tokens), vocab]. ``streams``, if a list, receives the stream after every layer."""
    W = {k: v.to(dtype) for k, v in tensors.items()}
    eps = config["norm"]["eps"]
    x = W["embed"][torch.tensor(tokens)]
    kept: dict = {}
    for i, layer in enumerate(config["layers"]):
        own = {k[len(f"l{i}."):]: v for k, v in W.items() if k.startswith(f"l{i}.")}
        mix = {k[len("mix."):]: v for k, v in own.items() if k.startswith("mix.")}
        h = rms_norm(x, own["norm1"], eps)
        if layer["type"] == "latent_attention":
            x = x + latent_attention(h, mix, layer["mixer"], eps)
        elif layer["type"] == "attention":
            x = x + attention(h, mix, layer["mixer"], kept)
        else:
            raise ValueError(layer["type"])
        mlp = layer.get("mlp")
        if mlp is not None:
            ff = {k[len("mlp."):]: v for k, v in own.items() if k.startswith("mlp.")}
            x = x + feed_forward(rms_norm(x, own["norm2"], eps), ff, mlp["limit"])
        if streams is not None:
            streams.append(x.clone())
    logits = rms_norm(x, W["final.norm"], eps) @ W["head"].T
    cap = config.get("logit_softcap")
    return cap * torch.tanh(logits / cap) if cap else logits


def greedy_generate(config: dict, tensors: dict, prompt, n: int, dtype=torch.float64) -> list[int]:
    """The ``n`` tokens that follow ``prompt`` when the most likely token is taken each time (the whole sequence is
    computed anew for every token)."""
    toks = list(prompt)
    for _ in range(n):
        toks.append(int(forward(config, tensors, toks, dtype)[-1].argmax()))
    return toks[len(prompt):]
