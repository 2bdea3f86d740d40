"""Plain, slow, whole-sequence Zigelorn decoder on the CPU: the oracle of the tests of this design.

No cache, no batching, no kernels and no code of the package: every function takes a whole sequence and writes
one mechanism out as loops and small tensor expressions. ``logits(config, tensors, tokens)`` runs a model
folder's contents (``read_model_folder``); ``dtype`` may be ``torch.float64`` for a sharper oracle.

Notation: T tokens, W the model's width, H heads, G key heads, D the query/key head size, E the value head size, p a
token's index in its sequence.
"""
from __future__ import annotations

import json
import math
import os

import torch


def read_model_folder(folder: str):
    """config.json as a dict and every tensor of model.safetensors (floats as float32)."""
    from safetensors import safe_open

    with open(os.path.join(folder, "config.json")) as f:
        config = json.load(f)
    tensors = {}
    with safe_open(os.path.join(folder, "model.safetensors"), framework="pt", device="cpu") as f:
        for name in f.keys():
            t = f.get_tensor(name)
            tensors[name] = t.to(torch.float32) if t.is_floating_point() else t
    return config, tensors


# ------------------------------------------------------------------ small pieces
def over_rms(x: torch.Tensor, eps: float) -> torch.Tensor:
    """x over its root mean square along the last axis, eps under the root."""
    return x / torch.sqrt(x.pow(2).mean(-1, keepdim=True) + eps)


def zero_centred_norm(x: torch.Tensor, weight: torch.Tensor, eps: float) -> torch.Tensor:
    """The norm whose weight is stored as its distance from one."""
    return over_rms(x, eps) * (1.0 + weight)


def silu(z):
    return z * torch.sigmoid(z)


def gelu_tanh(z):
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def pair_frequencies(dims: int, base: float, scaling: dict | None, dtype) -> tuple[torch.Tensor, float]:
    """([dims / 2] turns per position, the factor of cosines and sines). With ``scaling`` pairs that turn fast keep their
    frequency, pairs that turn slowly have it divided by ``factor``, and between the two a ramp leads over."""
    i = torch.arange(dims // 2, dtype=torch.float64)
    f = float(base) ** (-2.0 * i / dims)
    if not scaling:
        return f.to(dtype), 1.0

    def pair_with(turns: float) -> float:        # which pair turns so often over ``original`` positions
        return dims * math.log(scaling["original"] / (turns * 2.0 * math.pi)) / (2.0 * math.log(base))

    low = max(math.floor(pair_with(scaling["fast"])), 0)
    high = min(math.ceil(pair_with(scaling["slow"])), dims - 1)
    share = torch.clamp((i - low) / max(high - low, 0.001), 0.0, 1.0)
    return (share * f / scaling["factor"] + (1.0 - share) * f).to(dtype), 1.0 + 0.1 * math.log(scaling["factor"])


def turn(x: torch.Tensor, rot: dict | None) -> torch.Tensor:
    """x[T, heads, size]: coordinates i and i + dims / 2 (i < dims / 2) of every head are a pair, turned by p f_i; the
    coordinates from dims on pass."""
    dims = (rot or {}).get("dims", 0)
    if not dims:
        return x
    f, gain = pair_frequencies(dims, rot["base"], rot.get("scaling"), torch.float64)
    a = torch.arange(x.shape[0], dtype=torch.float64)[:, None] * f
    c, s = (gain * a.cos()).to(x.dtype)[:, None], (gain * a.sin()).to(x.dtype)[:, None]
    r = dims // 2
    u, v = x[..., :r], x[..., r:dims]
    return torch.cat((u * c - v * s, v * c + u * s, x[..., dims:]), dim=-1)


def windowed_softmax(q, k, v, scale: float, window: int | None) -> torch.Tensor:
    """q[T, H, D], k[T, G, D], v[T, G, E] -> [T, H, E]; query i sees the keys j with 0 <= i - j < window."""
    T, H, _ = q.shape
    per = H // k.shape[1]
    back = torch.arange(T)[:, None] - torch.arange(T)[None, :]
    hidden = (back < 0) | ((back >= window) if window else torch.zeros_like(back, dtype=torch.bool))
    out = []
    for h in range(H):
        s = (q[:, h] @ k[:, h // per].T * scale).masked_fill(hidden, -math.inf)
        out.append(torch.softmax(s, dim=-1) @ v[:, h // per])
    return torch.stack(out, dim=1)


def decayed_memory(q, k, v, decay) -> torch.Tensor:
    """Per head S <- decay_h S + k_t v_t^T from zero, read after the write: S^T q_t. q, k [T, H, D], v [T, H, E]."""
    T, H, D = q.shape
    out = torch.zeros(T, H, v.shape[-1], dtype=q.dtype)
    for h in range(H):
        S = torch.zeros(D, v.shape[-1], dtype=q.dtype)
        for t in range(T):
            S = decay[h] * S + torch.outer(k[t, h], v[t, h])
            out[t, h] = S.T @ q[t, h]
    return out


def bonus_memory(r, k, v, w, u) -> torch.Tensor:
    """Per head, from S = 0: o_t = (S + diag(u) k_t v_t^T)^T r_t, then S <- diag(w_t) S + k_t v_t^T. r, k, w [T, H, D],
    u [H, D], v [T, H, E]."""
    T, H, D = r.shape
    out = torch.zeros(T, H, v.shape[-1], dtype=r.dtype)
    for h in range(H):
        S = torch.zeros(D, v.shape[-1], dtype=r.dtype)
        for t in range(T):
            kv = torch.outer(k[t, h], v[t, h])
            out[t, h] = (S + u[h][:, None] * kv).T @ r[t, h]
            S = w[t, h][:, None] * S + kv
    return out


def shifted(x: torch.Tensor) -> torch.Tensor:
    """The row before each row; zeros before the first."""
    return torch.cat((torch.zeros_like(x[:1]), x[:-1]), dim=0)


# ------------------------------------------------------------------ mixers
def attention(x, w, p, m, eps):
    T, H, G, D = x.shape[0], m["heads"], m["kv_heads"], m["dim"]
    q = x @ w[p + "q"].T + w[p + "q.b"]
    k = x @ w[p + "k"].T + w[p + "k.b"]
    v = k.view(T, G, D)
    q = turn((over_rms(q, eps) * w[p + "q.norm"]).view(T, H, D), m.get("rot"))
    k = turn((over_rms(k, eps) * w[p + "k.norm"]).view(T, G, D), m.get("rot"))
    o = windowed_softmax(q, k, v, m["scale"], (m.get("mask") or {}).get("size"))
    o = o * torch.sigmoid(x @ w[p + "g"].T)[..., None]
    return o.reshape(T, H * D) @ w[p + "o"].T


def retention(x, w, p, m, eps):
    T, H, D, E = x.shape[0], m["heads"], m["dim"], m["vdim"]
    q = turn((x @ w[p + "q"].T).view(T, H, D), m.get("rot"))
    k = turn((x @ w[p + "k"].T).view(T, H, D), m.get("rot")) * D ** -0.5
    v = (x @ w[p + "v"].T).view(T, H, E)
    o = over_rms(decayed_memory(q, k, v, m["decay"]), eps).reshape(T, H * E)
    return (o * silu(x @ w[p + "g"].T)) @ w[p + "o"].T


def wkv(x, w, p, m, eps):
    T, H, D = x.shape[0], m["heads"], m["dim"]
    before = shifted(x)
    mixed = {n: x + (before - x) * w[p + "mu." + n] for n in "rkvgw"}
    r, k, v = ((mixed[n] @ w[p + n].T).view(T, H, D) for n in "rkv")
    gate = silu(mixed["g"] @ w[p + "g"].T)
    lin = torch.tanh(mixed["w"] @ w[p + "w1"].T) @ w[p + "w2"].T + w[p + "w0"]
    decay = torch.exp(-torch.exp(lin)).view(T, H, D)
    o = over_rms(bonus_memory(r, k, v, decay, w[p + "u"].view(H, D)), eps).reshape(T, H * D)
    return (o * w[p + "norm"] * gate) @ w[p + "o"].T


MIXERS = {"attention": attention, "retention": retention, "wkv": wkv}


# ------------------------------------------------------------------ feed-forwards
def dense(x, w, p):
    return gelu_tanh(x @ w[p + "up"].T) @ w[p + "down"].T


def choose(logits: torch.Tensor, correction: torch.Tensor, top: int, count: int, keep: int):
    """One token: (numbers of its ``top`` experts, all scores). The choice is by score plus correction among the
    experts of the ``keep`` groups whose best choice score is largest."""
    s = torch.softmax(logits, dim=-1)
    c = s + correction
    size = c.numel() // count
    best = [float(c[g * size:(g + 1) * size].max()) for g in range(count)]
    kept = sorted(range(count), key=lambda g: -best[g])[:keep]
    open_ = [e for g in kept for e in range(g * size, (g + 1) * size)]
    return sorted(open_, key=lambda e: -float(c[e]))[:top], s


def experts(x, w, p, mlp):
    r = mlp["router"]
    groups = r.get("groups") or {"count": 1, "keep": 1}
    z = x @ w[p + "router"].T
    out = torch.zeros_like(x)
    for t in range(x.shape[0]):
        chosen, s = choose(z[t], w[p + "correction"], r["top"], groups["count"], groups["keep"])
        for e in chosen:
            y = x[t]
            if e < r["experts"]:
                y = w[p + f"e{e}.down"] @ torch.relu(w[p + f"e{e}.up"] @ x[t]) ** 2
            out[t] += s[e] * y
    return out


# ------------------------------------------------------------------ the model
def hidden_states(config: dict, tensors: dict, tokens, dtype=torch.float32) -> list[torch.Tensor]:
    """[the embedding's rows, the stream after every layer run], each [T, W]."""
    w = {k: (t.to(dtype) if t.is_floating_point() else t) for k, t in tensors.items()}
    eps = config["norm"]["eps"]
    x = w["embed"][torch.as_tensor(tokens, dtype=torch.long)]
    out = [x]
    for i, layer in enumerate(config["layers"]):
        p = f"l{layer.get('weights_of', i)}."
        y = MIXERS[layer["type"]](zero_centred_norm(x, w[p + "norm1"], eps), w, p + "mix.", layer["mixer"], eps)
        x = x + zero_centred_norm(y, w[p + "norm1b"], eps)
        mlp = layer.get("mlp")
        if mlp is not None:
            h = zero_centred_norm(x, w[p + "norm2"], eps)
            y = dense(h, w, p + "mlp.") if mlp["kind"] == "dense" else experts(h, w, p + "mlp.", mlp)
            x = x + zero_centred_norm(y, w[p + "norm2b"], eps)
        out.append(x)
    return out


def logits(config: dict, tensors: dict, tokens, dtype=torch.float32) -> torch.Tensor:
    """[T, vocab]: the last norm, then the embedding table itself as the head."""
    x = hidden_states(config, tensors, tokens, dtype)[-1]
    x = zero_centred_norm(x, tensors["final.norm"].to(dtype), config["norm"]["eps"])
    return x @ tensors["embed"].to(dtype).T


def greedy_generate(config, tensors, prompt, n: int) -> list[int]:
    ids = list(prompt)
    for _ in range(n):
        ids.append(int(logits(config, tensors, ids)[-1].argmax()))
    return ids[len(prompt):]
