"""Attention over a cached latent: keys and values of all heads are made of one low-rank vector per token, and only
that vector (with an optional rotated key part that all heads share) is stored."""
from __future__ import annotations

import torch

from ..native import ops
from .base import MIXERS, CacheView, PagedKVNeed, ParamSpec, Part


@MIXERS.register("latent_attention")
class LatentAttention(Part):
    """Causal softmax attention whose keys and values come from a latent:

        c_q = rmsnorm(W_dq x),  q_h = W_uq,h c_q = [q_h' (``head_dim``) | q_h'' (``rot_dim``, turned by position)]
        c = rmsnorm(first ``kv_rank`` rows of W_dkv x),  r = the last ``rot_dim`` rows, turned by position
        k_h = [W_uk,h c | r],  v_h = W_uv,h c,  score = (q_h . k_h) * scale,  out = W_o [g_h softmax(score) v_h]_h

    with g_h = sigmoid(W_g x)_h if ``gated``. ``q_rank`` None: the queries have no latent, q_h = W_q,h x. A token stores the
    row [c | r] and nothing else. The products with
    W_uk and W_uv are moved to the query side, where they are made once per step's token instead of once per key:
    q_h . k_h = (W_uk,h^T q_h') . c + q_h'' . r, and sum_j p_j W_uv,h c_j = W_uv,h sum_j p_j c_j. So attention runs
    with one key/value head whose key is the stored row and whose value is the same row (``values_in_keys``); of the
    result the first ``kv_rank`` entries go through W_uv,h. Pairs of the rotated part, (2i, 2i + 1) or (i, i + rot_dim / 2)
    (``rotation`` "interleaved" or "halves"), turn by position * frequency i of ``position`` (an encoding that gives
    ``frequencies()`` and ``gain()``).
    ``window``: a query reads the last ``window`` positions up to its own. ``learned_sink``: the softmax's denominator has
    one more term exp(z_h), z a parameter per head. ``element_gate``: the concatenated heads are multiplied entry by entry
    with sigmoid(G x) (without a query latent; G is packed with the other projections of x).
    ``own_kv`` False: the layer has no W_dkv and reads the rows of the run-order entry it borrows from, with W_uk,
    W_uv, queries and output of its own; ``pad_dim``: entries of the lender's rows beyond this layer's ``kv_rank``
    (they meet zeros in the queries). ``row_multiple``: rows are filled with zeros up to a multiple of this (the kernels on
    the matrix cores take rows in steps of 16)."""

    def __init__(self, hidden_size: int, num_heads: int, head_dim: int, rot_dim: int, value_dim: int, q_rank: int | None,
                 kv_rank: int, scale: float, eps: float, gated: bool = False, own_kv: bool = True, pad_dim: int = 0,
                 position=None, window: int | None = None, learned_sink: bool = False, element_gate: bool = False,
                 rotation: str = "interleaved", row_multiple: int = 1):
        if (min(hidden_size, num_heads, head_dim, value_dim, kv_rank, row_multiple) <= 0 or (q_rank is not None and q_rank <= 0)
                or rot_dim < 0 or rot_dim % 2 or pad_dim < 0):
            raise ValueError("sizes must be positive, the rotated part even and not negative")
        if rot_dim and (position is None or not hasattr(position, "frequencies") or position.rotary_dim != rot_dim):
            raise ValueError(f"a rotated part of {rot_dim} entries needs a position encoding of that many frequencies")
        if not own_kv and (rot_dim or row_multiple != 1):
            raise ValueError("a layer that borrows its latent has no rotated key part and no rows of its own")
        if q_rank is None and (gated or not own_kv):
            raise ValueError("a layer without a query latent has a latent of its own and no gate per head")
        if element_gate and (gated or q_rank is not None):
            raise ValueError("a gate per entry goes with queries without a latent and without a gate per head")
        if rotation not in ("halves", "interleaved"):
            raise ValueError(f"rotation {rotation!r} is not known ('halves' and 'interleaved' are)")
        self.hidden_size, self.num_heads, self.head_dim, self.rot_dim = hidden_size, num_heads, head_dim, rot_dim
        self.value_dim, self.q_rank, self.kv_rank, self.scale, self.eps = value_dim, q_rank, kv_rank, scale, eps
        self.gated, self.own_kv, self.position, self.window = gated, own_kv, position, window or None
        self.learned_sink, self.element_gate, self.rotation = bool(learned_sink), bool(element_gate), rotation
        self.pad_dim = pad_dim + (-(kv_rank + rot_dim + pad_dim)) % row_multiple
        self.row = kv_rank + rot_dim + self.pad_dim               # what a token stores
        # rows of the packed projection of x: query latent or queries | latent and rotated key part | gates
        self.kv_off = num_heads * (head_dim + rot_dim) if q_rank is None else q_rank
        self.gate_off = self.kv_off + (kv_rank + rot_dim if own_kv else 0)
        self.down_rows = self.gate_off + (num_heads if gated else 0) + (num_heads * value_dim if element_gate else 0)
        self.sinks = None
        # the packed projection of a layer without a query latent gives rows of x's type, so x may come with its norm's
        # scaling left to do, which that product then makes (a product with a float32 result cannot)
        self.takes_deferred_norm = q_rank is None

    adds_to_residual = True       # the output projection can make the addition to the residual stream

    def first_product(self):
        """(weight, gated) of the product that x goes into."""
        return self.down_weight, False

    def param_specs(self):
        H = self.num_heads
        specs = {"down.weight": ParamSpec((self.down_rows, self.hidden_size)),
                 "uk.weight": ParamSpec((H * self.head_dim, self.kv_rank)),
                 "uv.weight": ParamSpec((H * self.value_dim, self.kv_rank)),
                 "o.weight": ParamSpec((self.hidden_size, H * self.value_dim))}
        if self.q_rank is not None:
            specs["q_norm.weight"] = ParamSpec((self.q_rank,), init="norm", always_float32=True)
            specs["uq.weight"] = ParamSpec((H * (self.head_dim + self.rot_dim), self.q_rank))
        if self.own_kv:
            specs["kv_norm.weight"] = ParamSpec((self.kv_rank,), init="norm", always_float32=True)
        if self.learned_sink:
            specs["sink"] = ParamSpec((H,), always_float32=True, init_mean=0.0, init_std=1.0)
        return specs

    def bind(self, params):
        self.down_weight, self.q_norm_weight = params["down.weight"], params.get("q_norm.weight")
        self.uq_weight, self.uv_weight = params.get("uq.weight"), params["uv.weight"]
        self.o_weight, self.kv_norm_weight, self.sinks = params["o.weight"], params.get("kv_norm.weight"), params.get("sink")
        # W_uk is used from its other side (W_uk,h^T q): the matrices are kept the way in which the product reads them
        H, D, C = self.num_heads, self.head_dim, self.kv_rank
        self.ukt_weight = params["uk.weight"].view(H, D, C).transpose(1, 2).contiguous().view(H * C, D)

    def cache_need(self):
        return PagedKVNeed(1, self.row, self.window, values_in_keys=True)

    def forward(self, x, step, cache: CacheView, add_to=None):
        if not self.own_kv and cache.writes:
            raise ValueError("a latent attention layer without a latent of its own must borrow another entry's cache")
        tables = step.groups[cache.group]
        T, H, D, R = x.shape[0], self.num_heads, self.head_dim, self.rot_dim
        writes = self.own_kv and cache.writes
        freqs = self.position.frequencies() if R else None
        gain = self.position.gain() if R else 1.0
        halves = self.rotation == "halves"
        a = ops.linear(x, self.down_weight, out_dtype=torch.float32 if self.q_rank is not None else None)
        rows_dtype = self.down_weight.dtype
        if self.q_rank is not None or writes:
            c_q = ops.latent_prepare(a, 0, self.q_rank or 0, self.kv_off, self.kv_rank, R, self.q_norm_weight, self.kv_norm_weight,
                                     self.eps, freqs, gain, step.token_positions, tables.slot_mapping if writes else None,
                                     cache.k if writes else None, rows_dtype, halves=halves)
        if self.q_rank is not None:
            q = ops.linear(c_q, self.uq_weight).view(T, H, D + R)
        else:
            q = a[:, :self.kv_off].unflatten(1, (H, D + R))       # (a view: the product that reads it takes rows any distance apart)
        # the query as the stored rows see it: [W_uk,h^T q_h' | q_h'' turned | zeros]
        make = torch.zeros if self.pad_dim else torch.empty
        q_row = make((T, H, self.row), dtype=rows_dtype, device=a.device)
        ops.head_gemm(q, self.ukt_weight, False, self.kv_rank, D, out=q_row,
                      turn=(R, D, self.kv_rank, freqs, gain, step.token_positions, halves) if R else None)
        mixed = ops.paged_attention(q_row, cache.k, cache.k, step.attention, tables.block_tables, self.scale, self.window,
                                    sink=self.sinks)
        gate = (a, self.gate_off) if self.gated else ((a, self.gate_off, "per entry") if self.element_gate else None)
        o = ops.head_gemm(mixed, self.uv_weight, False, self.value_dim, self.kv_rank, gate=gate)
        return ops.linear(o.view(T, H * self.value_dim), self.o_weight, add_to=add_to)
