"""Norms. ``RMSNorm`` follows nanovllm/layers/layernorm.py:16-40."""
from __future__ import annotations

import torch

from ..native import ops
from .base import NORMS, ParamSpec, Part


@NORMS.register("rmsnorm")
class RMSNorm(Part):
    """y = x / sqrt(mean(x^2) + eps) * weight; with a residual the sum is normed
    and carried on (layernorm.py:28-40)."""

    takes_summed = True           # ``forward_add`` takes an ``ops.Summed`` (a sum that a product has made already)
    defers_to_products = True     # ``forward_add(..., deferred=True)`` may return an ``ops.Normed``

    def __init__(self, size: int, eps: float, residual_float32: bool = True, rounds_between: bool = True):
        """``residual_float32`` (an engine option, offered to every part when a model is built): True: the residual
        stream is carried in float32 whatever the rows' element type, so the sum goes from layer to layer
        unrounded. False: it is carried in the rows' element type, rounded after every addition, as the
        reference carries it (layernorm.py:34-40; the norm itself still takes the unrounded float sum).
        ``rounds_between``: the normed row is rounded before it meets the weight and once more after it, as the
        reference does (layernorm.py:22-25); False: the weight joins in float and the row is rounded once."""
        self.size = size
        self.eps = eps
        self.residual_float32 = bool(residual_float32)
        self.rounds_between = bool(rounds_between)
        self.weight = None

    def param_specs(self):
        return {"weight": ParamSpec((self.size,), init="norm", keeps_float32=True)}

    def forward_start(self, x: torch.Tensor):
        """The first norm of a model: returns (norm(x), x as the residual that later norms add to)."""
        return ops.rmsnorm(x, self.weight, self.eps, start_residual=True, residual_float32=self.residual_float32,
                           rounds_between=self.rounds_between)

    def forward(self, x) -> torch.Tensor:
        return ops.rmsnorm(ops.dense(x), self.weight, self.eps, rounds_between=self.rounds_between)

    def add_to(self, residual: torch.Tensor, reader=None) -> ops.AddTo:
        """What the part before this norm is handed so that its last product can make the addition to ``residual``
        and this norm's product with its weight (``forward_add`` then gets an ``ops.Summed``). ``reader``: the part
        that reads this norm, if it says what its first product is (``first_product()``)."""
        first = getattr(reader, "first_product", None)
        return ops.AddTo(residual, self.weight, self.eps, first() if first is not None else None)

    def forward_add(self, x, residual: torch.Tensor, deferred: bool = False):
        """Returns (norm(x + residual), x + residual); ``residual`` is updated in place. ``x`` may be the
        ``ops.Summed`` that a product made from this norm's ``add_to``: the sum is in ``residual`` already, and what
        is left of the norm is the scaling of the rows. ``deferred``: the caller's next step is a product, which
        scales its rows itself; it then gets an ``ops.Normed`` in place of a tensor."""
        if isinstance(x, ops.Summed):
            if x.norm_weight is not self.weight or x.residual is not residual:
                raise ValueError("a sum that a product made for another norm, or into another residual stream")
            normed = ops.Normed(x)
            return (normed if deferred else normed.tensor()), residual
        y = ops.rmsnorm(x, self.weight, self.eps, residual=residual, rounds_between=self.rounds_between)
        return y, residual


@NORMS.register("scalar_rmsnorm")
class ScalarRMSNorm(Part):
    """y = x / sqrt(mean(x^2) + eps) * g with one number g for all coordinates. Statistics and the weight are
    float32; the rows that come in and go out may differ in element type (``forward(x, out_dtype)``)."""

    def __init__(self, eps: float, output: str = "same"):
        """``output``: the element type of the result where ``forward`` is not told: "same" as the input,
        "float32" (a stream carried in float32), or "rows" (the model's element type for rows)."""
        if output not in ("same", "float32", "rows"):
            raise ValueError(f"output must be 'same', 'float32' or 'rows', got {output!r}")
        self.eps, self.output = eps, output
        self.weight = None
        self.row_dtype = None         # set when the model's weights are bound

    def param_specs(self):
        return {"weight": ParamSpec((), init="norm", always_float32=True)}

    def forward(self, x, out_dtype=None) -> torch.Tensor:
        if out_dtype is None:
            out_dtype = {"same": x.dtype, "float32": torch.float32, "rows": self.row_dtype or x.dtype}[self.output]
        return ops.scalar_rmsnorm(x, self.weight, self.eps, out_dtype=out_dtype)


@NORMS.register("layernorm")
class LayerNorm(Part):
    """y = (x - mean) / sqrt(variance + eps) * weight + bias over the width, the variance being the mean of the squared
    deviations. It reads a float32 stream and gives rows of the model's element type; statistics, weight and bias
    are float32. Two such norms of one stream share their statistics: ``ops.layernorm_pair`` takes both at once (see
    the block ``parallel_two_norms``)."""

    def __init__(self, size: int, eps: float):
        self.size, self.eps = size, eps
        self.weight = self.bias = None
        self.row_dtype = None         # set when the model's weights are bound

    def param_specs(self):
        return {"weight": ParamSpec((self.size,), init="norm", always_float32=True),
                "bias": ParamSpec((self.size,), init="zeros", always_float32=True)}

    def forward(self, x, out_dtype=None) -> torch.Tensor:
        if x.dtype != torch.float32:
            x = x.float()
        y, _ = ops.layernorm_pair(x, (self.weight, self.bias), None, self.eps, out_dtype or self.row_dtype or torch.float32)
        return y


@NORMS.register("stream_rmsnorm")
class StreamRMSNorm(Part):
    """y = x / sqrt(mean(x^2) + eps) * weight of a float32 stream, given as rows of the model's element type;
    statistics and weight are float32. A block that carries several streams reads this norm's weight and eps and
    takes the norm in its own kernel (``ops.streams_step``); ``forward`` is the same for one stream. ``zero_centred``: the
    stored weight is its distance from one (one is added, in float32, when the weights are bound)."""

    def __init__(self, size: int, eps: float, zero_centred: bool = False):
        self.size, self.eps, self.zero_centred = size, eps, bool(zero_centred)
        self.weight = None
        self.row_dtype = None         # set when the model's weights are bound

    def param_specs(self):
        if self.zero_centred:
            return {"weight": ParamSpec((self.size,), always_float32=True, init_mean=0.0, init_std=0.1)}
        return {"weight": ParamSpec((self.size,), init="norm", always_float32=True)}

    def bind(self, params):
        self.weight = params["weight"] + 1.0 if self.zero_centred else params["weight"]

    def forward(self, x, out_dtype=None) -> torch.Tensor:
        if x.dtype != torch.float32:
            x = x.float()
        rows, width = x.shape
        y, _ = ops.streams_step(x.view(1, rows, width), rows, width, 1, out_dtype or self.row_dtype or torch.float32,
                                read=(None, self.weight, self.eps))
        return y
