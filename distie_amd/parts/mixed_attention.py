"""Softmax attention without rotation whose heads' scores are mixed ("talking heads", in front of the softmax: Shazeer
et al., "Talking-Heads Attention"), with a learned bias by distance and values that are the keys.

    q = W_q h + b_q (H heads),  k = W_k h + b_k (G heads; query head i uses i // (H / G)),  v = k as projected
    q, k <- x / sqrt(mean(x^2) + eps) for every head
    score_h = cap(q_h . k * scale) + rel[bucket(i - j), h],   cap(s) = score_cap * tanh(s / score_cap) (None: s itself)
    score_h <- sum_g talk[h, g] score_g
    weight = exp(score) / (exp(sink_score) + sum over the visible keys of exp(score))

Key j is visible to query i iff j <= i and (i - j < window or j < keep_first); without a window all j <= i are. The
distance n falls into bucket n up to half of the table's rows, `half` = rows / 2, then into logarithmically wider ones that
reach the table's end at bias_max: half + floor((rows - half) * log_(bias_max / half)(n / half)), at most rows - 1. The table is spread at load to one value
a distance, up to the distance from which on the last row holds (`distance_bias`). Scores, cap, bias, mixing and
softmax are float32 in either precision.

Both projections are one matrix product. The cache holds the normed keys and, as the values, the raw ones, with the
head size rounded up to what the kernels take (zeros in the places beyond).
"""

from __future__ import annotations

import bisect
import math

import torch

from ..config.model_config import PartSpec
from ..kernels.interface import ScoreExtras
from .attention import PagedKV, context_classes
from .base import Mixer, ParamSpec, register_part
from .conv_attention import padded_head_dim


def distance_bucket(n: int, rows: int, bias_max: float) -> int:
    """The row of a table of `rows` distance biases that a distance of n tokens has."""
    half = rows // 2
    if n < half:
        return n
    if half < 1 or bias_max <= half:             # no room for wider buckets: the last row
        return rows - 1
    place = math.log(n / half) / math.log(bias_max / half) * (rows - half)
    nearest = round(place)
    # a distance at which a bucket begins exactly must not fall short of it by a rounding of the logarithms
    whole = nearest if abs(place - nearest) < 1e-9 else math.floor(place)
    return min(rows - 1, half + whole)


def spread_distance_bias(table: torch.Tensor, bias_max: float) -> torch.Tensor:
    """A table [rows, H] of biases by bucket -> float32 [H, N], one value a distance; every distance of N - 1 and more
    has the last one."""
    rows = table.shape[0]
    buckets = [0]
    while buckets[-1] < rows - 1:
        buckets.append(distance_bucket(len(buckets), rows, bias_max))
    return table.float()[torch.tensor(buckets, dtype=torch.long, device=table.device)].t().contiguous()


class MixedHeadsAttention(Mixer):
    FIRST_CONTEXT = 1024

    def __init__(self, spec: PartSpec) -> None:
        super().__init__(spec)
        p = spec.params
        self.hidden_size = int(p["hidden_size"])
        self.num_heads = int(p["num_heads"])
        self.num_kv_heads = int(p["num_kv_heads"])
        self.head_dim = int(p["head_dim"])
        self.bias = bool(p.get("bias", True))
        self.scale = float(p["scale"])
        self.eps = float(p["eps"])
        self.window = p.get("window")
        self.keep_first = int(p.get("keep_first") or 0) if self.window is not None else 0
        self.score_cap = p.get("score_cap")
        self.bias_rows, self.bias_max = int(p["bias_rows"]), float(p["bias_max"])
        self.sink_score = p.get("sink_score")            # None: an ordinary softmax
        if self.num_heads % self.num_kv_heads:
            raise ValueError("num_heads must be a multiple of num_kv_heads")
        if self.bias_rows < 1:
            raise ValueError("the table of distance biases has at least one row")
        self.padded_dim = padded_head_dim(self.head_dim, self.head_dim)
        self.in_weight = self.in_bias = self.out_weight = self.ones = self.extras = None

    def cache_requirement(self):
        return PagedKV(self.num_kv_heads, self.padded_dim, self.window, self.keep_first)

    def param_specs(self):
        q, k, C = self.num_heads * self.head_dim, self.num_kv_heads * self.head_dim, self.hidden_size
        specs = {"q": ParamSpec((q, C)), "k": ParamSpec((k, C))}
        if self.bias:
            specs.update({"q.b": ParamSpec((q,)), "k.b": ParamSpec((k,))})
        specs.update({"rel": ParamSpec((self.bias_rows, self.num_heads)),
                      "talk": ParamSpec((self.num_heads, self.num_heads), "eye"), "o": ParamSpec((C, q))})
        return specs

    def load(self, tensors) -> None:
        q, k = tensors["q"], tensors["k"]
        dtype = torch.float32 if torch.float32 in (q.dtype, k.dtype) else q.dtype
        self.in_weight = torch.cat([q.to(dtype), k.to(dtype)], dim=0).contiguous()
        if self.bias:
            self.in_bias = torch.cat([tensors["q.b"].float(), tensors["k.b"].float()]).contiguous()
        self.out_weight = tensors["o"].contiguous()
        device = self.out_weight.device
        self.ones = torch.ones(self.head_dim, dtype=torch.float32, device=device)
        sinks = None if self.sink_score is None else torch.full((self.num_heads,), float(self.sink_score),
                                                                dtype=torch.float32, device=device)
        self.extras = ScoreExtras(score_cap=None if self.score_cap is None else float(self.score_cap), sinks=sinks,
                                  distance_bias=spread_distance_bias(tensors["rel"], self.bias_max),
                                  head_mix=tensors["talk"].float().contiguous(), keep_first=self.keep_first)

    def prepare(self, ops) -> None:
        ops.prepare_linear(self.in_weight, role="qkv")
        ops.prepare_linear(self.out_weight, role="attn_out")

    def capture_context(self, longest: int, limit: int):
        classes = context_classes(limit, self.FIRST_CONTEXT)
        return classes[min(bisect.bisect_left(classes, longest), len(classes) - 1)]

    def forward(self, ops, x, ctx, cache, writes_cache: bool):
        k_cache, v_cache = cache["k"], cache["v"]
        q = ops.conv_rope_kv_write(ops.linear(x, self.in_weight, self.in_bias), None, None, ctx.meta, cache.group, k_cache,
                                   v_cache, None, 1.0, self.num_heads, self.num_kv_heads, self.head_dim, self.head_dim,
                                   self.padded_dim, True, writes_cache, None, (self.ones, self.ones, self.eps),
                                   keys_are_values=True)
        mixed = ops.paged_attention(q, ctx.meta, cache.group, k_cache, v_cache, self.num_heads, self.num_kv_heads,
                                    self.padded_dim, self.scale, self.window, self.extras)
        if self.padded_dim != self.head_dim:
            mixed = ops.sigmoid_gate(mixed, self.num_heads, self.padded_dim, self.head_dim, None)
        return ops.linear(mixed, self.out_weight)


register_part("mixer", "mixed_heads_attention", MixedHeadsAttention)
