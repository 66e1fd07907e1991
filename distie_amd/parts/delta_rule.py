"""The gated delta rule (Yang, Kautz and Hatamizadeh, "Gated Delta Networks: Improving Mamba2 with Delta Rule"): a state
per head that forgets by a factor computed from the token and corrects what it holds under the token's key.

q and k (kv_heads heads of head_dim) and v (num_heads heads of value_dim) are projections of the mixer's input; every
channel of the three is filtered over time (`<q|k|v>.conv` [channels, taps], oldest row first; rows in front of a request's
first are zero) and goes through silu. num_heads / kv_heads value heads in a row share a q/k head. With k^ and q^ the
vectors of length one, x / sqrt(x . x + 1e-6), q^ times head_dim^(-1/2) besides, and two numbers a head and token,

    w = sigmoid(b),    b from W_b,        ln f = -exp(A_log) * softplus(a + dt_bias),    a from W_a,

a head's state S (head_dim x value_dim) goes from token t - 1 to t, and is read behind that, by

    S_t = f_t (1 - w_t k^_t k^_t^T) S_(t-1) + w_t k^_t v_t^T,        o_t = S_t^T q^_t:

what stood under k^_t is replaced, by the part w_t, with v_t. Every head's o goes through an RMS norm over its value_dim
columns (weight `norm` [value_dim], the same for all heads), then the gate's silu (from W_g), then `o`. For each request the
mixer keeps S, float32 [num_heads, head_dim, value_dim] and zero in the beginning, and the taps - 1 newest rows in front of
the filters. Everything behind the
projections and convolutions is float32 in either precision: unit norms, beta, the decay, the state and every sum into it,
the norm and the gate. The six projections are one matrix product: their weights are stacked at load (q, k, v, g, b, a, and
rows of zeros up to a multiple of 16).
"""

from __future__ import annotations

import torch

from ..config.model_config import PartSpec
from .base import FixedState, Mixer, ParamSpec, TensorDecl, register_part

UNIT_EPS = 1e-6        # inside the root that makes q and k unit vectors


class GatedDeltaRule(Mixer):
    STACKED = ("q", "k", "v", "g", "b", "a")

    def __init__(self, spec: PartSpec) -> None:
        super().__init__(spec)
        p = spec.params
        self.hidden_size = int(p["hidden_size"])
        self.num_heads = int(p["num_heads"])
        self.num_kv_heads = int(p.get("num_kv_heads") or self.num_heads)
        self.head_dim = int(p["head_dim"])
        self.value_dim = int(p.get("value_dim") or self.head_dim)
        self.taps = int(p["conv_taps"])
        self.eps = float(p["eps"])
        self.unit_eps = float(p.get("unit_eps", UNIT_EPS))
        self.q_scale = float(p.get("q_scale", self.head_dim ** -0.5))
        if self.num_heads % self.num_kv_heads:
            raise ValueError("delta rule: num_heads must be a multiple of num_kv_heads")
        if self.taps < 1:
            raise ValueError("the convolution has at least one tap")
        self.qk_width = self.num_kv_heads * self.head_dim
        self.inner = self.num_heads * self.value_dim
        self.conv_channels = 2 * self.qk_width + self.inner
        self.in_weight = self.conv_weight = self.a_log = self.dt_bias = self.norm_weight = self.out_weight = None

    def cache_requirement(self):
        tensors = [TensorDecl("state", (self.num_heads, self.head_dim, self.value_dim), torch.float32)]
        if self.taps > 1:
            tensors.append(TensorDecl("conv", (self.taps - 1, self.conv_channels), torch.float32))
        return FixedState(tuple(tensors))

    def _widths(self):
        return {"q": self.qk_width, "k": self.qk_width, "v": self.inner, "g": self.inner, "b": self.num_heads,
                "a": self.num_heads}

    def param_specs(self):
        C, H, widths = self.hidden_size, self.num_heads, self._widths()
        return {**{name: ParamSpec((widths[name], C)) for name in self.STACKED},
                **{name + ".conv": ParamSpec((widths[name], self.taps)) for name in "qkv"},
                "A_log": ParamSpec((H,)), "dt_bias": ParamSpec((H,)), "norm": ParamSpec((self.value_dim,), "ones"),
                "o": ParamSpec((C, self.inner))}

    def load(self, tensors) -> None:
        stacked = [tensors[name] for name in self.STACKED]
        dtype = torch.float32 if any(t.dtype == torch.float32 for t in stacked) else stacked[0].dtype
        rows = sum(t.shape[0] for t in stacked)
        if rows % 16:                                    # rows of the product that start at multiples of 16 bytes
            stacked.append(torch.zeros((-rows % 16, self.hidden_size), dtype=dtype, device=stacked[0].device))
        self.in_weight = torch.cat([t.to(dtype) for t in stacked], dim=0).contiguous()
        self.conv_weight = torch.cat([tensors[name + ".conv"] for name in "qkv"], dim=0).contiguous()
        self.a_log = tensors["A_log"].float().contiguous()
        self.dt_bias = tensors["dt_bias"].float().contiguous()
        self.norm_weight = tensors["norm"].float().contiguous()
        self.out_weight = tensors["o"].contiguous()

    def prepare(self, ops) -> None:
        ops.prepare_linear(self.in_weight, role="qkv")
        ops.prepare_linear(self.out_weight, role="attn_out")

    def forward(self, ops, x, ctx, cache, writes_cache: bool):
        H, channels = self.num_heads, self.conv_channels
        product = ops.linear_dense(x, self.in_weight)
        history = cache["conv"] if self.taps > 1 else None
        qkv = ops.causal_conv(product[:, :channels], self.conv_weight, history, ctx.meta, act="silu")
        behind = channels + self.inner
        mixed = ops.delta_scan(qkv, product[:, behind:behind + H], product[:, behind + H:behind + 2 * H], self.a_log,
                               self.dt_bias, cache["state"], ctx.meta, H, self.num_kv_heads, self.head_dim, self.value_dim,
                               self.q_scale, self.unit_eps)
        normed = ops.rmsnorm_gate(mixed, self.norm_weight, self.eps, product[:, channels:behind], ctx.act_dtype,
                                  group=self.value_dim, gate="silu")
        return ops.linear(normed, self.out_weight)


register_part("mixer", "gated_delta_rule", GatedDeltaRule)
