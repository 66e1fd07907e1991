"""Time mixing with a data-dependent decay (the recurrence of RWKV-6: Peng et al., "Eagle and Finch: RWKV with
Matrix-Valued States and Dynamic Recurrence").

x_t is what the mixer reads (x_(-1) = 0). The five projections read it blended with the row in front of it, every channel
at a rate of its own: b_s = (1 - mu_s) x_t + mu_s x_(t-1) for s = r, k, v, g, w. With [H, D] vectors

    r = R b_r,   k = K b_k,   v = V b_v,   gate = silu(G b_g),   keep = exp(-exp(w0 + W2 tanh(W1 b_w)))

(keep in (0, 1), one for every head and key channel d) a head computes, a column e of its state M at a time,

    y[e] = sum_d r[d] (M[d][e] + u[d] k[d] v[e])        the current token counts with a bonus u
    M[d][e] <- keep[d] M[d][e] + k[d] v[e]

y / sqrt(mean(y^2) + eps), all heads side by side, times a weight and the gate, is projected back to the width. A request's state is M
(float32 [heads, dim, dim], zero at the start) and its last x (float32). The decay, its exponentials, M and its sums, norm and gate are float32 in either precision.
"""

from __future__ import annotations

import torch

from ..config.model_config import PartSpec
from .base import FixedState, Mixer, ParamSpec, TensorDecl, register_part


class WKV(Mixer):
    MIXES = ("r", "k", "v", "g", "w")

    def __init__(self, spec: PartSpec) -> None:
        super().__init__(spec)
        p = spec.params
        self.hidden_size = int(p["hidden_size"])
        self.num_heads = int(p["num_heads"])
        self.head_dim = int(p["head_dim"])
        self.decay_rank = int(p["decay_rank"])
        self.eps = float(p["eps"])
        if self.decay_rank < 1:
            raise ValueError("the decay's projection has at least one dimension")
        self.inner = self.num_heads * self.head_dim
        self.mu = self.weights = self.up_weight = self.up_bias = self.bonus = self.norm_weight = self.out_weight = None

    def cache_requirement(self):
        return FixedState((TensorDecl("state", (self.num_heads, self.head_dim, self.head_dim), torch.float32),
                           TensorDecl("last", (self.hidden_size,), torch.float32)))

    def param_specs(self):
        C, N, R = self.hidden_size, self.inner, self.decay_rank
        return {**{f"mu.{name}": ParamSpec((C,)) for name in self.MIXES},
                **{name: ParamSpec((N, C)) for name in "rkvg"},
                "w1": ParamSpec((R, C)), "w2": ParamSpec((N, R)), "w0": ParamSpec((N,)),
                "u": ParamSpec((self.num_heads, self.head_dim)), "norm": ParamSpec((N,), "ones"), "o": ParamSpec((C, N))}

    def load(self, tensors) -> None:
        self.mu = torch.stack([tensors[f"mu.{name}"].float() for name in self.MIXES]).contiguous()
        self.weights = tuple(tensors[name].contiguous() for name in ("r", "k", "v", "g", "w1"))
        self.up_weight, self.up_bias = tensors["w2"].float().contiguous(), tensors["w0"].float().contiguous()
        self.bonus = tensors["u"].float().reshape(-1).contiguous()
        self.norm_weight = tensors["norm"].float().contiguous()
        self.out_weight = tensors["o"].contiguous()

    def prepare(self, ops) -> None:
        ops.prepare_linear_each(self.weights)
        ops.prepare_linear(self.out_weight, role="attn_out")

    def shift(self, cache):
        """What the token shift in front of this mixer takes, for an arrangement that runs it along with its own read of
        the residual (`forward_mixed` is handed the result): (mu, the state it keeps)."""
        return self.mu, cache["last"]

    def forward(self, ops, x, ctx, cache, writes_cache: bool):
        return self.forward_mixed(ops, ops.token_shift(x, *self.shift(cache), ctx.meta), ctx, cache)

    def forward_mixed(self, ops, mixes, ctx, cache):
        r, k, v, gates, low = ops.linear_each(mixes, self.weights, unrounded=(4,))
        mixed = ops.wkv_mix(r, k, v, gates, low, self.up_weight, self.up_bias, self.bonus, cache["state"], ctx.meta,
                            self.num_heads, self.head_dim, self.norm_weight, self.eps, ctx.act_dtype)
        return ops.linear(mixed, self.out_weight)


register_part("mixer", "wkv", WKV)
