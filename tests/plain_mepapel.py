"""The Mepapel decoder in the plainest way: float64, whole sequences, one function for each mechanism, loops where a
loop says it best. It shares no code with the package; the tests compare the engine with it.

Notation: T tokens, C the model width, rms(v) = v / sqrt(mean(v^2) + eps). Weights come as a dict by checkpoint name,
linear weights [out, in]."""

from __future__ import annotations

import math

import torch


def rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def silu(z):
    return z * torch.sigmoid(z)


def softplus(z):
    return torch.clamp(z, min=0) + torch.log1p(torch.exp(-z.abs()))


def short_conv(u, filters, bias=None):
    """u [T, N], filters [N, taps] (the last column meets the current row); zeros in front of the first row."""
    taps = filters.shape[1]
    full = torch.cat([torch.zeros(taps - 1, u.shape[1], dtype=u.dtype), u])
    out = torch.stack([(full[t:t + taps] * filters.T).sum(0) for t in range(u.shape[0])])
    return out if bias is None else out + bias


def rotate(x, rot, neighbours):
    """x [T, H, D], row t at position t: the first rot.dims dimensions turned, pair (2i, 2i + 1) or (i, i + dims / 2)."""
    T, dims = x.shape[0], int(rot["dims"])
    out = x.clone()
    for i in range(dims // 2):
        angle = torch.arange(T, dtype=torch.float64) * float(rot["base"]) ** (-2.0 * i / dims)
        cos, sin = torch.cos(angle)[:, None], torch.sin(angle)[:, None]
        a, b = (2 * i, 2 * i + 1) if neighbours else (i, i + dims // 2)
        out[..., a] = x[..., a] * cos - x[..., b] * sin
        out[..., b] = x[..., b] * cos + x[..., a] * sin
    return out


def visible(T, mask):
    """[T, T] (query, key): which keys a query sees. A key must lie in the query's own chunk of `size` positions."""
    i, j = torch.arange(T)[:, None], torch.arange(T)[None, :]
    seen = j <= i
    if mask:
        size = int(mask["size"])
        seen = seen & (i // size == j // size)
    return seen


def softmax_attention(q, k, v, scale, seen):
    """q [T, H, D], k [T, G, D], v [T, G, E] -> [T, H, E]."""
    H, G = q.shape[1], k.shape[1]
    heads = []
    for h in range(H):
        g = h // (H // G)
        scores = (q[:, h] @ k[:, g].T * scale).masked_fill(~seen, -math.inf)
        heads.append(torch.softmax(scores, -1) @ v[:, g])
    return torch.stack(heads, 1)


def attention(h, w, p, m, eps):
    """The left mixer of a parallel layer."""
    T = h.shape[0]
    H, G, D, E = int(m["heads"]), int(m["kv_heads"]), int(m["dim"]), int(m["vdim"])
    q, k, v = (h @ w[p + n].T + w[p + n + ".b"] for n in "qkv")
    if m.get("conv"):
        q, k, v = (short_conv(u, w[p + n + ".conv"]) for n, u in zip("qkv", (q, k, v)))
    q = rms(q.view(T, H, D), eps) * w[p + "q.norm"]
    k = rms(k.view(T, G, D), eps) * w[p + "k.norm"]
    if m.get("rot"):
        q, k = rotate(q, m["rot"], True), rotate(k, m["rot"], True)
    out = softmax_attention(q, k, v.view(T, G, E), float(m["scale"]), visible(T, m.get("mask")))
    return out.reshape(T, H * E) @ w[p + "o"].T + w[p + "o.b"]


def retention_scan(q, k, v, decay):
    """q, k [T, H, D], v [T, H, E], one decay a head -> [T, H, E]."""
    T, H, D = q.shape
    state = torch.zeros(H, D, v.shape[2], dtype=torch.float64)
    out = []
    for t in range(T):
        state = decay[:, None, None] * state + k[t][:, :, None] * v[t][:, None, :]
        out.append((state * q[t][:, :, None]).sum(1))
    return torch.stack(out)


def retention(h, w, p, m, eps, watch=None):
    """The right mixer of a parallel layer."""
    T = h.shape[0]
    H, D, E = int(m["heads"]), int(m["dim"]), int(m["vdim"])
    q, k = (h @ w[p + n].T for n in "qk")
    q, k, v = q.view(T, H, D), k.view(T, H, D), (h @ w[p + "v"].T).view(T, H, E)
    if m.get("rot"):
        q, k = rotate(q, m["rot"], False), rotate(k, m["rot"], False)
    k = k * D ** -0.5
    decay = torch.tensor([float(d) for d in m["decay"]], dtype=torch.float64)
    o = retention_scan(q, k, v, decay)
    if watch is not None:
        watch("heads", o, retention_scan(q ** 2, k ** 2, v ** 2, decay ** 2))
    return (rms(o, eps).reshape(T, H * E) * silu(h @ w[p + "g"].T)) @ w[p + "o"].T


def parallel(h, w, p, m, eps, watch=None):
    left = attention(h, w, p + "left.", m["left"], eps)
    right = retention(h, w, p + "right.", m["right"], eps, watch)
    return 0.5 * (rms(left, eps) * w[p + "left.out"] + rms(right, eps) * w[p + "right.out"])


def ssd_scan(x, B, C, d, rate, skip):
    """x [T, H, P], B and C [T, H, N], step sizes d [T, H], rate = exp(A_log) [H], skip [H] -> [T, H, P]."""
    T, H, P = x.shape
    state = torch.zeros(H, B.shape[2], P, dtype=torch.float64)
    out = []
    for t in range(T):
        state = torch.exp(-rate * d[t])[:, None, None] * state + d[t][:, None, None] * B[t][:, :, None] * x[t][:, None, :]
        out.append((state * C[t][:, :, None]).sum(1) + skip[:, None] * x[t])
    return torch.stack(out)


def mamba2(h, w, p, m, eps, watch=None):
    T = h.shape[0]
    H, P, N, G = int(m["heads"]), int(m["vdim"]), int(m["state"]), int(m["groups"])
    inner = H * P
    z, xbc, dt = torch.split(h @ w[p + "in"].T, [inner, inner + 2 * G * N, H], 1)
    x, B, C = torch.split(silu(short_conv(xbc, w[p + "conv"], w[p + "conv.b"])), [inner, G * N, G * N], 1)
    own = lambda u: torch.stack([u.view(T, G, N)[:, i // (H // G)] for i in range(H)], 1)
    y = ssd_scan(x.reshape(T, H, P), own(B.contiguous()), own(C.contiguous()), softplus(dt + w[p + "dt_bias"]),
                 torch.exp(w[p + "A_log"]), w[p + "D"])
    parts = int(m["norm_groups"])
    y = rms((y.reshape(T, inner) * silu(z)).view(T, parts, inner // parts), eps).reshape(T, inner) * w[p + "norm"]
    return y @ w[p + "o"].T


def delta_scan(q, k, v, beta, g):
    """q, k [T, H, D] (unit vectors, q scaled), v [T, H, E], beta and g [T, H] -> [T, H, E]."""
    T, H, D = q.shape
    out = torch.zeros(T, H, v.shape[2], dtype=torch.float64)
    for head in range(H):
        S = torch.zeros(D, v.shape[2], dtype=torch.float64)
        for t in range(T):
            S = g[t, head] * S
            u = beta[t, head] * (v[t, head] - S.T @ k[t, head])
            S = S + torch.outer(k[t, head], u)
            out[t, head] = S.T @ q[t, head]
    return out


def write_squares(q, k, v, beta, g):
    """The sum of the squares of what the tokens so far would add to an output without corrections."""
    T, H, D = q.shape
    state = torch.zeros(H, D, v.shape[2], dtype=torch.float64)
    out = []
    for t in range(T):
        write = beta[t][:, None] * v[t]
        state = (g[t] ** 2)[:, None, None] * state + (k[t] ** 2)[:, :, None] * (write ** 2)[:, None, :]
        out.append((state * (q[t] ** 2)[:, :, None]).sum(1))
    return torch.stack(out)


def delta(h, w, p, m, eps, watch=None):
    T = h.shape[0]
    H, G, D, E = int(m["heads"]), int(m["kv_heads"]), int(m["dim"]), int(m["vdim"])
    q, k, v = (silu(short_conv(h @ w[p + n].T, w[p + n + ".conv"])) for n in "qkv")
    unit = lambda u: u / torch.sqrt((u * u).sum(-1, keepdim=True) + 1e-6)
    q, k = unit(q.view(T, G, D)) * D ** -0.5, unit(k.view(T, G, D))
    own = lambda u: torch.stack([u[:, i // (H // G)] for i in range(H)], 1)
    beta = torch.sigmoid(h @ w[p + "b"].T)
    g = torch.exp(-torch.exp(w[p + "A_log"]) * softplus(h @ w[p + "a"].T + w[p + "dt_bias"]))
    o = delta_scan(own(q), own(k), v.view(T, H, E), beta, g)
    if watch is not None:
        # (the corrections depend on each other; the squares of an uncorrected write stand for its terms' size)
        watch("heads", o, write_squares(own(q), own(k), v.view(T, H, E), beta, g))
    return (rms(o, eps) * w[p + "norm"]).reshape(T, H * E).mul(silu(h @ w[p + "g"].T)) @ w[p + "o"].T


def clamped(h, w, p, limit):
    gate = (h @ w[p + "gate"].T).clamp(max=limit)
    up = (h @ w[p + "up"].T).clamp(-limit, limit)
    return (gate * torch.sigmoid(1.702 * gate) * (up + 1)) @ w[p + "down"].T


def gated(h, w, p):
    return (silu(h @ w[p + "gate"].T) * (h @ w[p + "up"].T)) @ w[p + "down"].T


def choose(scores, choice, r):
    """One token: scores and choice scores [E] -> {expert: weight}. Groups of neighbours compete first, by the sum of
    their two largest choice scores; then the experts of the groups that stay."""
    experts, top = len(choice), int(r["top"])
    open_experts = list(range(experts))
    if r.get("groups"):
        count, keep = int(r["groups"]["count"]), int(r["groups"]["keep"])
        size = experts // count
        strength = [sum(sorted(choice[g * size:(g + 1) * size].tolist(), reverse=True)[:2]) for g in range(count)]
        kept = sorted(range(count), key=lambda g: (-strength[g], g))[:keep]
        open_experts = [e for e in open_experts if e // size in kept]
    chosen = sorted(open_experts, key=lambda e: (-float(choice[e]), e))[:top]
    total = sum(float(scores[e]) for e in chosen) + 1e-20
    return {e: float(scores[e]) / total * float(r["scale"]) for e in chosen}


def mixture(h, w, p, mlp, watch=None):
    scores = torch.sigmoid(h @ w[p + "router"].T)
    choice = scores + w[p + "correction"]
    if watch is not None:
        watch("router", choice, mlp["router"])
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e, weight in choose(scores[t], choice[t], mlp["router"]).items():
            out[t] += weight * gated(h[t:t + 1], w, f"{p}e{e}.")[0]
    if mlp.get("shared"):
        out = out + torch.sigmoid(h @ w[p + "shared.sg"].T) * gated(h, w, p + "shared.")
    return out


def feed_forward(h, w, p, mlp, watch=None):
    return clamped(h, w, p, float(mlp["limit"])) if mlp["kind"] == "dense" else mixture(h, w, p, mlp, watch)


MIXERS = {"parallel": parallel, "mamba2": mamba2, "delta": delta}


def forward(cfg, weights, ids, watch=None):
    """-> (float64 logits [T, vocab], the residual behind every layer). `watch(what, ...)` is shown the choice scores of
    the routers and the heads' outputs in front of their norms."""
    w = {name: t.double() for name, t in weights.items()}
    eps, mult = float(cfg["norm"]["eps"]), float(cfg["residual_mult"])
    x = w["embed"][torch.as_tensor(ids, dtype=torch.long)]
    after = []
    for i, layer in enumerate(cfg["layers"]):
        p = f"l{i}."
        x = x + mult * rms(MIXERS[layer["type"]](x, w, p + "mix.", layer["mixer"], eps, watch), eps) * w[p + "norm1"]
        if layer.get("mlp"):
            x = x + mult * rms(feed_forward(x, w, p + "mlp.", layer["mlp"], watch), eps) * w[p + "norm2"]
        after.append(x.clone())
    return rms(x, eps) * w["final.norm"] @ w["head"].T, after
