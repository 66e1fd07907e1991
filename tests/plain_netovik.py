"""The Netovik decoder in the plainest way: float64, whole sequences, one function for each mechanism, loops where a
loop says it best. It shares no code with the package; the tests compare the engine with it.

Notation: T tokens, C the model width, rms(v) = v / sqrt(mean(v^2) + eps). Weights come as a dict by checkpoint name,
linear weights [out, in]."""

from __future__ import annotations

import math

import torch


def rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def group_norm(x, weight, groups, eps):
    """Every one of `groups` equal parts of a row divided by its own root mean square, then the weight."""
    T, C = x.shape
    return rms(x.view(T, groups, C // groups), eps).reshape(T, C) * weight


def silu(z):
    return z * torch.sigmoid(z)


def token_shift(h):
    """The row of the token before; zeros for the first."""
    return torch.cat([torch.zeros_like(h[:1]), h[:-1]])


def wkv_decay(mixed, w1, w2, w0):
    """[T, C] -> the factor on every key channel, [T, N]."""
    return torch.exp(-torch.exp(torch.tanh(mixed @ w1.T) @ w2.T + w0))


def wkv_scan(r, k, v, decay, u):
    """r, k, v, decay [T, H, D], u [H, D] -> o [T, H, D]."""
    T, H, D = r.shape
    state = torch.zeros(H, D, D, dtype=torch.float64)
    out = torch.zeros(T, H, D, dtype=torch.float64)
    for t in range(T):
        pair = k[t][:, :, None] * v[t][:, None, :]
        out[t] = ((state + u[:, :, None] * pair) * r[t][:, :, None]).sum(1)
        state = decay[t][:, :, None] * state + pair
    return out


def wkv(h, w, p, m, eps, watch=None):
    T = h.shape[0]
    H, D = int(m["heads"]), int(m["dim"])
    before = token_shift(h)
    mix = {name: h + (before - h) * w[p + "mu." + name] for name in "rkvgw"}
    r, k, v = ((mix[name] @ w[p + name].T).view(T, H, D) for name in "rkv")
    gate = silu(mix["g"] @ w[p + "g"].T)
    decay = wkv_decay(mix["w"], w[p + "w1"], w[p + "w2"], w[p + "w0"]).view(T, H, D)
    o = wkv_scan(r, k, v, decay, w[p + "u"])
    if watch is not None:
        watch("heads", o, wkv_scan(r ** 2, k ** 2, v ** 2, decay ** 2, w[p + "u"] ** 2))     # and its terms' squares, summed
    return (rms(o, eps).reshape(T, H * D) * w[p + "norm"] * gate) @ w[p + "o"].T


def bucket(n, rows, bias_max):
    """Which of `rows` entries a distance of n tokens has: one each up to rows / 2, then logarithmically wider ones."""
    half = rows // 2
    if n < half:
        return n
    place = math.log(n / half) / math.log(bias_max / half) * (rows - half)
    if abs(place - round(place)) < 1e-9:
        place = round(place)
    return min(rows - 1, half + math.floor(place))


def visible(T, mask):
    """[T, T] (query, key): which keys a query sees."""
    i, j = torch.arange(T)[:, None], torch.arange(T)[None, :]
    seen = j <= i
    if mask:
        seen = seen & ((i - j < int(mask["size"])) | (j < int(mask.get("keep_first") or 0)))
    return seen


def attention_scores(q, k, m, rel, talk):
    """q [T, H, D] and k [T, G, D] (normed) -> the mixed scores [H, T, T], not masked."""
    T, H, _ = q.shape
    G = k.shape[1]
    scores = torch.stack([q[:, h] @ k[:, h // (H // G)].T * float(m["scale"]) for h in range(H)])
    if m.get("softcap"):
        scores = float(m["softcap"]) * torch.tanh(scores / float(m["softcap"]))
    by_distance = torch.stack([rel[bucket(n, rel.shape[0], float(m["bias_max"]))] for n in range(T)])      # [T, H]
    distance = (torch.arange(T)[:, None] - torch.arange(T)[None, :]).clamp(min=0)
    scores = scores + by_distance[distance].permute(2, 0, 1)
    return (talk @ scores.reshape(H, T * T)).view(H, T, T)


def softmax_one(scores, seen):
    """exp(s) / (1 + sum exp(s)) over the keys that are seen."""
    scores = scores.masked_fill(~seen, -math.inf)
    top = scores.max(-1, keepdim=True).values.clamp(min=0.0)
    e = torch.exp(scores - top)
    return e / (e.sum(-1, keepdim=True) + torch.exp(-top))


def attention(h, w, p, m, eps):
    T = h.shape[0]
    H, G, D = int(m["heads"]), int(m["kv_heads"]), int(m["dim"])
    q = rms((h @ w[p + "q"].T + w[p + "q.b"]).view(T, H, D), eps)
    v = (h @ w[p + "k"].T + w[p + "k.b"]).view(T, G, D)
    weights = softmax_one(attention_scores(q, rms(v, eps), m, w[p + "rel"], w[p + "talk"]), visible(T, m.get("mask")))
    return torch.cat([weights[i] @ v[:, i // (H // G)] for i in range(H)], -1) @ w[p + "o"].T


def gated(h, w, p):
    return (silu(h @ w[p + "gate"].T) * (h @ w[p + "up"].T)) @ w[p + "down"].T


def route(h, router, top):
    """-> (chosen experts [T, top], their softmax scores over all experts)."""
    scores = torch.softmax(h @ router.T, -1)
    order = torch.sort(scores, dim=-1, descending=True, stable=True)
    return order.indices[:, :top], order.values[:, :top]


def mixture(h, w, p, mlp, watch=None):
    chosen, scores = route(h, w[p + "router"], int(mlp["router"]["top"]))
    if watch is not None:
        watch("router", h @ w[p + "router"].T, int(mlp["router"]["top"]))
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e, s in zip(chosen[t].tolist(), scores[t]):
            out[t] += s * gated(h[t:t + 1], w, f"{p}e{e}.")[0]
    return out


def feed_forward(h, w, p, mlp, watch=None):
    return gated(h, w, p) if mlp["kind"] == "dense" else mixture(h, w, p, mlp, watch)


def depth_average(results, weights):
    return sum(weights[j] * x for j, x in enumerate(results))


def forward(cfg, weights, ids, watch=None):
    """-> (float64 logits [T, vocab], the averaged residual behind every layer). `watch(what, ...)` is shown the heads'
    outputs in front of their norms and the routers' logits."""
    w = {name: t.double() for name, t in weights.items()}
    eps, groups = float(cfg["norm"]["eps"]), int(cfg["norm"].get("groups") or 1)
    ids = torch.as_tensor(ids, dtype=torch.long)
    x = w["embed"][ids] * float((cfg.get("embedding") or {}).get("scale", 1.0))
    results, after = [x], []
    for i, layer in enumerate(cfg["layers"]):
        p = f"l{i}."
        if layer["type"] == "wkv":
            y = wkv(x, w, p + "mix.", layer["mixer"], eps, watch)
        else:
            y = attention(x, w, p + "mix.", layer["mixer"], eps)
        x = x + group_norm(y, w[p + "norm1"], groups, eps)
        if layer.get("mlp"):
            x = x + group_norm(feed_forward(x, w, p + "mlp.", layer["mlp"], watch), w[p + "norm2"], groups, eps)
        results.append(x)
        x = depth_average(results, w[p + "dwa"])
        after.append(x.clone())
    return group_norm(x, w["final.norm"], groups, eps) @ w["embed"].T, after
