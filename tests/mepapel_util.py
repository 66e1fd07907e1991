"""Small Mepapel models for the tests: configurations, random weights by tensor name, model folders. The names and
shapes of the tensors are written out here from the design, not taken from the package."""

from __future__ import annotations

import json
import math
from pathlib import Path

import torch

import plain_mepapel as plain
from distie_amd.weights.safetensors_io import write_safetensors


def dense(ff=40, limit=1.2):
    return {"kind": "dense", "ff": ff, "limit": limit}


def moe(experts=6, top=2, ff=12, count=3, keep=2, scale=1.3, shared=10):
    out = {"kind": "moe", "router": {"experts": experts, "top": top, "scale": scale}, "expert": {"ff": ff}}
    if count:
        out["router"]["groups"] = {"count": count, "keep": keep}
    if shared:
        out["shared"] = {"ff": shared}
    return out


def _layer(kind, mixer, mlp):
    return {"type": kind, "mixer": mixer, "mlp": dense() if mlp == "dense" else mlp}


def mamba2(heads=6, vdim=10, state=14, groups=3, conv=3, norm_groups=2, mlp="dense"):
    return _layer("mamba2", {"heads": heads, "vdim": vdim, "state": state, "groups": groups, "conv": conv,
                             "norm_groups": norm_groups}, mlp)


def delta(heads=6, kv_heads=2, dim=12, vdim=20, conv=4, mlp="dense"):
    return _layer("delta", {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": conv}, mlp)


def parallel(heads=6, kv_heads=3, dim=12, vdim=16, conv=3, left_dims=8, left_base=10000.0, scale=0.4, size=11,
             r_heads=3, r_dim=14, r_vdim=10, right_dims=6, right_base=5000.0, decay=(0.9, 0.99, 0.6), mlp="dense"):
    left = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale,
            "rot": {"base": left_base, "dims": left_dims}}
    if conv:
        left["conv"] = conv
    if size:
        left["mask"] = {"size": size}
    right = {"heads": r_heads, "dim": r_dim, "vdim": r_vdim, "rot": {"base": right_base, "dims": right_dims},
             "decay": list(decay)[:r_heads]}
    return _layer("parallel", {"left": left, "right": right}, mlp)


def make_config(layers, vocab=61, width=48, eps=1e-5, mult=0.6):
    return {"architecture": "Mepapel", "vocab": vocab, "width": width, "norm": {"eps": eps}, "residual_mult": mult,
            "layers": layers}


def tensor_shapes(cfg):
    """Checkpoint name -> shape, from the design."""
    C = cfg["width"]
    out = {"embed": (cfg["vocab"], C), "head": (cfg["vocab"], C), "final.norm": (C,)}
    for i, lay in enumerate(cfg["layers"]):
        p, m = f"l{i}.", lay["mixer"]
        out[p + "norm1"] = (C,)
        if lay["type"] == "mamba2":
            inner, bc = m["heads"] * m["vdim"], m["groups"] * m["state"]
            channels = inner + 2 * bc
            out.update({p + "mix.in": (inner + channels + m["heads"], C), p + "mix.conv": (channels, m["conv"]),
                        p + "mix.conv.b": (channels,), p + "mix.norm": (inner,), p + "mix.o": (C, inner)})
            out.update({p + "mix." + n: (m["heads"],) for n in ("dt_bias", "A_log", "D")})
        elif lay["type"] == "delta":
            rows = {"q": m["kv_heads"] * m["dim"], "k": m["kv_heads"] * m["dim"], "v": m["heads"] * m["vdim"]}
            out.update({p + "mix." + n: (r, C) for n, r in rows.items()})
            out.update({p + f"mix.{n}.conv": (r, m["conv"]) for n, r in rows.items()})
            out.update({p + "mix.g": (rows["v"], C), p + "mix.b": (m["heads"], C), p + "mix.a": (m["heads"], C),
                        p + "mix.dt_bias": (m["heads"],), p + "mix.A_log": (m["heads"],), p + "mix.norm": (m["vdim"],),
                        p + "mix.o": (C, rows["v"])})
        else:
            a, r = m["left"], m["right"]
            rows = {"q": a["heads"] * a["dim"], "k": a["kv_heads"] * a["dim"], "v": a["kv_heads"] * a["vdim"]}
            for n, count in rows.items():
                out.update({p + f"mix.left.{n}": (count, C), p + f"mix.left.{n}.b": (count,)})
                if a.get("conv"):
                    out[p + f"mix.left.{n}.conv"] = (count, a["conv"])
            out.update({p + "mix.left.q.norm": (a["dim"],), p + "mix.left.k.norm": (a["dim"],),
                        p + "mix.left.o": (C, a["heads"] * a["vdim"]), p + "mix.left.o.b": (C,)})
            qk, v = r["heads"] * r["dim"], r["heads"] * r["vdim"]
            out.update({p + "mix.right.q": (qk, C), p + "mix.right.k": (qk, C), p + "mix.right.v": (v, C),
                        p + "mix.right.g": (v, C), p + "mix.right.o": (C, v)})
            out.update({p + f"mix.{side}.out": (C,) for side in ("left", "right")})
        mlp = lay.get("mlp")
        if not mlp:
            continue
        out[p + "norm2"] = (C,)
        if mlp["kind"] == "dense":
            parts = {"mlp.": mlp["ff"]}
        else:
            E = mlp["router"]["experts"]
            parts = {f"mlp.e{e}.": mlp["expert"]["ff"] for e in range(E)}
            out.update({p + "mlp.router": (E, C), p + "mlp.correction": (E,)})
            if mlp.get("shared"):
                parts["mlp.shared."] = mlp["shared"]["ff"]
                out[p + "mlp.shared.sg"] = (1, C)
        for prefix, F in parts.items():
            out.update({p + prefix + "gate": (F, C), p + prefix + "up": (F, C), p + prefix + "down": (C, F)})
    return out


def random_weights(cfg, seed=0, dtype=torch.float32):
    """Values that keep every mechanism alive: projections ~ N(0, 1/in), norm weights around one, filters in which the
    current token stands out, decays spread so that some heads forget within a token or two and others keep hundreds,
    corrections as large as the scores they correct (some choice scores are negative), gates and clamps of order one.
    Rounded to `dtype` (the oracle computes with what the file holds)."""
    g = torch.Generator().manual_seed(seed)
    rnd = lambda *shape: torch.randn(*shape, generator=g)
    w = {}
    for name, shape in tensor_shapes(cfg).items():
        last = name.split(".")[-1]
        if last in ("norm", "norm1", "norm2", "out"):
            t = 1.0 + 0.2 * rnd(*shape)
        elif last == "conv":
            t = 0.4 * rnd(*shape)
            t[:, -1] += 1.0
        elif last == "A_log":
            t = torch.linspace(-2.5, 1.5, shape[0])[torch.randperm(shape[0], generator=g)]
        elif last == "dt_bias":
            t = -2.0 + rnd(*shape)
        elif last == "D":
            t = 0.5 + 0.5 * rnd(*shape)
        elif last == "correction":
            t = 0.6 * rnd(*shape)
        elif last == "b" and len(shape) == 1:
            t = 0.3 * rnd(*shape)
        elif name == "embed":
            t = rnd(*shape)
        elif last in ("router", "gate", "up"):
            t = 1.5 * rnd(*shape) / math.sqrt(shape[-1])
        else:
            t = rnd(*shape) / math.sqrt(shape[-1])
        w[name] = t.to(dtype)
    return w


def write_model(folder, cfg, weights) -> Path:
    folder = Path(folder)
    folder.mkdir(parents=True, exist_ok=True)
    (folder / "config.json").write_text(json.dumps(cfg))
    names = list(weights)
    write_safetensors(folder / "model.safetensors", [(n, weights[n].dtype, tuple(weights[n].shape)) for n in names],
                      ((n, weights[n].contiguous()) for n in names), {"format": "pt"})
    return folder


def oracle(cfg, weights, ids):
    """float64 logits of the plain implementation as float32 [T, vocab]."""
    return plain.forward(cfg, weights, ids)[0].float()


def random_ids(cfg, n, seed):
    return torch.randint(0, cfg["vocab"], (n,), generator=torch.Generator().manual_seed(seed)).tolist()


def router_gap(choice, r):
    """How far a token's choice scores are from another choice: the smaller of the gap between the last kept and the
    first dropped group's strength and that between the last chosen and the first unchosen open expert's score."""
    gap = 1.0
    open_scores = choice
    if r.get("groups") and r["groups"]["keep"] < r["groups"]["count"]:
        parts = choice.view(r["groups"]["count"], -1)
        strength = parts.sort(descending=True).values[:, :2].sum(-1)
        order = strength.argsort(descending=True)
        keep = r["groups"]["keep"]
        gap = float(strength[order[keep - 1]] - strength[order[keep]])
        open_scores = parts[order[:keep]].reshape(-1)
    s = open_scores.sort(descending=True).values
    if r["top"] < len(s):
        gap = min(gap, float(s[r["top"] - 1] - s[r["top"]]))
    return gap


def close_calls(cfg, weights, ids):
    """For every position, two measures of how much rounding can change what the token computes (1.0 where the model has
    nothing of the kind): `router_gap`, and the smallest size of a head's output in front of its norm, relative to the root
    of the sum of its terms' squares (what is left of a cancellation, as the first token's output is when its q and k are
    nearly orthogonal, comes out of the norm with a size and sign that rounding decides)."""
    gaps, sizes = torch.ones(len(ids), dtype=torch.float64), torch.ones(len(ids), dtype=torch.float64)

    def watch(what, *values):
        nonlocal gaps, sizes
        if what == "router":
            own = torch.tensor([router_gap(row, values[1]) for row in values[0]], dtype=torch.float64)
            gaps = torch.minimum(gaps, own)
        else:
            o, squares = values
            sizes = torch.minimum(sizes, (o.pow(2).mean(-1) / squares.mean(-1)).sqrt().min(-1).values)

    plain.forward(cfg, weights, ids, watch)
    return gaps, sizes


MARGIN, SIZE = 0.03, 0.25


def clear_ids(cfg, weights, n, seed):
    """`n` random token ids none of which hangs on a close call (`close_calls`): the first token that does is drawn
    again (what stands before it stays as it is, being causal), until none is left."""
    g = torch.Generator().manual_seed(seed)
    ids = torch.randint(0, cfg["vocab"], (n,), generator=g).tolist()
    for _ in range(40 * n):
        gaps, sizes = close_calls(cfg, weights, ids)
        close = ((gaps < MARGIN) | (sizes < SIZE)).nonzero()
        if not len(close):
            return ids
        ids[int(close[0])] = int(torch.randint(0, cfg["vocab"], (1,), generator=g))
    raise AssertionError("no sequence without a close call found")


def logit_error(got, want):
    """Per row: root mean square of the difference (its mean taken off), over that of the wanted logits."""
    d = got.double() - want.double()
    d = d - d.mean(-1, keepdim=True)
    ref = want.double() - want.double().mean(-1, keepdim=True)
    return (d.pow(2).mean(-1).sqrt() / ref.pow(2).mean().sqrt()).float()


TOL = {torch.float32: 5e-5, torch.bfloat16: 6e-2}
