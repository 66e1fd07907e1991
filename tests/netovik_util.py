"""Small Netovik models for the tests: configurations, random weights by tensor name, model folders. The names and
shapes of the tensors are written out here from the design, not taken from the package."""

from __future__ import annotations

import json
import math
from pathlib import Path

import torch

import plain_netovik as plain
from distie_amd.weights.safetensors_io import write_safetensors


def dense(ff=40):
    return {"kind": "dense", "ff": ff}


def moe(experts=5, top=2, ff=12):
    return {"kind": "moe", "router": {"experts": experts, "top": top}, "expert": {"ff": ff}}


def wkv(heads=3, dim=8, rank=5, mlp="dense"):
    """(`rank`, like `bias_rows` below, is not a key of a model folder's config.json: `write_model` takes it out)"""
    return _layer("wkv", {"heads": heads, "dim": dim, "rank": rank}, mlp)


def attention(heads=6, kv_heads=3, dim=12, scale=0.4, softcap=8.0, bias_max=30, bias_rows=10, size=9, keep_first=3, mlp="dense"):
    mixer = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": dim, "scale": scale, "bias_max": bias_max,
             "bias_rows": bias_rows}
    if softcap is not None:
        mixer["softcap"] = softcap
    if size is not None:
        mixer["mask"] = {"size": size, "keep_first": keep_first}
    return _layer("attention", mixer, mlp)


def _layer(kind, mixer, mlp):
    return {"type": kind, "mixer": mixer, "mlp": dense() if mlp == "dense" else mlp}


def make_config(layers, vocab=61, width=48, eps=1e-5, groups=4, embed_scale=2.0):
    return {"architecture": "Netovik", "vocab": vocab, "width": width, "norm": {"eps": eps, "groups": groups},
            "embedding": {"scale": embed_scale}, "layers": layers}


def tensor_shapes(cfg):
    """Checkpoint name -> shape, from the design."""
    C = cfg["width"]
    out = {"embed": (cfg["vocab"], C), "final.norm": (C,)}
    for i, lay in enumerate(cfg["layers"]):
        p, m = f"l{i}.", lay["mixer"]
        out.update({p + "norm1": (C,), p + "dwa": (i + 2,)})
        H, D = m["heads"], m["dim"]
        if lay["type"] == "wkv":
            N, R = H * D, m["rank"]
            out.update({p + f"mix.mu.{x}": (C,) for x in "rkvgw"})
            out.update({p + f"mix.{x}": (N, C) for x in "rkvg"})
            out.update({p + "mix.w1": (R, C), p + "mix.w2": (N, R), p + "mix.w0": (N,), p + "mix.u": (H, D),
                        p + "mix.norm": (N,), p + "mix.o": (C, N)})
        else:
            G = m["kv_heads"]
            out.update({p + "mix.q": (H * D, C), p + "mix.q.b": (H * D,), p + "mix.k": (G * D, C), p + "mix.k.b": (G * D,),
                        p + "mix.rel": (m["bias_rows"], H), p + "mix.talk": (H, H), p + "mix.o": (C, H * D)})
        mlp = lay.get("mlp")
        if not mlp:
            continue
        out[p + "norm2"] = (C,)
        if mlp["kind"] == "dense":
            parts = {"mlp.": mlp["ff"]}
        else:
            parts = {f"mlp.e{e}.": mlp["expert"]["ff"] for e in range(mlp["router"]["experts"])}
            out[p + "mlp.router"] = (mlp["router"]["experts"], C)
        for prefix, F in parts.items():
            out.update({p + prefix + "gate": (F, C), p + prefix + "up": (F, C), p + prefix + "down": (C, F)})
    return out


def random_weights(cfg, seed=0, dtype=torch.float32):
    """Values that keep every mechanism alive: projections ~ N(0, 1/in), norm weights around one, mixes with the token
    before of every sign, decays spread so that some channels forget within a token or two and others keep hundreds,
    bonuses, biases, distance biases and mixing of order one, averages that give every earlier result a say. Rounded to
    `dtype` (the oracle computes with what the file holds)."""
    g = torch.Generator().manual_seed(seed)
    rnd = lambda *shape: torch.randn(*shape, generator=g)
    w = {}
    for name, shape in tensor_shapes(cfg).items():
        last = name.split(".")[-1]
        if last in ("norm", "norm1", "norm2"):
            t = 1.0 + 0.2 * rnd(*shape)
        elif last == "dwa":
            t = 0.25 * rnd(*shape)
            t[-1] = 1.0 + 0.1 * float(rnd(1))
        elif ".mu." in name:
            t = 0.5 + 0.4 * rnd(*shape)
        elif last == "w0":
            t = torch.linspace(-6.5, 1.0, shape[0])[torch.randperm(shape[0], generator=g)]
        elif last == "w2":
            t = rnd(*shape) / math.sqrt(shape[-1])
        elif last == "u":
            t = 1.0 + 0.5 * rnd(*shape)
        elif last == "rel":
            t = 0.8 * rnd(*shape)
        elif last == "talk":
            t = torch.eye(shape[0]) + 0.4 * rnd(*shape) / math.sqrt(shape[0])
        elif last == "b":
            t = 0.3 * rnd(*shape)
        elif name == "embed":
            t = rnd(*shape)
        elif last == "router":
            t = 1.5 * rnd(*shape) / math.sqrt(shape[-1])
        else:
            t = rnd(*shape) / math.sqrt(shape[-1])
        w[name] = t.to(dtype)
    return w


def folder_config(cfg):
    """What config.json of a model folder holds: the sizes that the tensors tell are not among it."""
    out = json.loads(json.dumps(cfg))
    for layer in out["layers"]:
        layer["mixer"].pop("rank", None)
        layer["mixer"].pop("bias_rows", None)
    return out


def write_model(folder, cfg, weights) -> Path:
    folder = Path(folder)
    folder.mkdir(parents=True, exist_ok=True)
    (folder / "config.json").write_text(json.dumps(folder_config(cfg)))
    names = list(weights)
    write_safetensors(folder / "model.safetensors", [(n, weights[n].dtype, tuple(weights[n].shape)) for n in names],
                      ((n, weights[n].contiguous()) for n in names), {"format": "pt"})
    return folder


def oracle(cfg, weights, ids):
    """float64 logits of the plain implementation as float32 [T, vocab]."""
    return plain.forward(cfg, weights, ids)[0].float()


def random_ids(cfg, n, seed):
    return torch.randint(0, cfg["vocab"], (n,), generator=torch.Generator().manual_seed(seed)).tolist()


def close_calls(cfg, weights, ids):
    """For every position, two measures of how much rounding can change what the token computes (both 1.0 where the
    model has nothing of the kind): the smallest gap between the last chosen and the first unchosen router logit,
    relative to the largest logit of its row; and the smallest size of a time-mixing head's output in front of its norm,
    relative to the root of the sum of its terms' squares (what is left of a cancellation, as the first token's output is
    when its r and k are nearly orthogonal, comes out of the norm with a size and sign that rounding decides)."""
    gaps, sizes = torch.ones(len(ids), dtype=torch.float64), torch.ones(len(ids), dtype=torch.float64)

    def watch(what, *values):
        nonlocal gaps, sizes
        if what == "router":
            z, top = values
            if top < z.shape[1]:
                s = torch.sort(z, dim=-1, descending=True).values
                gaps = torch.minimum(gaps, (s[:, top - 1] - s[:, top]) / z.abs().max(-1).values)
        else:
            o, squares = values
            sizes = torch.minimum(sizes, (o.pow(2).mean(-1) / squares.mean(-1)).sqrt().min(-1).values)

    plain.forward(cfg, weights, ids, watch)
    return gaps, sizes


def clear_ids(cfg, weights, n, seed, margin=0.1, size=0.12):
    """`n` random token ids none of which hangs on a close call (`close_calls`): the first token that does is drawn
    again (what stands before it stays as it is, being causal), until none is left."""
    g = torch.Generator().manual_seed(seed)
    ids = torch.randint(0, cfg["vocab"], (n,), generator=g).tolist()
    for _ in range(40 * n):
        gaps, sizes = close_calls(cfg, weights, ids)
        close = ((gaps < margin) | (sizes < size)).nonzero()
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
