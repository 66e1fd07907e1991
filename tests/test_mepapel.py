"""The Mepapel decoder in the engine against the plain implementation (`plain_mepapel`), on the CPU test double (the
engine's logic: batching, cache, chunks of positions, state slots, scheduler) and on the GPU (the kernels, float32 and
bfloat16).

Models are tiny and their weights random (`mepapel_util.random_weights`); sizes are chosen so that nothing the design
lets differ is equal by accident, with variants where they are equal or 1. In bfloat16 a router's close call or a head's
output that is all cancellation may fall either way in any implementation; the sequences hold none
(`mepapel_util.clear_ids`)."""

import json

import pytest
import torch

import mepapel_util as mu
import plain_mepapel as plain
from distie_amd import LLM, SamplingParams
from distie_amd.config import ConfigError, config_from_dict
from distie_amd.engine.batch import StepEntry
from distie_amd.engine.model import Model
from torch_ops import TorchOps

DTYPES = {"float32": torch.float32, "bfloat16": torch.bfloat16}


@pytest.fixture(scope="module", params=["cpu", pytest.param("hip", marks=pytest.mark.gpu)])
def ops(request):
    if request.param == "cpu":
        return TorchOps()
    from distie_amd.kernels.hip_ops import HipOps

    return HipOps("cuda:0")


def precisions(ops):
    return ["float32"] if ops.device.type == "cpu" else ["float32", "bfloat16"]


def engine(folder, ops, dtype, **options):
    options.setdefault("block_size", 4 if ops.device.type == "cpu" else 16)
    options.setdefault("num_blocks", 96)
    options.setdefault("max_seqs", 4)
    options.setdefault("use_graphs", False)
    return LLM(folder, dtype=dtype, device=str(ops.device), ops=ops, **options)


def whole(llm, rid, ids):
    out = llm.step([StepEntry(rid, list(ids), list(range(len(ids))))])
    llm.finish(rid)
    return out.float().cpu()


def in_portions(llm, rid, ids, cuts):
    """`ids` in portions of the sizes `cuts`, the rest one token a step; every row's logits."""
    out, at, sizes = [], 0, list(cuts)
    while at < len(ids):
        n = min(sizes.pop(0) if sizes else 1, len(ids) - at)
        out.append(llm.step([StepEntry(rid, list(ids[at:at + n]), list(range(n)))]).float().cpu())
        at += n
    llm.finish(rid)
    return torch.cat(out)


def rounded_bound(folder, ids, want):
    """For every row, how far bfloat16 may be off: the usual bound, or (a branch that nearly cancels in front of its norm makes
    a row more sensitive to rounding than others) twice what the CPU test double is off in bfloat16, which rounds at the same
    places."""
    llm = LLM(folder, dtype="bfloat16", device="cpu", ops=TorchOps(), block_size=16, num_blocks=32, max_seqs=1, use_graphs=False)
    err = mu.logit_error(whole(llm, "a", ids), want)
    llm.close()
    return (2 * err).clamp(min=mu.TOL[torch.bfloat16])


def check(got, want, dtype, what="", bound=None):
    """float32: every row within the bound. bfloat16 (`bound`: a bound for every row, see above): one row in twenty may pass
    its bound, none 2.5 times it (a wrong key, a lost state or another expert moves a row by far more)."""
    err = mu.logit_error(got, want)
    tol = mu.TOL[DTYPES[dtype]]
    if dtype == "float32":
        assert float(err.max()) < tol, f"{what}: error {float(err.max())} at row {int(err.argmax())}"
        return
    over = err / (tol if bound is None else bound)
    worst = f"{what}: error {float(err[over.argmax()])} at row {int(over.argmax())}, {float(over.max())} times its bound"
    assert float(over.max()) < 2.5 and int((over > 1).sum()) <= max(1, len(err) // 20), worst


# nothing equal by accident: heads, head sizes, states, taps, chunks and feed-forwards of their own in every layer, every
# kind of mixer beside every kind of feed-forward; the last layer has none
MIXED = mu.make_config([
    mu.mamba2(heads=6, vdim=10, state=14, groups=3, conv=3, norm_groups=2, mlp=mu.moe(6, 2, 12, 3, 2, 1.3, 10)),
    mu.parallel(heads=6, kv_heads=3, dim=12, vdim=16, conv=3, left_dims=8, scale=0.4, size=11, r_heads=3, r_dim=14, r_vdim=10,
                right_dims=6, mlp=mu.dense(40, 0.9)),
    mu.delta(heads=6, kv_heads=2, dim=12, vdim=20, conv=4, mlp=mu.dense(24, 1.4)),
    mu.parallel(heads=4, kv_heads=1, dim=20, vdim=8, conv=4, left_dims=20, left_base=500.0, scale=0.25, size=40, r_heads=2,
                r_dim=10, r_vdim=18, right_dims=10, decay=(0.97, 0.8), mlp=mu.moe(8, 3, 20, 4, 2, 2.0, 14)),
    mu.delta(heads=3, kv_heads=3, dim=18, vdim=8, conv=2, mlp=mu.moe(5, 2, 16, 0, 0, 0.7, 0)),
    mu.mamba2(heads=4, vdim=16, state=10, groups=2, conv=4, norm_groups=4, mlp=None),
], vocab=61, width=48, mult=0.6)

# values that the model above makes different made equal, or 1: one head, one group of everything, one tap, every expert
# chosen, a chunk of a single position, whole heads turned, a residual that is not scaled
EQUAL = mu.make_config([
    mu.parallel(heads=1, kv_heads=1, dim=32, vdim=32, conv=1, left_dims=32, scale=1.0, size=1, r_heads=1, r_dim=32, r_vdim=32,
                right_dims=32, decay=(1.0,), mlp=mu.moe(2, 2, 32, 1, 1, 1.0, 32)),
    mu.delta(heads=1, kv_heads=1, dim=32, vdim=32, conv=1, mlp=mu.moe(1, 1, 32, 1, 1, 1.0, 32)),
    mu.mamba2(heads=1, vdim=32, state=32, groups=1, conv=1, norm_groups=1, mlp=mu.dense(32, 1.0)),
    mu.parallel(heads=2, kv_heads=2, dim=16, vdim=16, conv=2, left_dims=16, scale=0.25, size=16, r_heads=2, r_dim=16,
                r_vdim=16, right_dims=16, decay=(0.5, 0.5)),
], vocab=40, width=32, mult=1.0)

# sizes that fit no tile: a width of 42, five heads on one key/value head, a chunk that divides nothing, seven heads of 6
ODD = mu.make_config([
    mu.delta(heads=5, kv_heads=1, dim=22, vdim=10, conv=3, mlp=mu.dense(10, 2.0)),
    mu.parallel(heads=5, kv_heads=1, dim=20, vdim=6, conv=2, left_dims=2, scale=0.3, size=23, r_heads=3, r_dim=6, r_vdim=22,
                right_dims=4, decay=(0.99, 0.2, 0.9), mlp=mu.moe(9, 2, 10, 3, 1, 1.7, 6)),
    mu.mamba2(heads=7, vdim=6, state=9, groups=7, conv=2, norm_groups=3, mlp=None),
    mu.delta(heads=7, kv_heads=7, dim=6, vdim=14, conv=4, mlp=mu.moe(7, 3, 6, 7, 5, 1.0, 0)),
], vocab=50, width=42, mult=-0.4, eps=1e-6)

CONFIGS = {"mixed": MIXED, "equal": EQUAL, "odd": ODD}


@pytest.fixture(scope="module")
def folders(tmp_path_factory):
    made = {}
    for name, cfg in CONFIGS.items():
        weights = mu.random_weights(cfg, seed=3 + len(made), dtype=torch.bfloat16)
        made[name] = (mu.write_model(tmp_path_factory.mktemp(name), cfg, weights), cfg, weights)
    return made


def test_configuration_and_tensors():
    for cfg in CONFIGS.values():
        declared = {n: tuple(spec.shape) for n, spec in Model.declare(config_from_dict(cfg).model_spec()).items()}
        assert declared == mu.tensor_shapes(cfg)
    # what a file may leave out is off, or its only possible value
    short = json.loads(json.dumps(EQUAL))
    left, right = short["layers"][0]["mixer"]["left"], short["layers"][0]["mixer"]["right"]
    router = short["layers"][0]["mlp"]["router"]
    del left["kv_heads"], left["vdim"], right["vdim"], router["groups"], router["scale"], short["residual_mult"]
    for key in ("kv_heads", "vdim"):
        del short["layers"][1]["mixer"][key]
    for key in ("groups", "norm_groups"):
        del short["layers"][2]["mixer"][key]
    got, want = (config_from_dict(c).model_spec() for c in (short, EQUAL))
    for mine, theirs in zip(got.layers, want.layers):
        assert mine == theirs
    plain_left = json.loads(json.dumps(MIXED["layers"][1]))
    for key in ("conv", "mask", "rot"):
        del plain_left["mixer"]["left"][key]
    params = config_from_dict({**MIXED, "layers": [plain_left]}).model_spec().layers[0].parts["mixer"].params["mixers"]["left"].params
    assert params["conv_taps"] == 0 and params["chunk"] is None and params["position"] is None
    change = lambda layer, *path, value: _changed(layer, path, value)
    broken_layers = [
        mu.parallel(heads=3, kv_heads=2), mu.parallel(size=-1), mu.parallel(left_dims=7), mu.parallel(left_dims=14),
        mu.parallel(scale=0.0), mu.parallel(r_heads=2, decay=(0.5,)), mu.delta(heads=3, kv_heads=2), mu.delta(conv=0),
        mu.mamba2(heads=4, groups=3), mu.mamba2(heads=5, vdim=3, groups=1, norm_groups=2), mu.delta(mlp=mu.moe(3, 4, 8, 0, 0)),
        mu.delta(mlp=mu.moe(6, 3, 8, 3, 1)), mu.delta(mlp=mu.moe(6, 2, 8, 4, 2)), mu.delta(mlp=mu.moe(6, 2, 8, 3, 4)),
        mu.delta(mlp={"kind": "other"}), mu.delta(mlp={"kind": "dense", "ff": 8}), mu.delta(mlp=mu.dense(8, 0.0)),
        {"type": "other", "mixer": {"heads": 1, "dim": 4}, "mlp": None}, {"type": "delta", "mlp": None},
        change(mu.parallel(), "mixer", "right", value=None)]
    for layer in broken_layers:
        with pytest.raises(ConfigError):
            config_from_dict({**MIXED, "layers": [layer]})
    for missing in ("norm", "width", "vocab", "layers"):
        with pytest.raises(ConfigError):
            config_from_dict({k: v for k, v in MIXED.items() if k != missing})


def _changed(layer, path, value):
    out = json.loads(json.dumps(layer))
    at = out
    for key in path[:-1]:
        at = at[key]
    at[path[-1]] = value
    return out


def test_layers_one_by_one(ops, folders):
    """The residual behind every layer, through the engine's blocks, against the plain implementation."""
    from distie_amd.parts import ResidualStream, StepContext

    for name in CONFIGS:
        folder, cfg, weights = folders[name]
        ids = mu.random_ids(cfg, 21, seed=1)
        _, after = plain.forward(cfg, weights, ids)
        llm = engine(folder, ops, "float32")
        llm.cache.add("a")
        llm.cache.reserve("a", len(ids))
        tokens, meta, _ = llm.runner.builder.build([StepEntry("a", ids, [0])])
        stream = ResidualStream(llm.model.embed.forward(ops, tokens, meta))
        ctx = StepContext(meta, torch.float32)
        for i, block in enumerate(llm.model.blocks):
            block.forward(ops, stream, ctx, llm.cache.layer(i), True)
            delta, norm = stream.lanes["pending"]
            held = stream.hidden.clone()
            ops.add_normed(held, delta, norm.weight, norm.eps)
            err = (held.double().cpu() - after[i]).abs().max() / after[i].abs().max()
            assert float(err) < 2e-5, f"{name} layer {i}: {float(err)}"


@pytest.mark.parametrize("name", list(CONFIGS))
def test_prompt_decode_and_portions(ops, folders, name):
    """One prompt whole, token by token, and in portions of several sizes down to two tokens: every row's logits against
    the plain implementation, and the same whatever the cut."""
    folder, cfg, weights = folders[name]
    ids = mu.clear_ids(cfg, weights, 45, seed=11)
    want = mu.oracle(cfg, weights, ids)
    for dtype in precisions(ops):
        llm = engine(folder, ops, dtype)
        runs = {"whole": whole(llm, "a", ids), "token by token": in_portions(llm, "b", ids, []),
                "portions": in_portions(llm, "c", ids, [2, 7, 3, 2, 13, 5, 2, 4]),
                "a long portion, then tokens": in_portions(llm, "d", ids, [29])}
        bound = rounded_bound(folder, ids, want) if dtype == "bfloat16" else None
        for what, got in runs.items():
            check(got, want, dtype, f"{name} {dtype} {what}", bound)
        llm.cache.check()
        assert not llm.cache.live()


def test_portions_around_the_scans_chunks(ops, folders):
    """Portions that end just before, at and just behind the multiples of 16 and 64 rows in which a long portion's state is
    scanned, and short ones between them: the state and the last token's input handed from chunk to chunk, from portion
    to portion and on to decoding."""
    folder, cfg, weights = folders["mixed"]
    ids = mu.random_ids(cfg, 300, seed=12)
    want = mu.oracle(cfg, weights, ids)
    for dtype in ["float32"]:
        llm = engine(folder, ops, dtype, num_blocks=160)
        check(whole(llm, "a", ids), want, dtype, f"whole {dtype}")
        check(in_portions(llm, "b", ids, [63, 2, 64, 65, 33, 2, 32, 31]), want, dtype, f"portions {dtype}")
        check(in_portions(llm, "c", ids, [129, 128]), want, dtype, f"long portions {dtype}")
        check(in_portions(llm, "d", ids, [15, 16, 17, 48, 47, 49]), want, dtype, f"runs of sixteen {dtype}")
        llm.cache.check()


def test_unequal_batches_and_reuse(ops, folders):
    """Requests of unequal length side by side, portions beside single tokens, some left out of a step; more requests
    than state slots one after the other, so that pages and slots are used again with what the last owner left."""
    folder, cfg, weights = folders["mixed"]
    prompts = {i: mu.clear_ids(cfg, weights, n, seed=20 + i) for i, n in enumerate([31, 6, 19, 2, 70, 1, 23, 12])}
    want = {i: mu.oracle(cfg, weights, ids) for i, ids in prompts.items()}
    for dtype in precisions(ops):
        llm = engine(folder, ops, dtype, num_blocks=48, max_seqs=3)
        at = {i: 0 for i in prompts}
        got = {i: [] for i in prompts}
        waiting, live, turn = list(prompts), [], 0
        while waiting or live:
            while waiting and len(live) < 3:
                live.append(waiting.pop(0))
            entries = []
            for slot, i in enumerate(live):
                if (turn + slot) % 4 == 3 and len(live) > 1:
                    continue                                  # left out of this step
                left = len(prompts[i]) - at[i]
                n = min(left, [1, 5, 2, 37][(turn + i) % 4])
                entries.append((i, n))
            logits = llm.step([StepEntry(f"r{i}", prompts[i][at[i]:at[i] + n], list(range(n))) for i, n in entries])
            row = 0
            for i, n in entries:
                got[i].append(logits[row:row + n].float().cpu())
                row += n
                at[i] += n
                if at[i] == len(prompts[i]):
                    llm.finish(f"r{i}")
                    live.remove(i)
            llm.cache.check()
            turn += 1
        for i in prompts:
            check(torch.cat(got[i]), want[i], dtype, f"request {i} {dtype}",
                  rounded_bound(folder, prompts[i], want[i]) if dtype == "bfloat16" else None)
        assert not llm.cache.live() and llm.cache.free_pages() == [48] * len(llm.cache.groups)


def planted(cfg, weights, token_a, token_b):
    """Make what token `token_a` leaves in layer 0 stand out for token `token_b`. The embeddings get two channels of their
    own: only a has a value in the first, only b in the second. Keys (and what stands for them) read the first channel and
    queries the second, so that b's query meets a's key; a's value is large. What a state would forget or blur on the way is
    calmed: slow decays, filters that pass the current token on."""
    w = {k: v.clone().float() for k, v in weights.items()}
    w["embed"][:, :2] = 0.0
    w["embed"][token_a, 0] = 6.0
    w["embed"][token_b, 1] = 6.0

    def read(name, channel, strength=4.0, rows=slice(None)):
        w[name][rows, :2] = 0.0
        w[name][rows, channel] = strength

    kind, m, p = cfg["layers"][0]["type"], cfg["layers"][0]["mixer"], "l0.mix."
    for name in w:
        if name.startswith(p) and name.endswith(".conv"):
            w[name][:, :-1] *= 0.1
    if kind == "parallel":
        w[p + "left.k.b"] *= 0.1
        w[p + "left.q.b"] *= 0.1
        for side, strength in (("left.", 4.0), ("right.", 3.0)):
            read(p + side + "k", 0, strength)
            read(p + side + "q", 1, strength)
            w[p + side + "v"][:, 0] = 4.0
    elif kind == "delta":
        # a's key points along the first dimensions, everyone else's away from them: nobody writes over what a wrote
        G, D = m["kv_heads"], m["dim"]
        own = torch.arange(G * D) % D < 4
        for name, channel in (("k", 0), ("q", 1)):
            w[p + name][own] = 0.0
            read(p + name, channel, 6.0, own)
            w[p + name][~own, :2] = 0.0
        w[p + "v"][:, 0] = 4.0
        w[p + "b"][:, 0] = 4.0
        w[p + "a"] *= 0.1
        w[p + "dt_bias"].fill_(-6.0)
        w[p + "A_log"].fill_(-3.0)
    else:
        inner, bc = m["heads"] * m["vdim"], m["groups"] * m["state"]
        x, b, c = inner, 2 * inner, 2 * inner + bc
        read(p + "in", 0, 4.0, slice(b, b + bc))
        read(p + "in", 1, 4.0, slice(c, c + bc))
        w[p + "in"][x:x + inner, 0] = 4.0
        w[p + "in"][-m["heads"]:] *= 0.1
        w[p + "in"][-m["heads"]:, 0] = 1.0
        w[p + "dt_bias"].fill_(-3.0)
        w[p + "A_log"].fill_(-6.0)
    return {k: v.to(torch.bfloat16) for k, v in w.items()}


CHUNK = 70
FAR = {
    "delta": mu.make_config([mu.delta(heads=4, kv_heads=2, dim=24, vdim=16, conv=3), mu.parallel(mlp=None)], vocab=30, width=32),
    "mamba2": mu.make_config([mu.mamba2(heads=4, vdim=12, state=12, groups=2, conv=3, norm_groups=2), mu.delta(mlp=None)],
                             vocab=30, width=32),
    "retention": mu.make_config([mu.parallel(heads=4, kv_heads=2, dim=16, vdim=16, left_dims=4, left_base=1e6, scale=0.5, size=7,
                                             r_heads=2, r_dim=32, r_vdim=16, right_dims=2, right_base=10.0,
                                             decay=(0.999, 0.9998)), mu.delta(mlp=None)], vocab=30, width=32),
    "all": mu.make_config([mu.parallel(heads=4, kv_heads=2, dim=16, vdim=16, left_dims=4, left_base=1e6, scale=0.8, size=None,
                                       r_heads=2, r_dim=8, r_vdim=8, right_dims=8, decay=(0.5, 0.2)), mu.delta(mlp=None)],
                          vocab=30, width=32),
    "chunks": mu.make_config([mu.parallel(heads=4, kv_heads=2, dim=16, vdim=16, left_dims=4, left_base=1e6, scale=0.8, size=CHUNK,
                                          r_heads=2, r_dim=8, r_vdim=8, right_dims=8, decay=(0.5, 0.2)), mu.mamba2(mlp=None)],
                             vocab=30, width=32),
}


@pytest.mark.parametrize("kind", ["delta", "mamba2", "retention", "all"])
def test_a_far_token_among_hundreds(ops, tmp_path, kind):
    """What token A leaves behind (a key and value in the cache, or its mark on a state) stands out for token B. A lies up to
    hundreds of tokens back: the very first token, or the last of a page, or the first of the next; B asks for it in a
    prompt, in a later portion and in decoding. A lost or mixed-up page, or a state that is dropped between portions, moves
    the logits there by far more than the tolerance, which the plain implementation shows with A taken out."""
    A, B = 7, 11
    cfg = FAR[kind]
    weights = planted(cfg, mu.random_weights(cfg, seed=9, dtype=torch.float32), A, B)
    folder = mu.write_model(tmp_path / "far", cfg, weights)
    filler = [t for t in mu.random_ids(cfg, 900, seed=2) if t not in (A, B)]
    for first in (0, 15, 16, 64):
        ids = filler[:330]
        ids[first] = A
        asks = [first + 1, 200, 255, 256, 300, 329]
        for at in asks:
            ids[at] = B
        want = mu.oracle(cfg, weights, ids)
        without = mu.oracle(cfg, weights, ids[:first] + [filler[500]] + ids[first + 1:])
        assert float(mu.logit_error(without, want)[asks].min()) > 2 * mu.TOL[torch.bfloat16], \
            (kind, first, mu.logit_error(without, want)[asks])
        for dtype in precisions(ops):
            llm = engine(folder, ops, dtype, block_size=16, num_blocks=30)
            check(whole(llm, "a", ids)[asks], want[asks], dtype, f"{kind} prompt, A at {first}, {dtype}")
            got = in_portions(llm, "b", ids, [first + 1, 2, 197 - first, 56, 2, 50])
            check(got[asks], want[asks], dtype, f"{kind} portions, then decoding, A at {first}, {dtype}")


def test_edges_of_the_chunks(ops, tmp_path):
    """Token A is the first of a chunk, the last, one inside, or the last of the chunk before; B asks for it from the chunk's
    own last place, the next chunk's first places and from one further on, in a prompt, in portions that end around the
    asking places (and inside the chunk, so that a cut must not move the chunks), and in decoding. The plain implementation
    shows that seeing A or not makes a difference far beyond the tolerance."""
    A, B = 7, 11
    cfg = FAR["chunks"]
    weights = planted(cfg, mu.random_weights(cfg, seed=9, dtype=torch.float32), A, B)
    folder = mu.write_model(tmp_path / "edges", cfg, weights)
    filler = [t for t in mu.random_ids(cfg, 900, seed=4) if t not in (A, B)]
    for at in (0, CHUNK - 2, CHUNK - 1, CHUNK, CHUNK + 30, 2 * CHUNK - 12):
        end = (at // CHUNK + 1) * CHUNK                             # the first position of the next chunk
        ids = filler[:end + CHUNK + 5]
        ids[at] = A
        asks = [a for a in (at + 1, end - 1, end, end + 1, end + CHUNK - 1, end + CHUNK) if a > at]
        for ask in asks:
            ids[ask] = B
        want = mu.oracle(cfg, weights, ids)
        without = mu.oracle(cfg, weights, ids[:at] + [filler[500]] + ids[at + 1:])
        moved = mu.logit_error(without, want)
        for ask in asks:
            if ask < end:
                assert float(moved[ask]) > 2 * mu.TOL[torch.bfloat16], (at, ask, moved[ask])
        # were the chunks counted from another place, or not there, B would see A from the next one too
        free = json.loads(json.dumps(cfg))
        del free["layers"][0]["mixer"]["left"]["mask"]
        assert float(mu.logit_error(mu.oracle(free, weights, ids), want)[end]) > 2 * mu.TOL[torch.bfloat16]
        for dtype in precisions(ops):
            llm = engine(folder, ops, dtype, block_size=16, num_blocks=30)
            for what, got in (("prompt", whole(llm, "a", ids)),
                              ("portions", in_portions(llm, "b", ids, [at + 1, 2, max(1, end - at - 5), 2, 3, 17, 2, CHUNK - 24, 2])),
                              ("decoding", in_portions(llm, "c", ids, [max(at + 1, end - 3)]))):
                check(got[asks], want[asks], dtype, f"{what}, A at {at}, {dtype}")
            llm.cache.check()


def test_first_tokens_and_long_decoding(ops, folders):
    """The first tokens of a sequence one by one (a token that sees only itself and the sink; a first token without one
    before it), then decoding for hundreds of tokens across many pages and far past the window."""
    for name, dtypes in (("mixed", precisions(ops)), ("odd", ["float32"])):
        folder, cfg, weights = folders[name]
        ids = mu.clear_ids(cfg, weights, 150, seed=31) if "bfloat16" in dtypes else mu.random_ids(cfg, 150, seed=31)
        want = mu.oracle(cfg, weights, ids)
        for dtype in dtypes:
            llm = engine(folder, ops, dtype, num_blocks=48)
            got = in_portions(llm, "a", ids, [1, 1, 1, 2])
            check(got, want, dtype, f"{name} long decoding {dtype}", rounded_bound(folder, ids, want) if dtype == "bfloat16" else None)
            llm.cache.check()
            assert not llm.cache.live()


def test_greedy_generation_through_the_scheduler(ops, folders):
    """`LLM.generate`: continuous batching with a token budget that cuts the prompts, more requests than seats, and
    (on the GPU) captured decode steps. Every token is the plain implementation's greedy pick given what came before,
    or a near tie."""
    for name, dtypes in (("mixed", precisions(ops)), ("odd", ["float32"])):
        folder, cfg, weights = folders[name]
        prompts = [mu.random_ids(cfg, n, seed=40 + n) for n in (23, 5, 14, 9, 2)]
        for dtype in dtypes:
            llm = engine(folder, ops, dtype, num_blocks=64, max_seqs=3, token_budget=16,
                         use_graphs=ops.device.type != "cpu")
            outs = llm.generate(prompts, SamplingParams(max_new_tokens=12))
            slack = 1e-3 if dtype == "float32" else 0.35
            for prompt, out in zip(prompts, outs):
                assert len(out.token_ids) == 12
                ids = list(prompt) + list(out.token_ids)
                logits = mu.oracle(cfg, weights, ids)
                for at, token in enumerate(out.token_ids, len(prompt)):
                    row = logits[at - 1]
                    assert float(row[token]) >= float(row.max()) - slack * float(row.abs().max()), (dtype, out.token_ids)
            assert not llm.cache.live()
            llm.close()


@pytest.mark.gpu
def test_captured_steps_replay(folders):
    """A captured decode step replayed many times, with eager steps between the replays (new requests' prompts): the same
    tokens as without captured steps."""
    from distie_amd.kernels.hip_ops import HipOps

    ops = HipOps("cuda:0")
    folder, cfg, weights = folders["mixed"]
    prompts = [mu.random_ids(cfg, n, seed=80 + n) for n in (33, 4, 18, 27, 9, 40)]
    outs = {}
    for graphs in (False, True):
        llm = engine(folder, ops, "float32", num_blocks=96, max_seqs=4, token_budget=32, use_graphs=graphs)
        outs[graphs] = [o.token_ids for o in llm.generate(prompts, SamplingParams(max_new_tokens=20))]
        llm.close()
    assert outs[True] == outs[False]


def test_random_model_folder_reads_back(tmp_path):
    """`random-model` of the command line writes a folder that the loader takes, tensor for tensor as the design names
    them."""
    from distie_amd import cli
    from distie_amd.weights.safetensors_io import SafetensorsFile

    (tmp_path / "config.json").write_text(json.dumps(ODD))
    assert cli.main(["random-model", "--config-json", str(tmp_path / "config.json"), "--out", str(tmp_path / "m"),
                     "--seed", "3", "--dtype", "bf16", "--std", "0.1"]) == 0
    stored = SafetensorsFile(tmp_path / "m" / "model.safetensors")
    assert {name: tuple(entry[1]) for name, entry in stored.index.items()} == mu.tensor_shapes(ODD)
    stored.close()
    llm = engine(tmp_path / "m", TorchOps(), "float32")
    assert llm.step([StepEntry("a", [1, 2, 3], [2])]).shape == (1, ODD["vocab"])


@pytest.mark.gpu
def test_trace_runner_and_command_line(folders, tmp_path):
    """The trace runner as a program (its own process, steps on standard input, four requests live, pages and
    slots used again) and `generate` of the command line, on a Mepapel model, against the plain implementation."""
    import subprocess
    import sys
    from pathlib import Path

    import numpy as np

    root = Path(__file__).resolve().parents[1]
    folder, cfg, weights = folders["mixed"]
    lengths = {"p": 70, "q": 33, "r": 64, "s": 5, "t": 50, "u": 21}
    reqs = {r: mu.clear_ids(cfg, weights, n, 60 + n) for r, n in lengths.items()}
    want = {r: mu.oracle(cfg, weights, ids) for r, ids in reqs.items()}
    max_tokens = sum(-(-n // 64) * 64 for n in sorted(lengths.values())[-4:])
    for dtype in ("float32", "bfloat16"):
        out = tmp_path / dtype
        proc = subprocess.Popen([sys.executable, str(root / "bin" / "trace_run"), "--model", str(folder), "--dtype", dtype,
                                 "--out", str(out), "--max-tokens", str(max_tokens)],
                                stdin=subprocess.PIPE, stdout=subprocess.PIPE, text=True)
        got, at = {r: [] for r in reqs}, {r: 0 for r in reqs}
        waiting, live, step = list(reqs), [], 0
        while waiting or live:
            while waiting and len(live) < 4:
                live.append(waiting.pop(0))
            entries, end = [], []
            for k, r in enumerate(live):
                left = len(reqs[r]) - at[r]
                n = min(left, 1 if left <= 8 else [13, 2, 30, 7][(step + k) % 4])
                entries.append({"id": r, "tokens": reqs[r][at[r]:at[r] + n], "want": list(range(n))})
                at[r] += n
                if at[r] == len(reqs[r]):
                    end.append(r)
            proc.stdin.write(json.dumps({"step": step, "entries": entries, "end": end}) + "\n")
            proc.stdin.flush()
            assert proc.stdout.readline().strip() == f"done {step}"
            rows = torch.from_numpy(np.fromfile(out / f"{step}.f32", dtype="<f4").reshape(-1, cfg["vocab"]).copy())
            row = 0
            for e in entries:
                got[e["id"]].append(rows[row:row + len(e["tokens"])])
                row += len(e["tokens"])
            live = [r for r in live if r not in end]
            step += 1
        proc.stdin.close()
        assert proc.wait(timeout=60) == 0
        for r in reqs:
            check(torch.cat(got[r]), want[r], dtype, f"request {r} {dtype}",
                  rounded_bound(folder, reqs[r], want[r]) if dtype == "bfloat16" else None)
    prompts = [reqs["s"], reqs["q"][:9]]
    (tmp_path / "prompts.json").write_text(json.dumps(prompts))
    done = subprocess.run([sys.executable, "-m", "distie_amd.cli", "generate", "--model", str(folder), "--dtype", "fp32",
                           "--prompts", str(tmp_path / "prompts.json"), "--max-new-tokens", "6", "--num-blocks", "32",
                           "--out", str(tmp_path / "report.json")], cwd=str(root), capture_output=True, text=True, timeout=110)
    assert done.returncode == 0, done.stderr
    for prompt, record in zip(prompts, json.loads((tmp_path / "report.json").read_text())):
        ids = list(prompt)
        for token in record["token_ids"]:
            logits = mu.oracle(cfg, weights, ids)[-1]
            assert float(logits[token]) >= float(logits.max()) - 1e-3 * float(logits.abs().max())
            ids.append(token)


def test_preemption_recomputes(ops, folders):
    """So few pages that running requests are preempted and recomputed (their states start from zero again): every
    token still is the plain implementation's pick."""
    folder, cfg, weights = folders["mixed"]
    prompts = [mu.random_ids(cfg, n, seed=70 + n) for n in (20, 26, 17)]
    block = 4 if ops.device.type == "cpu" else 16
    new = 24 if block == 4 else 40
    llm = engine(folder, ops, "float32", block_size=block, num_blocks=-(-(26 + new) // block) + 1, max_seqs=3, token_budget=32)
    outs = llm.generate(prompts, SamplingParams(max_new_tokens=new))
    assert sum(o.preemptions for o in outs) > 0, "the pool was not small enough to preempt anybody"
    for prompt, out in zip(prompts, outs):
        logits = mu.oracle(cfg, weights, list(prompt) + list(out.token_ids))
        for at, token in enumerate(out.token_ids, len(prompt)):
            row = logits[at - 1]
            assert float(row[token]) >= float(row.max()) - 1e-3 * float(row.abs().max())
    llm.cache.check()
    assert not llm.cache.live()
