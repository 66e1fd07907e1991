"""The Netovik decoder in the engine against the plain implementation (`plain_netovik`), on the CPU test double (the
engine's logic: batching, cache, kept first pages, state slots, scheduler) and on the GPU (the kernels, float32 and
bfloat16).

Models are tiny and their weights random (`netovik_util.random_weights`); sizes are chosen so that nothing the design
lets differ is equal by accident, with variants where they are equal or 1. In bfloat16 a router's close call or a head's
output that is all cancellation may fall either way in any implementation; the sequences hold none
(`netovik_util.clear_ids`)."""

import json

import pytest
import torch

import netovik_util as nu
import plain_netovik as plain
from distie_amd import LLM, SamplingParams
from distie_amd.cache import CacheManager
from distie_amd.config import ConfigError, config_from_dict
from distie_amd.engine.batch import StepEntry
from distie_amd.engine.model import Model
from distie_amd.parts import PagedKV
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


def check(got, want, dtype, what=""):
    """float32: every row within the bound. bfloat16: norms behind the sub-layers make a row now and then more sensitive
    to rounding than the others, so one row in twenty may pass the bound, none 2.5 times it (a wrong key, a lost state
    or a sink left out moves a row by far more)."""
    err = nu.logit_error(got, want)
    tol = nu.TOL[DTYPES[dtype]]
    worst = f"{what}: error {float(err.max())} at row {int(err.argmax())}"
    if dtype == "float32":
        assert float(err.max()) < tol, worst
    else:
        assert float(err.max()) < 2.5 * tol and int((err > tol).sum()) <= max(1, len(err) // 20), worst


# nothing equal by accident: heads, head sizes, ranks, tables and feed-forwards of their own in every layer; attention with a
# window and kept first keys, and attention that sees everything without a cap; the last layer has no feed-forward
MIXED = nu.make_config([
    nu.wkv(heads=3, dim=8, rank=5, mlp=nu.moe(5, 2, 12)),
    nu.attention(heads=6, kv_heads=3, dim=12, scale=0.4, softcap=8.0, bias_max=30, bias_rows=10, size=9, keep_first=3),
    nu.wkv(heads=2, dim=16, rank=4, mlp=nu.dense(24)),
    nu.attention(heads=4, kv_heads=1, dim=16, scale=0.3, softcap=None, bias_max=50, bias_rows=7, size=None,
                 mlp=nu.moe(4, 1, 20)),
    nu.wkv(heads=5, dim=10, rank=3, mlp=None),
], vocab=61, width=48, groups=4, embed_scale=2.0)

# values that the model above makes different made equal, or 1: one head, one group of the norm, an embedding that is not
# scaled, every expert used, a window without kept keys, a decay through one dimension
EQUAL = nu.make_config([
    nu.attention(heads=1, kv_heads=1, dim=32, scale=0.25, softcap=1.0, bias_max=8, bias_rows=4, size=5, keep_first=0,
                 mlp=nu.moe(2, 2, 32)),
    nu.wkv(heads=1, dim=32, rank=1, mlp=nu.moe(1, 1, 32)),
    nu.attention(heads=2, kv_heads=2, dim=16, scale=1.0, softcap=20.0, bias_max=8, bias_rows=2, size=1, keep_first=1),
], vocab=40, width=32, groups=1, embed_scale=1.0)

# sizes that fit no tile: a width of 42 in three groups, five heads on one key/value head of 20, a table of odd length, more
# kept keys than the window holds, a feed-forward of 10
ODD = nu.make_config([
    nu.wkv(heads=7, dim=6, rank=9, mlp=nu.dense(10)),
    nu.attention(heads=5, kv_heads=1, dim=20, scale=0.2, softcap=3.0, bias_max=17, bias_rows=9, size=6, keep_first=21,
                 mlp=nu.moe(3, 2, 10)),
    nu.attention(heads=3, kv_heads=3, dim=14, scale=0.35, softcap=30.0, bias_max=100, bias_rows=16, size=40, keep_first=5,
                 mlp=None),
    nu.wkv(heads=1, dim=22, rank=2, mlp=nu.moe(7, 3, 6)),
], vocab=50, width=42, groups=3, embed_scale=0.5)

CONFIGS = {"mixed": MIXED, "equal": EQUAL, "odd": ODD}


@pytest.fixture(scope="module")
def folders(tmp_path_factory):
    made = {}
    for name, cfg in CONFIGS.items():
        weights = nu.random_weights(cfg, seed=3 + len(made), dtype=torch.bfloat16)
        made[name] = (nu.write_model(tmp_path_factory.mktemp(name), cfg, weights), cfg, weights)
    return made


def test_configuration_and_tensors():
    for cfg in CONFIGS.values():
        bare = config_from_dict(nu.folder_config(cfg))
        with pytest.raises(ConfigError):
            bare.model_spec()                              # two sizes come from the tensors
        for config in (config_from_dict(cfg), bare.with_tensor_shapes(nu.tensor_shapes(cfg))):
            declared = {n: tuple(spec.shape) for n, spec in Model.declare(config.model_spec()).items()}
            assert declared == nu.tensor_shapes(cfg)
    # what a file may leave out is off, or its only possible value
    short = json.loads(json.dumps(EQUAL))
    del short["norm"]["groups"], short["embedding"], short["layers"][0]["mixer"]["kv_heads"]
    del short["layers"][0]["mixer"]["vdim"], short["layers"][0]["mixer"]["mask"]["keep_first"]
    spec = config_from_dict(short).model_spec()
    assert spec.embedding.params["scale"] == 1.0 and spec.final_norm.params["groups"] == 1
    assert spec.layers[0].parts["mixer"].params == config_from_dict(EQUAL).model_spec().layers[0].parts["mixer"].params
    for broken in ({**MIXED, "layers": [nu.attention(heads=3, kv_heads=2)]},
                   {**MIXED, "layers": [{**nu.attention(), "mixer": {**nu.attention()["mixer"], "vdim": 8}}]},
                   {**MIXED, "layers": [nu.attention(size=0)]},
                   {**MIXED, "layers": [nu.attention(keep_first=-1)]},
                   {**MIXED, "layers": [nu.attention(softcap=0.0)]},
                   {**MIXED, "layers": [nu.wkv(heads=0)]},
                   {**MIXED, "layers": [nu.wkv(mlp=nu.moe(3, 4, 8))]},
                   {**MIXED, "layers": [nu.wkv(mlp={"kind": "other"})]},
                   {**MIXED, "layers": [{"type": "other", "mixer": {"heads": 1, "dim": 4}, "mlp": None}]},
                   {**MIXED, "norm": {"eps": 1e-5, "groups": 5}},
                   {k: v for k, v in MIXED.items() if k != "norm"}):
        with pytest.raises(ConfigError):
            config_from_dict(broken)


def test_pages_of_kept_first_tokens_stay():
    """A window gives back the pages it has passed, but for those that hold the first tokens; when the request ends (or is
    preempted) they come back too."""
    cache = CacheManager([PagedKV(1, 4, window=8, keep_first=6), PagedKV(1, 4, window=8)], 4, 20, 2, allocate=False)
    cache.add("a")
    for n in (10, 7, 1, 1, 13):
        cache.reserve("a", n)
        cache.commit("a", n)
        cache.check()
    first = (32 - 8 + 1) // 4                              # the page of the oldest key that token 32 sees
    kept, plain_window = cache.request("a").tables
    assert [page >= 0 for page in kept] == [i < 2 or i >= first for i in range(8)]
    assert [page >= 0 for page in plain_window] == [i >= first for i in range(8)]
    cache.reset("a")
    assert cache.free_pages() == [20, 20]
    cache.reserve("a", 3)
    cache.commit("a", 3)
    cache.release("a")
    cache.check()
    assert cache.free_pages() == [20, 20]


def test_layers_one_by_one(ops, folders):
    """The averaged residual behind every layer, through the engine's blocks, against the plain implementation."""
    from distie_amd.parts import ResidualStream, StepContext

    for name in CONFIGS:
        folder, cfg, weights = folders[name]
        ids = nu.random_ids(cfg, 21, seed=1)
        _, after = plain.forward(cfg, weights, ids)
        llm = engine(folder, ops, "float32")
        llm.cache.add("a")
        llm.cache.reserve("a", len(ids))
        tokens, meta, _ = llm.runner.builder.build([StepEntry("a", ids, [0])])
        stream = ResidualStream(llm.model.embed.forward(ops, tokens, meta))
        ctx = StepContext(meta, torch.float32)
        for i, block in enumerate(llm.model.blocks):
            block.forward(ops, stream, ctx, llm.cache.layer(i), True)
            delta, norm, (index, depth) = stream.lanes["pending"]
            history = (stream.lanes["first"], stream.lanes["rest"].clone(), index, depth)
            held, _ = ops.add_group_normed(stream.hidden.clone(), delta, norm.weight, norm.eps, norm.groups, None, True, history)
            err = (held.double().cpu() - after[i]).abs().max() / after[i].abs().max()
            assert float(err) < 2e-5, f"{name} layer {i}: {float(err)}"


@pytest.mark.parametrize("name", list(CONFIGS))
def test_prompt_decode_and_portions(ops, folders, name):
    """One prompt whole, token by token, and in portions of several sizes down to two tokens: every row's logits against
    the plain implementation, and the same whatever the cut."""
    folder, cfg, weights = folders[name]
    ids = nu.clear_ids(cfg, weights, 45, seed=11)
    want = nu.oracle(cfg, weights, ids)
    for dtype in precisions(ops):
        llm = engine(folder, ops, dtype)
        runs = {"whole": whole(llm, "a", ids), "token by token": in_portions(llm, "b", ids, []),
                "portions": in_portions(llm, "c", ids, [2, 7, 3, 2, 13, 5, 2, 4]),
                "a long portion, then tokens": in_portions(llm, "d", ids, [29])}
        for what, got in runs.items():
            check(got, want, dtype, f"{name} {dtype} {what}")
        llm.cache.check()
        assert not llm.cache.live()


def test_portions_around_the_scans_chunks(ops, folders):
    """Portions that end just before, at and just behind the multiples of 16 and 64 rows in which a long portion's state is
    scanned, and short ones between them: the state and the last token's input handed from chunk to chunk, from portion
    to portion and on to decoding."""
    folder, cfg, weights = folders["mixed"]
    ids = nu.random_ids(cfg, 300, seed=12)
    want = nu.oracle(cfg, weights, ids)
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
    prompts = {i: nu.clear_ids(cfg, weights, n, seed=20 + i) for i, n in enumerate([31, 6, 19, 2, 70, 1, 23, 12])}
    want = {i: nu.oracle(cfg, weights, ids) for i, ids in prompts.items()}
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
            check(torch.cat(got[i]), want[i], dtype, f"request {i} {dtype}")
        assert not llm.cache.live() and llm.cache.free_pages() == [48] * len(llm.cache.groups)


def planted(cfg, weights, token_a, token_b):
    """Make what token `token_a` leaves in layer 0 stand out for token `token_b`. The embeddings get two channels of their
    own: only a has a value in the first, only b in the second.

    attention: every key row reads the first channel, every query row the second, so that behind their norms a's key and
    b's query point the same way and b's score for a is large wherever a is seen; a's value is its key and large too.
    wkv: a's keys and values are large (so what it writes into the state outweighs hundreds of later tokens) and the decay
    is slow; nothing is mixed with the token before."""
    w = {k: v.clone().float() for k, v in weights.items()}
    w["embed"][:, :2] = 0.0
    w["embed"][token_a, 0] = 6.0
    w["embed"][token_b, 1] = 6.0
    if cfg["layers"][0]["type"] == "attention":
        for name, channel in (("l0.mix.k", 0), ("l0.mix.q", 1)):
            w[name][:, :2] = 0.0
            w[name][:, channel] = 4.0
            w[name + ".b"] *= 0.1
        w["l0.mix.talk"] = torch.eye(len(w["l0.mix.talk"])) + 0.05 * w["l0.mix.talk"]
        w["l0.mix.rel"] *= 0.5
    else:
        for name in "rkvgw":
            w["l0.mix.mu." + name].zero_()
        for name in "rkv":
            w["l0.mix." + name][:, :2] = 0.0
        w["l0.mix.k"][:, 0] = 4.0
        w["l0.mix.v"][:, 0] = 4.0
        w["l0.mix.r"][:, 1] = 4.0
        w["l0.mix.w0"].fill_(-9.0)
        w["l0.mix.w2"] *= 0.1
    return {k: v.to(torch.bfloat16) for k, v in w.items()}


FAR_WINDOW, FAR_KEEP = 70, 19
FAR = {
    "all": nu.make_config([nu.attention(heads=4, kv_heads=2, dim=16, scale=0.6, softcap=12.0, bias_max=64, bias_rows=12, size=None),
                           nu.wkv(heads=2, dim=12, rank=3, mlp=None)], vocab=30, width=32, groups=2, embed_scale=1.0),
    "window": nu.make_config([nu.attention(heads=4, kv_heads=2, dim=16, scale=0.6, softcap=12.0, bias_max=64, bias_rows=12,
                                           size=FAR_WINDOW, keep_first=FAR_KEEP),
                              nu.wkv(heads=2, dim=12, rank=3, mlp=None)], vocab=30, width=32, groups=2, embed_scale=1.0),
    "wkv": nu.make_config([nu.wkv(heads=2, dim=12, rank=3),
                           nu.attention(heads=2, kv_heads=1, dim=16, mlp=None)], vocab=30, width=32, groups=2, embed_scale=1.0),
}


@pytest.mark.parametrize("kind", ["all", "wkv"])
def test_a_far_token_among_hundreds(ops, tmp_path, kind):
    """What token A leaves behind (a key and value in the cache, or its mark on the state) stands out for token B. A
    lies hundreds of tokens back: the very first token, or the last of a page, or the first of the next; B asks for it
    in a prompt, in a later portion and in decoding. A lost or mixed-up page, or a state that is dropped between
    portions, moves the logits there by far more than the tolerance, which the plain implementation shows with A
    taken out."""
    A, B = 7, 11
    cfg = FAR[kind]
    weights = planted(cfg, nu.random_weights(cfg, seed=9, dtype=torch.float32), A, B)
    folder = nu.write_model(tmp_path / "far", cfg, weights)
    filler = [t for t in nu.random_ids(cfg, 900, seed=2) if t not in (A, B)]
    for first in (0, 15, 16, 64):
        ids = filler[:330]
        ids[first] = A
        asks = [first + 1, 200, 255, 256, 300, 329]
        for at in asks:
            ids[at] = B
        want = nu.oracle(cfg, weights, ids)
        without = nu.oracle(cfg, weights, ids[:first] + [filler[500]] + ids[first + 1:])
        assert float(nu.logit_error(without, want)[asks].min()) > 2 * nu.TOL[torch.bfloat16], kind
        for dtype in precisions(ops):
            llm = engine(folder, ops, dtype, block_size=16, num_blocks=30)
            check(whole(llm, "a", ids)[asks], want[asks], dtype, f"prompt, A at {first}, {dtype}")
            got = in_portions(llm, "b", ids, [first + 1, 2, 197 - first, 56, 2, 50])
            check(got[asks], want[asks], dtype, f"portions, then decoding, A at {first}, {dtype}")


def test_edges_of_the_window_and_of_the_kept_tokens(ops, tmp_path):
    """Token B asks for token A just inside and just outside the window, with A among the kept first tokens (the first, the
    last of them) and just behind them (the next one, one at a page's start), in a prompt, in portions that end around the
    asking places, and in decoding. The plain implementation shows that seeing A or not makes a difference far beyond
    the tolerance."""
    A, B = 7, 11
    cfg = FAR["window"]
    weights = planted(cfg, nu.random_weights(cfg, seed=9, dtype=torch.float32), A, B)
    folder = nu.write_model(tmp_path / "edges", cfg, weights)
    filler = [t for t in nu.random_ids(cfg, 900, seed=4) if t not in (A, B)]
    for at in (0, FAR_KEEP - 1, FAR_KEEP, 31, 32, 48):
        ids = filler[:160]
        ids[at] = A
        asks = [at + FAR_WINDOW - 1, at + FAR_WINDOW, at + FAR_WINDOW + 1, at + FAR_WINDOW + 20, 159]
        for ask in asks:
            ids[ask] = B
        want = nu.oracle(cfg, weights, ids)
        without = nu.oracle(cfg, weights, ids[:at] + [filler[500]] + ids[at + 1:])
        moved = nu.logit_error(without, want)[asks]
        seen = [True] + [at < FAR_KEEP] * 4
        for m, s in zip(moved.tolist(), seen):
            assert not s or m > 2 * nu.TOL[torch.bfloat16], (at, moved)
        for dtype in precisions(ops):
            llm = engine(folder, ops, dtype, block_size=16, num_blocks=30)
            for what, got in (("prompt", whole(llm, "a", ids)),
                              ("portions", in_portions(llm, "b", ids, [at + 1, 2, FAR_WINDOW - 3, 2, 3, 17, 2])),
                              ("decoding", in_portions(llm, "c", ids, [at + FAR_WINDOW - 3]))):
                check(got[asks], want[asks], dtype, f"{what}, A at {at}, {dtype}")
            llm.cache.check()


def test_the_sink_counts(ops, folders, monkeypatch):
    """A softmax with one more in its denominator, where that matters: few visible keys with small scores."""
    cfg = nu.make_config([nu.wkv(heads=2, dim=8, rank=3, mlp=None),
                          nu.attention(heads=4, kv_heads=2, dim=16, scale=0.2, softcap=2.0, size=3, keep_first=1),
                          nu.attention(heads=2, kv_heads=2, dim=8, scale=0.5, softcap=1.0, size=2, keep_first=0)],
                         vocab=30, width=32, groups=2)
    weights = nu.random_weights(cfg, seed=6, dtype=torch.bfloat16)
    folder = nu.write_model(folders["mixed"][0].parent / "sinks", cfg, weights)
    ids = nu.clear_ids(cfg, weights, 40, seed=5)
    want = nu.oracle(cfg, weights, ids)
    with monkeypatch.context() as patch:
        patch.setattr(plain, "softmax_one", lambda s, seen: torch.softmax(s.masked_fill(~seen, -torch.inf), -1))
        moved = nu.logit_error(nu.oracle(cfg, weights, ids), want)
    # (not at the first token: what a sink takes from the only key's weight, the norm behind the mixer gives back)
    assert float(moved[3:].max()) > 2 * nu.TOL[torch.bfloat16] and float(moved[3:].median()) > 500 * nu.TOL[torch.float32]
    for dtype in precisions(ops):
        llm = engine(folder, ops, dtype)
        check(whole(llm, "a", ids), want, dtype, f"prompt {dtype}")
        check(in_portions(llm, "b", ids, [1, 1, 6]), want, dtype, f"first tokens one by one {dtype}")


def test_first_tokens_and_long_decoding(ops, folders):
    """The first tokens of a sequence one by one (a token that sees only itself and the sink; a first token without one
    before it), then decoding for hundreds of tokens across many pages and far past the window."""
    for name, dtypes in (("mixed", precisions(ops)), ("odd", ["float32"])):
        folder, cfg, weights = folders[name]
        ids = nu.clear_ids(cfg, weights, 150, seed=31) if "bfloat16" in dtypes else nu.random_ids(cfg, 150, seed=31)
        want = nu.oracle(cfg, weights, ids)
        for dtype in dtypes:
            llm = engine(folder, ops, dtype, num_blocks=48)
            got = in_portions(llm, "a", ids, [1, 1, 1, 2])
            check(got, want, dtype, f"{name} long decoding {dtype}")
            llm.cache.check()
            assert not llm.cache.live()


def test_greedy_generation_through_the_scheduler(ops, folders):
    """`LLM.generate`: continuous batching with a token budget that cuts the prompts, more requests than seats, and
    (on the GPU) captured decode steps. Every token is the plain implementation's greedy pick given what came before,
    or a near tie."""
    for name, dtypes in (("mixed", precisions(ops)), ("odd", ["float32"])):
        folder, cfg, weights = folders[name]
        prompts = [nu.random_ids(cfg, n, seed=40 + n) for n in (23, 5, 14, 9, 2)]
        for dtype in dtypes:
            llm = engine(folder, ops, dtype, num_blocks=64, max_seqs=3, token_budget=16,
                         use_graphs=ops.device.type != "cpu")
            outs = llm.generate(prompts, SamplingParams(max_new_tokens=12))
            slack = 1e-3 if dtype == "float32" else 0.35
            for prompt, out in zip(prompts, outs):
                assert len(out.token_ids) == 12
                ids = list(prompt) + list(out.token_ids)
                logits = nu.oracle(cfg, weights, ids)
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
    prompts = [nu.random_ids(cfg, n, seed=80 + n) for n in (33, 4, 18, 27, 9, 40)]
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
    assert {name: tuple(entry[1]) for name, entry in stored.index.items()} == nu.tensor_shapes(ODD)
    stored.close()
    llm = engine(tmp_path / "m", TorchOps(), "float32")
    assert llm.step([StepEntry("a", [1, 2, 3], [2])]).shape == (1, ODD["vocab"])


@pytest.mark.gpu
def test_trace_runner_and_command_line(folders, tmp_path):
    """The trace runner as a program (its own process, steps on standard input, four requests live, pages and
    slots used again) and `generate` of the command line, on a Netovik model, against the plain implementation."""
    import subprocess
    import sys
    from pathlib import Path

    import numpy as np

    root = Path(__file__).resolve().parents[1]
    folder, cfg, weights = folders["mixed"]
    lengths = {"p": 70, "q": 33, "r": 64, "s": 5, "t": 50, "u": 21}
    reqs = {r: nu.clear_ids(cfg, weights, n, 60 + n) for r, n in lengths.items()}
    want = {r: nu.oracle(cfg, weights, ids) for r, ids in reqs.items()}
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
            check(torch.cat(got[r]), want[r], dtype, f"request {r} {dtype}")
    prompts = [reqs["s"], reqs["q"][:9]]
    (tmp_path / "prompts.json").write_text(json.dumps(prompts))
    done = subprocess.run([sys.executable, "-m", "distie_amd.cli", "generate", "--model", str(folder), "--dtype", "fp32",
                           "--prompts", str(tmp_path / "prompts.json"), "--max-new-tokens", "6", "--num-blocks", "32",
                           "--out", str(tmp_path / "report.json")], cwd=str(root), capture_output=True, text=True, timeout=110)
    assert done.returncode == 0, done.stderr
    for prompt, record in zip(prompts, json.loads((tmp_path / "report.json").read_text())):
        ids = list(prompt)
        for token in record["token_ids"]:
            logits = nu.oracle(cfg, weights, ids)[-1]
            assert float(logits[token]) >= float(logits.max()) - 1e-3 * float(logits.abs().max())
            ids.append(token)


def test_preemption_recomputes(ops, folders):
    """So few pages that running requests are preempted and recomputed (their states start from zero again): every
    token still is the plain implementation's pick."""
    folder, cfg, weights = folders["mixed"]
    prompts = [nu.random_ids(cfg, n, seed=70 + n) for n in (20, 26, 17)]
    block = 4 if ops.device.type == "cpu" else 16
    new = 24 if block == 4 else 40
    llm = engine(folder, ops, "float32", block_size=block, num_blocks=-(-(26 + new) // block) + 1, max_seqs=3, token_budget=32)
    outs = llm.generate(prompts, SamplingParams(max_new_tokens=new))
    assert sum(o.preemptions for o in outs) > 0, "the pool was not small enough to preempt anybody"
    for prompt, out in zip(prompts, outs):
        logits = nu.oracle(cfg, weights, list(prompt) + list(out.token_ids))
        for at, token in enumerate(out.token_ids, len(prompt)):
            row = logits[at - 1]
            assert float(row[token]) >= float(row.max()) - 1e-3 * float(row.abs().max())
    llm.cache.check()
    assert not llm.cache.live()
