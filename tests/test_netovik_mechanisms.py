"""Each mechanism of the Netovik decoder alone, as the kernel surface and the parts offer it, against the matching
function of the plain implementation: on the CPU test double and on the GPU kernels (float32 and bfloat16 operands).

A step of a mixer's test is a batch of several requests' rows; cache and state are carried over several steps, with
slots that are taken in any order, and the result must be that of every sequence run at once."""

import math

import pytest
import torch

import netovik_util as nu
import plain_netovik as plain
from distie_amd.cache import CacheManager
from distie_amd.engine.batch import BatchBuilder, StepEntry
from distie_amd.parts import StepContext, build_part
from distie_amd.parts.mixed_attention import distance_bucket, spread_distance_bias
from torch_ops import TorchOps

F = torch.float64


@pytest.fixture(scope="module", params=["cpu", pytest.param("hip", marks=pytest.mark.gpu)])
def ops(request):
    if request.param == "cpu":
        return TorchOps()
    from distie_amd.kernels.hip_ops import HipOps

    return HipOps("cuda:0")


def rnd(*shape, seed=0, scale=1.0):
    return torch.randn(*shape, generator=torch.Generator().manual_seed(seed)) * scale


def act_types(ops):
    return [torch.float32] if ops.device.type == "cpu" else [torch.float32, torch.bfloat16]


def close(got, want, dtype, what="", slack=1.0):
    tol = (2e-5 if dtype == torch.float32 else 2e-2) * slack
    err = (got.double().cpu() - want.double()).abs().max() / (want.double().abs().max() + 1e-9)
    assert float(err) < tol, f"{what}: {float(err)}"


LENGTHS = (13, 1, 9, 6)
CUTS = ((5, 1, 2, 0), (1, 0, 1, 6), (2, 0, 0, 0), (1, 0, 6, 0), (4, 0, 0, 0))
LONG_LENGTHS = (150, 1, 70, 33)
LONG_CUTS = ((100, 1, 2, 0), (17, 0, 64, 33), (2, 0, 4, 0), (1, 0, 0, 0), (30, 0, 0, 0))


def run_mixer(ops, spec, tensors, seqs, cuts, dtype, slots=3, pages=64, block=None):
    """The mixer `spec` with `tensors` over the sequences `seqs` (inputs [n, C]), `cuts[step][i]` rows of sequence i in
    each step; a sequence takes its slot when it first appears and gives it back at its end, so slots and pages are
    used again. -> every sequence's output rows."""
    mixer = build_part("mixer", spec)
    mixer.load({k: v.to(ops.device) for k, v in tensors.items()})
    mixer.prepare(ops)
    cache = CacheManager([{"mixer": mixer.cache_requirement()}], block or (16 if ops.device.type != "cpu" else 4), pages, slots,
                         device=ops.device, dtype=dtype)
    builder = BatchBuilder(cache, 4096, ops.device, 4096)
    at = [0] * len(seqs)
    outs = [[] for _ in seqs]
    for step in cuts:
        entries, rows = [], []
        for i, n in enumerate(step):
            if not n:
                continue
            if i not in cache:
                cache.add(i)
            cache.reserve(i, n)
            entries.append(StepEntry(i, [0] * n, []))
            rows.append((i, at[i], n))
        _, meta, _ = builder.build(entries)
        x = torch.cat([seqs[i][a:a + n] for i, a, n in rows]).to(dtype).to(ops.device)
        y = ops.dense(mixer.forward(ops, x, StepContext(meta, dtype), cache.layer(0)["mixer"], True)).float().cpu()
        row = 0
        for i, a, n in rows:
            outs[i].append(y[row:row + n])
            row += n
            at[i] += n
            cache.commit(i, n)
            if at[i] == len(seqs[i]):
                cache.release(i)
    assert at == [len(s) for s in seqs]
    return [torch.cat(o) for o in outs]


def prefixed(weights, prefix):
    return {k[len(prefix):]: v for k, v in weights.items() if k.startswith(prefix)}


def mixer_case(ops, layer, plain_of, lengths, cuts, width=40, seed=0, slack=1.0, pages=64, change=None, block=None):
    from distie_amd.config import config_from_dict

    cfg = nu.make_config([layer], width=width)
    spec = config_from_dict(cfg).model_spec().layers[0].parts["mixer"]
    for dtype in act_types(ops):
        weights = nu.random_weights(cfg, seed=seed, dtype=dtype)
        if change is not None:
            change(weights)
        seqs = [rnd(n, width, seed=50 + i).to(dtype) for i, n in enumerate(lengths)]
        got = run_mixer(ops, spec, prefixed(weights, "l0.mix."), seqs, cuts, dtype, pages=pages, block=block)
        w = {k: v.to(F) for k, v in weights.items()}
        for i, s in enumerate(seqs):
            want = plain_of(s.to(F), w, "l0.mix.", layer["mixer"], float(cfg["norm"]["eps"]))
            close(got[i], want, dtype, f"sequence {i} {dtype}", slack)


def calm(weights):
    """Bonus and keys such that no head's output is all cancellation (its norm would turn rounding into a sign): every
    query, key and bonus mostly positive."""
    weights["l0.mix.u"] = weights["l0.mix.u"].abs() + 0.5
    weights["l0.mix.k"] = (weights["l0.mix.r"].float() + 0.3 * weights["l0.mix.k"].float()).to(weights["l0.mix.k"].dtype)
    weights["l0.mix.mu.k"] = weights["l0.mix.mu.r"].clone()


@pytest.mark.parametrize("heads,dim,rank", [(3, 8, 5), (1, 16, 1), (7, 6, 9), (2, 20, 33), (2, 48, 4), (3, 64, 16), (1, 72, 3),
                                            (2, 96, 40), (1, 128, 8), (1, 160, 7), (5, 64, 300)])
def test_time_mixing_alone(ops, heads, dim, rank):
    """Time mixing as a part over batches in steps: token shift, decay, bonus, head norm and gate; the state and the last
    input carried from step to step, row after row and in chunks of rows; heads of every kernel's size and of none, and
    beyond the chunks' largest."""
    layer = nu.wkv(heads=heads, dim=dim, rank=rank)
    mixer_case(ops, layer, plain.wkv, LENGTHS, CUTS, slack=3.0, change=calm)
    mixer_case(ops, layer, plain.wkv, LONG_LENGTHS, LONG_CUTS, seed=1, slack=3.0, change=calm, width=64)


@pytest.mark.parametrize("low,high", [(-12.0, -10.0), (-6.0, 2.0), (3.0, 6.0), (-8.0, 95.0)])
def test_decays_from_slow_to_none(ops, low, high):
    """Decays that keep everything, mixed ones, ones that forget at once, and ones whose exponent overflows: channels of
    every kind side by side, over many chunks."""
    def change(weights):
        calm(weights)
        w0 = weights["l0.mix.w0"]
        weights["l0.mix.w0"] = torch.linspace(low, high, w0.shape[0])[torch.randperm(
            w0.shape[0], generator=torch.Generator().manual_seed(1))].to(w0.dtype)

    mixer_case(ops, nu.wkv(heads=2, dim=32, rank=6), plain.wkv, (290, 40), ((200, 1), (1, 17), (64, 2), (25, 20)), seed=3,
               slack=3.0, change=change, width=64)


def test_decays_that_come_and_go(ops):
    """A decay that differs from token to token between nothing and almost everything."""
    def change(weights):
        calm(weights)
        weights["l0.mix.w2"] = (weights["l0.mix.w2"].float() * 6.0).to(weights["l0.mix.w2"].dtype)
        weights["l0.mix.w0"] = torch.full_like(weights["l0.mix.w0"], -1.0)

    mixer_case(ops, nu.wkv(heads=2, dim=64, rank=6), plain.wkv, (150, 33), ((130, 1), (20, 32)), seed=4, slack=3.0,
               change=change, width=64)


@pytest.mark.parametrize("sizes", [dict(heads=6, kv_heads=3, dim=12, size=9, keep_first=3),
                                   dict(heads=1, kv_heads=1, dim=32, size=5, keep_first=0),
                                   dict(heads=5, kv_heads=1, dim=20, size=6, keep_first=21, bias_rows=9, bias_max=17),
                                   dict(heads=3, kv_heads=3, dim=14, size=None, softcap=None, bias_rows=2, bias_max=4),
                                   dict(heads=16, kv_heads=4, dim=64, size=20, keep_first=17, bias_rows=32, bias_max=64),
                                   dict(heads=18, kv_heads=9, dim=96, size=33, keep_first=1),
                                   dict(heads=8, kv_heads=8, dim=128, size=None, bias_rows=16, bias_max=200),
                                   dict(heads=2, kv_heads=1, dim=160, size=70, keep_first=5),
                                   dict(heads=40, kv_heads=2, dim=16, size=16, keep_first=16),
                                   dict(heads=66, kv_heads=66, dim=8, size=12, keep_first=2)])
def test_attention_with_mixed_heads_alone(ops, sizes):
    """Attention as a part over batches in steps: head norms, raw keys as values, cap, bias by distance, scores mixed
    between the heads, window with kept first keys, the sink. Groups from one to twenty heads, heads beyond a tile and
    beyond what the matrix-core kernels take, head sizes that are padded and that are not."""
    layer = nu.attention(scale=0.3, **sizes)
    mixer_case(ops, layer, plain.attention, LENGTHS, CUTS, slack=2.0)
    mixer_case(ops, layer, plain.attention, LONG_LENGTHS, LONG_CUTS, seed=1, slack=2.0)


def test_attention_over_larger_pages_and_many_queries(ops):
    """Pages of 32 tokens, a portion of several hundred, decoding behind it: window edges and kept keys inside pages."""
    layer = nu.attention(heads=4, kv_heads=2, dim=32, scale=0.3, size=100, keep_first=37, bias_rows=12, bias_max=90)
    mixer_case(ops, layer, plain.attention, (330, 9), ((300, 1), (17, 5), (1, 1), (1, 1), (11, 1)), seed=2, slack=2.0,
               block=32)


@pytest.mark.gpu
def test_sixteen_queries_a_workgroup():
    """The wide form of the prefill kernel (steps of many tokens take it by themselves)."""
    from distie_amd.kernels.hip_ops import HipOps

    ops = HipOps("cuda:0")
    ops.MIXED_WIDE_TOKENS = 1
    for sizes in (dict(heads=6, kv_heads=3, dim=48, size=40, keep_first=18), dict(heads=16, kv_heads=4, dim=128, size=None)):
        mixer_case(ops, nu.attention(scale=0.3, **sizes), plain.attention, LONG_LENGTHS, LONG_CUTS, seed=1, slack=2.0)


def test_one_key_stands_out_at_every_distance(ops):
    """A key whose score towers over the others', at distances on both sides of the window's edge, of the kept keys' end and
    of every 16, 32 and 64 keys: seen where it should be, in a prompt and decoded."""
    size, keep, n = 50, 21, 140
    layer = nu.attention(heads=3, kv_heads=1, dim=16, scale=2.0, softcap=40.0, size=size, keep_first=keep)

    def change(weights):
        for name in ("q", "k"):
            weights["l0.mix." + name][:, 0] = 8.0          # whoever holds the first input channel looks for its like
            weights["l0.mix." + name + ".b"].zero_()

    from distie_amd.config import config_from_dict

    cfg = nu.make_config([layer], width=24)
    spec = config_from_dict(cfg).model_spec().layers[0].parts["mixer"]
    for dtype in act_types(ops):
        weights = nu.random_weights(cfg, seed=5, dtype=dtype)
        change(weights)
        w = {k: v.to(F) for k, v in weights.items()}
        for at in (0, 15, 16, keep - 1, keep, 31, 32, 63, 64):
            x = rnd(n, 24, seed=at)
            x[:, 0] = 0.0
            x[at, 0] = 5.0
            for ask in (at + 1, at + size - 1, at + size, at + size + 1, n - 1):
                if ask < n:
                    x[ask, 0] = 5.0
            x = x.to(dtype)
            want = plain.attention(x.to(F), w, "l0.mix.", layer["mixer"], 1e-5)
            for cuts in (((n,),), tuple((c,) for c in (at + 2, size - 3, 1, 1, 1, 1)) + tuple((1,) for _ in range(n - at - size - 3))):
                got = run_mixer(ops, spec, prefixed(weights, "l0.mix."), [x], cuts, dtype)
                close(got[0], want, dtype, f"key {at} {dtype}", 2.0)


def test_distance_buckets():
    """One row a distance up to half of the table, then logarithmically wider ones; the last row for all that is farther.
    Where a bucket begins exactly at a whole number, it begins there."""
    for rows, bias_max in ((16, 120.0), (32, 512.0), (10, 30.0), (9, 17.0), (2, 4.0), (2, 1e6), (4, 8.0)):
        table = torch.arange(rows, dtype=torch.float32)[:, None].repeat(1, 2)
        spread = spread_distance_bias(table, bias_max)
        last = spread.shape[1] - 1
        assert spread.shape[0] == 2 and float(spread[0, -1]) == rows - 1
        for n in list(range(0, min(last, 3000) + 40)) + [10 ** 6 + 1]:
            assert float(spread[1, min(n, last)]) == plain.bucket(n, rows, bias_max), (rows, bias_max, n)
    # 8 * 16^(k / 8) = 8 * 2^(k / 2): rows 10, 12 and 14 begin at 16, 32 and 64
    assert [distance_bucket(n, 16, 128.0) for n in (7, 8, 15, 16, 31, 32, 63, 64, 127, 128, 10 ** 6)] == \
        [7, 8, 9, 10, 11, 12, 13, 14, 15, 15, 15]
    assert distance_bucket(0, 1, 5.0) == 0 and distance_bucket(9, 1, 5.0) == 0 and distance_bucket(9, 8, 3.0) == 7


@pytest.mark.parametrize("width,groups", [(48, 4), (42, 3), (40, 1), (10, 10), (2048, 4), (8192, 8), (5000, 2), (6, 2)])
def test_norm_in_groups_and_average_over_the_depth(ops, width, groups):
    """The norm behind a sub-layer, its sum with the residual and the average over all earlier results, at several depths;
    the residual in place and not; the delta as a tensor and as a product hands it out; parts whose sizes differ by
    orders of magnitude keep their own root mean square."""
    T = 5
    for dtype in act_types(ops):
        delta = rnd(T, width, seed=1) * torch.logspace(-2, 2, groups).repeat_interleave(width // groups)
        delta = delta.to(dtype)
        weight = 1.0 + 0.2 * rnd(width, seed=2)
        dev = lambda t: t.to(ops.device)
        normed = plain.group_norm(delta.to(F), weight.to(F), groups, 1e-5)
        close(ops.group_rmsnorm(dev(delta.float()), dev(weight), 1e-5, groups, dtype), normed, dtype, "norm alone")
        for index in (0, 1, 8, 11):
            residual = rnd(T, width, seed=3)
            earlier = [rnd(T, width, seed=10 + j) for j in range(index + 1)]
            depth = rnd(index + 2, seed=4)
            first = dev(earlier[0])
            rest = torch.zeros(13, T, width)
            for j in range(index):
                rest[j] = earlier[j + 1]
            rest = dev(rest)
            x = residual.to(F) + normed
            want = plain.depth_average([e.to(F) for e in earlier] + [x], depth.to(F))
            for in_place in (True, False):
                held = dev(residual.clone())
                got, read = ops.add_group_normed(held, dev(delta), dev(weight), 1e-5, groups, dtype, in_place,
                                                 (first, rest, index, dev(depth)))
                assert (got is held) == in_place
                close(got, want, torch.float32, f"average {index}")
                close(read, want, dtype, f"read {index}")
                close(rest[index], x, torch.float32, f"kept {index}")
                if not in_place:
                    assert torch.equal(held.cpu(), residual)
            got, read = ops.add_group_normed(dev(residual.clone()), dev(delta), dev(weight), 1e-5, groups, None)
            assert read is None
            close(got, x, torch.float32, "sum alone")
        # as a product hands it out (partial sums for few rows)
        if width % 8 == 0:
            a, b = rnd(T, 256, seed=5).to(dtype), (rnd(width, 256, seed=6) / 16.0).to(dtype)
            weights = dev(b)
            ops.prepare_linear(weights)
            want = residual.to(F) + plain.group_norm(a.to(F) @ b.to(F).T, weight.to(F), groups, 1e-5)
            got, _ = ops.add_group_normed(dev(residual.clone()), ops.linear(dev(a), weights), dev(weight), 1e-5, groups, None)
            close(got, want, dtype, "behind a product")


@pytest.mark.parametrize("experts,top,width", [(5, 2, 48), (12, 3, 64), (1, 1, 40), (70, 5, 128), (3, 3, 42)])
def test_router_weights_over_all_experts(ops, experts, top, width):
    """The largest scores choose; the weights are the softmax over all experts, not renormalised."""
    for dtype in act_types(ops):
        for T in (1, 7, 70):
            x, router = rnd(T, width, seed=T).to(dtype), (rnd(experts, width, seed=7) * 0.4).to(dtype)
            chosen, weights = ops.route_topk(x.to(ops.device), router.to(ops.device), None, top, "softmax_all")
            want_ids, want = plain.route(x.to(F), router.to(F), top)
            assert torch.equal(chosen.cpu().long(), want_ids)
            close(weights, want, torch.float32, f"{T} rows")


def test_mixture_alone(ops):
    """The routed feed-forward as a part, few rows and many."""
    from distie_amd.config import config_from_dict

    for experts, top, ff, width in ((5, 2, 12, 48), (3, 1, 16, 64), (4, 4, 10, 42)):
        cfg = nu.make_config([nu.wkv(heads=1, dim=8, rank=2, mlp=nu.moe(experts, top, ff))], width=width, groups=1)
        spec = config_from_dict(cfg).model_spec().layers[0].parts["feed_forward"]
        for dtype in act_types(ops):
            weights = nu.random_weights(cfg, seed=2, dtype=dtype)
            part = build_part("feed_forward", spec)
            part.load({k: v.to(ops.device) for k, v in prefixed(weights, "l0.mlp.").items()})
            part.prepare(ops)
            w = {k: v.to(F) for k, v in weights.items()}
            for T in (1, 6, 80):
                x = rnd(4 * T, width, seed=T).to(dtype)
                z = x.to(F) @ w["l0.mlp.router"].T                   # rows whose choice is clear
                if top < experts:
                    s = torch.sort(z, -1, descending=True).values
                    x = x[(s[:, top - 1] - s[:, top]) > 0.05]
                x = x[:T]
                got = ops.dense(part.forward(ops, x.to(ops.device), StepContext(None, dtype)))
                close(got.float(), plain.mixture(x.to(F), w, "l0.mlp.", cfg["layers"][0]["mlp"]), dtype, f"{T} rows {dtype}", 1.5)


def test_products_of_each_mix(ops):
    """`linear_each`: every input with its own weights, of widths that fit tiles and that do not, few rows and many."""
    for rows, widths in ((1, (48, 48, 16)), (5, (64, 64, 64, 64, 7)), (8, (30, 30, 30, 30, 3)), (16, (128,) * 4 + (32,)),
                         (40, (64,) * 4 + (5,)), (200, (48,) * 4 + (16,))):
        for K in (64, 40):
            for dtype in act_types(ops):
                xs = rnd(len(widths), rows, K, seed=rows).to(dtype)
                weights = [(rnd(n, K, seed=20 + i) / math.sqrt(K)).to(dtype) for i, n in enumerate(widths)]
                held = tuple(w.to(ops.device) for w in weights)
                ops.prepare_linear_each(held)
                got = ops.linear_each(xs.to(ops.device), held, unrounded=(len(widths) - 1,))
                assert got[-1].dtype == torch.float32 and len({t.stride(0) for t in got[:-1] if t.shape == got[0].shape}) == 1
                for k, w in enumerate(weights):
                    close(got[k].float(), xs[k].to(F) @ w.to(F).T, dtype, f"{rows} rows, product {k}", 0.6)


def test_attention_refuses_what_it_does_not_take():
    """A cap that is not positive is an error, and what mixes heads is not plain."""
    from distie_amd.kernels.interface import ScoreExtras

    with pytest.raises(ValueError):
        ScoreExtras(score_cap=0.0)
    assert ScoreExtras().plain and not ScoreExtras(keep_first=3).plain and ScoreExtras(keep_first=3).mixes_heads
    assert ScoreExtras(head_mix=torch.eye(2)).mixes_heads and not ScoreExtras(sinks=torch.zeros(2)).mixes_heads
