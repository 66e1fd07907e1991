"""Each mechanism of the Mepapel decoder alone, as the kernel surface and the parts offer it, against the matching function
of the plain implementation: on the CPU test double and on the GPU kernels (float32 and bfloat16 operands).

A step of a mixer's test is a batch of several requests' rows; cache and state are carried over several steps, with
slots and pages that are used again, and the result must be that of every sequence run at once."""

import pytest
import torch

import mepapel_util as mu
import plain_mepapel as plain
from distie_amd.cache import CacheManager
from distie_amd.config import config_from_dict
from distie_amd.config.model_config import PartSpec
from distie_amd.engine.batch import BatchBuilder, StepEntry
from distie_amd.kernels.interface import RouteRule, ScoreExtras
from distie_amd.parts import FixedState, PagedKV, PagedTensors, StepContext, build_part
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


LENGTHS, CUTS = (13, 1, 9, 6), ((5, 1, 2, 0), (1, 0, 1, 6), (2, 0, 0, 0), (1, 0, 6, 0), (4, 0, 0, 0))
LONG_LENGTHS = (150, 1, 70, 33)
LONG_CUTS = ((100, 1, 2, 0), (17, 0, 64, 33), (2, 0, 4, 0), (1, 0, 0, 0), (30, 0, 0, 0))


def steps_of(ops, cache, cuts, lengths):
    """The batches of a schedule: (rows [(sequence, first row, rows)], the step's meta); cache slots come and go."""
    builder = BatchBuilder(cache, 4096, ops.device, 4096)
    at = [0] * len(lengths)
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
            at[i] += n
        _, meta, _ = builder.build(entries)
        yield rows, meta
        for i, a, n in rows:
            cache.commit(i, n)
            if at[i] == lengths[i]:
                cache.release(i)
        cache.check()
    assert at == list(lengths)


def run_mixer(ops, spec, tensors, seqs, cuts, dtype, slots=3, pages=64):
    """The mixer `spec` with `tensors` over the sequences `seqs` (inputs [n, C]), `cuts[step][i]` rows of sequence i in
    each step -> every sequence's output rows."""
    mixer = build_part("mixer", spec)
    loading = list(mixer.parts()) if hasattr(mixer, "mixers") else [mixer]
    for part in loading:
        own = part.spec.prefix[len(spec.prefix):]
        part.load({k: tensors[own + k].to(ops.device) for k in part.param_specs()})
        part.prepare(ops)
    cache = CacheManager([{"mixer": mixer.cache_requirement()}], 16 if ops.device.type != "cpu" else 4, pages, slots,
                         device=ops.device, dtype=dtype)
    outs = [[] for _ in seqs]
    for rows, meta in steps_of(ops, cache, cuts, [len(s) for s in seqs]):
        x = torch.cat([seqs[i][a:a + n] for i, a, n in rows]).to(dtype).to(ops.device)
        y = ops.dense(mixer.forward(ops, x, StepContext(meta, dtype), cache.layer(0)["mixer"], True)).float().cpu()
        for (i, _, n), own in zip(rows, y.split([n for _, _, n in rows])):
            outs[i].append(own)
    return [torch.cat(o) for o in outs]


def mixer_case(ops, layer, lengths, cuts, width=40, seed=0, slack=1.0, pages=64, side=None, change=None):
    """`side`: of a parallel layer, the mixer of that side alone."""
    cfg = mu.make_config([layer], width=width)
    spec = config_from_dict(cfg).model_spec().layers[0].parts["mixer"]
    prefix, m, function = "l0.mix.", layer["mixer"], plain.MIXERS[layer["type"]]
    if side:
        spec, prefix, m = spec.params["mixers"][side], f"l0.mix.{side}.", m[side]
        function = plain.attention if side == "left" else plain.retention
    for dtype in act_types(ops):
        weights = mu.random_weights(cfg, seed=seed, dtype=dtype)
        if change is not None:
            change(weights)
        seqs = [rnd(n, width, seed=50 + i).to(dtype) for i, n in enumerate(lengths)]
        own = {k[len(prefix):]: v for k, v in weights.items() if k.startswith(prefix)}
        got = run_mixer(ops, spec, own, seqs, cuts, dtype, pages=pages)
        w = {k: v.to(F) for k, v in weights.items()}
        for i, s in enumerate(seqs):
            want = function(s.to(F), w, prefix, m, float(cfg["norm"]["eps"]))
            close(got[i], want, dtype, f"sequence {i} {dtype}", slack)


# ---------------------------------------------------------------- attention in chunks
@pytest.mark.parametrize("sizes", [dict(heads=6, kv_heads=3, dim=12, vdim=16, left_dims=8, size=11, conv=3),
                                   dict(heads=1, kv_heads=1, dim=32, vdim=32, left_dims=32, size=16, conv=0),
                                   dict(heads=5, kv_heads=1, dim=20, vdim=10, left_dims=6, size=None, conv=1),
                                   dict(heads=4, kv_heads=4, dim=80, vdim=40, left_dims=48, size=33, conv=4),
                                   dict(heads=8, kv_heads=2, dim=64, vdim=64, left_dims=32, size=1, conv=2),
                                   dict(heads=2, kv_heads=1, dim=48, vdim=96, left_dims=48, size=70, conv=4)])
def test_attention_in_chunks_alone(ops, sizes):
    """The left mixer as a part over batches in steps: biases, filters, head norms, rotation of neighbours, and keys of the
    query's own chunk only. Sizes that fit no tile, all equal, one key a chunk, no chunks."""
    layer = mu.parallel(scale=0.3, left_base=200.0, **sizes)
    mixer_case(ops, layer, LENGTHS, CUTS, slack=2.0, side="left")
    mixer_case(ops, layer, LONG_LENGTHS, LONG_CUTS, seed=1, slack=2.0, side="left")
    # a portion long enough for the kernels that many rows choose
    mixer_case(ops, layer, (300, 3), ((290, 1), (10, 2)), seed=2, slack=2.0, pages=128, side="left")


def test_one_key_in_every_chunk_stands_out(ops):
    """Attention over the cache alone, with one key whose score towers over all others: at chunk sizes that divide a page,
    that pages divide, and that do neither, for single tokens and portions on both sides of the edges. A query sees the
    value of its own chunk's tall key from that key on, and never another chunk's."""
    H, G, D, n = 4, 2, 32, 210
    for dtype in act_types(ops):
        for size in (5, 16, 48, 64, 100, 150):
            cache = CacheManager([{"mixer": PagedKV(G, D, chunk=size)}], 16, 32, 1, device=ops.device, dtype=dtype)
            q = torch.zeros(n, H * D)
            q[:, ::D] = 4.0
            k, v = rnd(n, G, D, seed=1, scale=0.1), rnd(n, G, D, seed=2, scale=0.1)
            tall = [c + min(7, size - 1) // 2 for c in range(0, n, size)]
            tall = [t for t in tall if t < n]
            k[tall, :, 0] = 10.0
            v[tall, :, :] = torch.arange(1, len(tall) + 1, dtype=torch.float32)[:, None, None]
            view = cache.layer(0)["mixer"]
            cuts, left = [], n
            for wanted in (size - 1, 1, 2, 58, 1, 1, n - 3 - size - 62, 1, 1, 1, 1, n):
                if left and wanted > 0:
                    cuts.append((min(wanted, left),))
                    left -= cuts[-1][0]
            got = []
            for rows, meta in steps_of(ops, cache, cuts, [n]):
                (_, a, count), = rows
                slots = meta.groups[0].slots.long()
                view["k"][slots // 16, :, slots % 16] = k[a:a + count].to(dtype).to(ops.device)
                view["v"][slots // 16, :, :, slots % 16] = v[a:a + count].to(dtype).to(ops.device)
                got.append(ops.paged_attention(q[a:a + count].to(dtype).to(ops.device), meta, 0, view["k"], view["v"], H, G, D,
                                               0.5, None, ScoreExtras(chunk=size)).float().cpu())
            got = torch.cat(got).view(n, H, D)
            want = plain.softmax_attention(q.view(n, H, D).to(dtype).to(F), k.to(dtype).to(F), v.to(dtype).to(F), 0.5,
                                           plain.visible(n, {"size": size}))
            close(got, want, dtype, f"chunks of {size}", slack=1.0 if dtype == torch.float32 else 0.5)
            for at, t in enumerate(tall, 1):
                end = min(n, (t // size + 1) * size)
                assert float((want[t:end] - at).abs().max()) < 1e-3
                assert t % size == 0 or float(want[t - t % size:t].abs().max()) < 0.5


def test_chunks_in_the_cache():
    """Pages of a finished chunk come back when the next one begins, a page that holds the edge of two chunks stays with
    the later one, and a chunk does not go with a window."""
    cache = CacheManager([PagedKV(1, 4, chunk=10), PagedKV(1, 4)], 4, 20, 2, allocate=False)
    cache.add("a")
    held = []
    for n in (9, 1, 1, 8, 1, 13, 6):
        cache.reserve("a", n)
        cache.commit("a", n)
        cache.check()
        held.append([page >= 0 for page in cache.request("a").tables[0]])
    assert held[0] == [True] * 3
    assert held[1] == [False, False, True]                       # token 10 begins a chunk: the page of 8 .. 11 stays
    assert held[2] == [False, False, True] and held[3] == [False, False, True, True, True]
    assert held[4] == [False] * 5                                # the chunk ends with its page
    assert held[5] == [i * 4 + 3 >= 30 for i in range(9)]
    assert held[6] == [i * 4 + 3 >= 30 for i in range(10)]
    assert len(cache.request("a").tables[1]) == 10 and all(p >= 0 for p in cache.request("a").tables[1])
    cache.reset("a")
    assert cache.free_pages() == [20, 20]
    for broken in (dict(chunk=0), dict(chunk=8, window=4), dict(chunk=8, keep_first=2)):
        with pytest.raises(ValueError):
            PagedTensors((), **broken)


def test_rotation_of_neighbours_and_norms_in_one_step(ops):
    """What the kernel behind the projections hands on: q and k convolved, normed by head, their first dimensions turned in
    pairs (2i, 2i + 1) by the token's position, the rest unchanged; in steps of few rows and of many."""
    H, G, D, E, dims, taps = 3, 1, 24, 16, 16, 3
    inv_freq = torch.tensor([100.0 ** (-2 * i / dims) for i in range(dims // 2)])
    weight_q, weight_k = 1 + rnd(D, seed=5, scale=0.3), 1 + rnd(D, seed=6, scale=0.3)
    channels = H * D + G * (D + E)
    for dtype in act_types(ops):
        for n, cuts in ((7, ((3,), (1,), (1,), (2,))), (90, ((50,), (2,), (38,)))):
            product, filters = rnd(n, channels + 8, seed=3).to(dtype), rnd(channels, taps, seed=4, scale=0.5).to(dtype)
            need = PagedKV(G, 32)
            cache = CacheManager([{"mixer": need, "state": FixedState.of((taps - 1, channels), "conv")}], 16, 8, 1,
                                 device=ops.device, dtype=dtype)
            view, state = cache.layer(0)["mixer"], cache.layer(0)["state"]["conv"]
            dev = lambda t: t.to(ops.device)
            got = []
            for rows, meta in steps_of(ops, cache, cuts, [n]):
                (_, a, count), = rows
                got.append(ops.conv_rope_kv_write(dev(product[a:a + count]), dev(filters), state, meta, 0, view["k"], view["v"],
                                                  dev(inv_freq), 1.0, H, G, D, E, 32, True, True, None,
                                                  (dev(weight_q), dev(weight_k), 1e-5), neighbours=True).float().cpu())
                pages = list(cache.request(0).tables[0])
                keys = torch.cat([view["k"][p, 0] for p in pages]).float().cpu()[:n]
                values = torch.cat([view["v"][p, 0].T for p in pages]).float().cpu()[:n]
            u = plain.short_conv(product[:, :channels].to(F), filters.to(F))
            rot = {"base": 100.0, "dims": dims}
            q = plain.rotate(plain.rms(u[:, :H * D].reshape(n, H, D), 1e-5) * weight_q.to(F), rot, True)
            k = plain.rotate(plain.rms(u[:, H * D:(H + G) * D].reshape(n, G, D), 1e-5) * weight_k.to(F), rot, True)
            got = torch.cat(got).view(n, H, 32)
            close(got[..., :D], q, dtype, f"q of {n} rows")
            assert not got[..., D:].any()
            close(keys[:, :D], k[:, 0], dtype, f"k of {n} rows")
            close(values[:, :E], u[:, (H + G) * D:], dtype, f"v of {n} rows")
            halves = plain.rotate(plain.rms(u[:, :H * D].reshape(n, H, D), 1e-5) * weight_q.to(F), rot, False)
            assert float((halves - q).abs().max()) > 0.3             # the other pairing is another function


# ---------------------------------------------------------------- retention
@pytest.mark.parametrize("sizes", [dict(r_heads=3, r_dim=14, r_vdim=10, right_dims=6),
                                   dict(r_heads=1, r_dim=32, r_vdim=32, right_dims=32, decay=(1.0,)),
                                   dict(r_heads=2, r_dim=64, r_vdim=72, right_dims=48, decay=(0.999, 0.3)),
                                   dict(r_heads=2, r_dim=160, r_vdim=20, right_dims=160, decay=(0.97, 0.0)),
                                   dict(r_heads=4, r_dim=128, r_vdim=128, right_dims=2, decay=(0.9, 0.99, 0.5, 0.75))])
def test_retention_alone(ops, sizes):
    """The right mixer as a part: rotation by halves, k's factor, a fixed decay per head, the state carried from step to step
    (row by row in short steps, in chunks in long ones), the norm without a weight and the gate."""
    layer = mu.parallel(right_base=300.0, **sizes)
    mixer_case(ops, layer, LENGTHS, CUTS, slack=3.0, side="right")
    mixer_case(ops, layer, LONG_LENGTHS, LONG_CUTS, seed=1, slack=3.0, side="right")


def test_mixers_side_by_side(ops):
    """Both mixers on one input: half the sum of their results, each normed with its own weight."""
    layer = mu.parallel(heads=4, kv_heads=2, dim=16, vdim=12, size=9)
    mixer_case(ops, layer, LENGTHS, CUTS, slack=4.0)
    mixer_case(ops, layer, LONG_LENGTHS, LONG_CUTS, seed=1, slack=4.0)


# ---------------------------------------------------------------- the delta rule
@pytest.mark.parametrize("sizes", [dict(heads=6, kv_heads=2, dim=12, vdim=20, conv=4),
                                   dict(heads=1, kv_heads=1, dim=32, vdim=32, conv=1),
                                   dict(heads=3, kv_heads=3, dim=10, vdim=6, conv=2),
                                   dict(heads=4, kv_heads=1, dim=64, vdim=96, conv=4),
                                   dict(heads=2, kv_heads=2, dim=128, vdim=72, conv=3),
                                   dict(heads=2, kv_heads=1, dim=200, vdim=24, conv=4)])
def test_delta_rule_mixer_alone(ops, sizes):
    """The delta rule as a part: filters and silu on q, k and v, unit vectors, write strengths and decays, the state carried
    from step to step (row by row in short steps, in chunks in long ones), the norm by head and the gate."""
    layer = mu.delta(**sizes)
    mixer_case(ops, layer, LENGTHS, CUTS, slack=3.0)
    mixer_case(ops, layer, LONG_LENGTHS, LONG_CUTS, seed=1, slack=3.0)


@pytest.mark.parametrize("H,G,D,E", [(3, 3, 8, 12), (4, 2, 20, 40), (2, 1, 64, 64), (2, 2, 130, 80), (1, 1, 256, 16)])
def test_delta_scan_with_fast_and_slow_heads(ops, H, G, D, E):
    """The recurrence alone: decays from none to complete in one sequence (the softplus far out on both sides), write strengths
    from nothing to everything, keys that repeat (so that what is written under a key must take back what stood there),
    rows of zeros, over rows enough for several chunks, then row by row from the state that the long step left."""
    lengths = (203, 3, 65, 64)
    for dtype in act_types(ops):
        qkv, beta, decay = [], [], []
        for i, n in enumerate(lengths):
            x = rnd(n, 2 * G * D + H * E + 3, seed=i)
            x[5::7, G * D:2 * G * D] = x[4:5, G * D:2 * G * D] if n > 5 else 0.0         # the same key again and again
            x[9::31, :2 * G * D] = 0.0
            qkv.append(x.to(dtype))
            beta.append((rnd(n, H, seed=20 + i, scale=3.0)).to(dtype))
            decay.append((rnd(n, H, seed=40 + i, scale=3.0) + torch.linspace(-14, 6, n)[:, None]).to(dtype))
        a_log, dt_bias = torch.linspace(-6.0, 2.0, H), torch.linspace(-1.0, 1.0, H)
        want = []
        for x, b, a in zip(qkv, beta, decay):
            n, x = x.shape[0], x.to(F)
            unit = lambda z: z / torch.sqrt((z * z).sum(-1, keepdim=True) + 1e-6)
            own = lambda z: unit(z.reshape(n, G, D)).repeat_interleave(H // G, dim=1)
            f = torch.exp(-torch.exp(a_log.to(F)) * plain.softplus(a.to(F) + dt_bias.to(F)))
            want.append(plain.delta_scan(own(x[:, :G * D]) * 0.3, own(x[:, G * D:2 * G * D]),
                                         x[:, 2 * G * D:2 * G * D + H * E].reshape(n, H, E), torch.sigmoid(b.to(F)), f).reshape(n, H * E))
        dev = lambda t: t.to(ops.device)
        cache = CacheManager([{"mixer": FixedState.of((H, D, E))}], 16, 8, len(lengths), device=ops.device)
        state = cache.layer(0)["mixer"]["state"]
        got = [[] for _ in lengths]
        cuts = [[max(n - 5, 1) for n in lengths]] + [[1 if n - max(n - 5, 1) > k else 0 for n in lengths] for k in range(5)]
        for rows, meta in steps_of(ops, cache, cuts, lengths):
            part = lambda seqs: dev(torch.cat([seqs[i][a:a + n] for i, a, n in rows]))
            y = ops.delta_scan(part(qkv), part(beta), part(decay), dev(a_log), dev(dt_bias), state, meta, H, G, D, E, 0.3, 1e-6).cpu()
            for (i, _, n), own_rows in zip(rows, y.split([n for _, _, n in rows])):
                got[i].append(own_rows)
        for i in range(len(lengths)):
            close(torch.cat(got[i]), want[i], torch.float32, f"sequence {i} {dtype}", slack=3.0)


def test_delta_rule_takes_back_what_stood_under_a_key(ops):
    """A value written with full strength under a key is what that key reads from then on, whatever stood there, hundreds of
    tokens with other (orthogonal) keys later, in portions and token by token."""
    D = E = 16
    n = 330
    dev = lambda t: t.to(ops.device)
    for dtype in act_types(ops):
        x = torch.zeros(n, 2 * D + E)
        keys = 1 + torch.arange(n) % (D - 1)                        # keys 1 .. D - 1 in turn, key 0 at two places
        keys[[3, 40]] = 0
        x[torch.arange(n), D + keys] = 2.0
        x[:, 2 * D:] = rnd(n, E, seed=1)
        x[:, 0] = 3.0                                               # everyone asks for key 0
        beta, decay = torch.full((n, 1), 30.0), torch.full((n, 1), -30.0)      # full strength, nothing forgotten
        x, beta, decay = x.to(dtype), beta.to(dtype), decay.to(dtype)
        cache = CacheManager([{"mixer": FixedState.of((1, D, E))}], 16, 32, 1, device=ops.device)
        got = []
        for rows, meta in steps_of(ops, cache, [(64,), (2,), (1,), (100,), (16,), (3,), (140,), (1,), (1,), (2,)], [n]):
            (_, a, count), = rows
            got.append(ops.delta_scan(dev(x[a:a + count]), dev(beta[a:a + count]), dev(decay[a:a + count]), dev(torch.zeros(1)),
                                      dev(torch.zeros(1)), cache.layer(0)["mixer"]["state"], meta, 1, 1, D, E, 1.0, 1e-6).cpu())
        got, v = torch.cat(got), x[:, 2 * D:].float()
        assert float(got[:3].abs().max()) < 1e-4
        close(got[3:40], v[3].expand(37, E), torch.float32, "the first value", slack=4.0)
        close(got[40:], v[40].expand(n - 40, E), torch.float32, "the value that took its place", slack=4.0)


# ---------------------------------------------------------------- the state-space mixer in this design's sizes
@pytest.mark.parametrize("sizes", [dict(heads=6, vdim=10, state=14, groups=3, conv=3, norm_groups=2),
                                   dict(heads=1, vdim=32, state=16, groups=1, conv=1, norm_groups=1),
                                   dict(heads=4, vdim=40, state=24, groups=4, conv=4, norm_groups=4)])
def test_state_space_mixer_alone(ops, sizes):
    layer = mu.mamba2(**sizes)
    mixer_case(ops, layer, LENGTHS, CUTS, slack=2.0)
    mixer_case(ops, layer, LONG_LENGTHS, LONG_CUTS, seed=1, slack=2.0)


# ---------------------------------------------------------------- feed-forwards
def test_clamped_feed_forward(ops):
    """g * sigmoid(slope g) * (u + shift) behind clamps (the gate from above only): alone, and as products of few rows and
    many, on sizes that fit the packed kernels and that do not. Values lie on both sides of every clamp."""
    limit, slope, shift = 0.8, 1.702, 1.0
    dev = lambda t: t.to(ops.device)

    def bent(g, u):
        g, u = g.clamp(max=limit), u.clamp(-limit, limit)
        return g * torch.sigmoid(slope * g) * (u + shift)

    for dtype in act_types(ops):
        for inter in (44, 64, 7):
            x = rnd(9, 2 * inter, seed=1, scale=2.0).to(dtype)
            want = bent(x.to(F)[:, :inter], x.to(F)[:, inter:])
            close(ops.clamped_glu(dev(x), limit, slope, shift), want, dtype, f"alone, {inter}")
            assert float(((x.float()[:, :inter] < -limit) & (want.abs() > 0.01)).sum()) > 0     # no clamp from below on the gate
        for T, K, inter in ((1, 40, 44), (5, 64, 48), (12, 128, 96), (40, 256, 64), (120, 72, 40), (300, 64, 128), (3, 42, 10)):
            w, x = rnd(2 * inter, K, seed=2, scale=K ** -0.5 * 1.5).to(dtype), rnd(T, K, seed=3).to(dtype)
            w = dev(w)
            ops.prepare_linear(w, gated=True, role="gate_up")
            product = x.to(F) @ w.cpu().to(F).T
            got = ops.dense(ops.linear_clamped_glu(dev(x), w, limit, slope, shift))
            close(got, bent(product[:, :inter], product[:, inter:]), dtype, f"product {T} x {K} x {inter}", slack=2.0)


def feed_forward_case(ops, mlp, T, width=40, seed=0):
    cfg = mu.make_config([mu.delta(mlp=mlp)], width=width)
    spec = config_from_dict(cfg).model_spec().layers[0].parts["feed_forward"]
    for dtype in act_types(ops):
        weights = mu.random_weights(cfg, seed=seed, dtype=dtype)
        part = build_part("feed_forward", spec)
        part.load({k: weights["l0.mlp." + k].to(ops.device) for k in part.param_specs()})
        part.prepare(ops)
        x = rnd(4 * T + 60, width, seed=7).to(dtype)
        w = {k: v.to(F) for k, v in weights.items()}
        if mlp["kind"] == "moe":                                    # rows whose choice is no close call
            choice = torch.sigmoid(x.to(F) @ w["l0.mlp.router"].T) + w["l0.mlp.correction"]
            x = x[[i for i in range(len(x)) if mu.router_gap(choice[i], mlp["router"]) > 0.01]]
        x = x[:T]
        assert len(x) == T
        got = ops.dense(part.forward(ops, x.to(ops.device), StepContext(None, dtype)))
        close(got, plain.feed_forward(x.to(F), w, "l0.mlp.", mlp), dtype, f"{T} rows {dtype}", slack=2.0)


@pytest.mark.parametrize("mlp", [mu.dense(24, 0.7), mu.moe(6, 2, 12, 3, 2, 1.3, 10), mu.moe(8, 3, 16, 4, 2, 0.5, 0),
                                 mu.moe(12, 4, 8, 2, 1, 2.5, 24), mu.moe(5, 5, 6, 0, 0, 1.0, 8), mu.moe(1, 1, 16, 1, 1, 1.0, 16),
                                 mu.moe(7, 2, 10, 7, 3, 1.5, 6), mu.moe(24, 6, 8, 6, 3, 1.0, 40)])
def test_feed_forwards_alone(ops, mlp):
    """Dense and mixture, with and without groups and a shared expert, one expert, one expert a group, every expert chosen;
    for few rows (router and hidden values in one launch), some, and many."""
    for T in (1, 5, 70):
        feed_forward_case(ops, mlp, T)
    feed_forward_case(ops, mlp, 9, width=42, seed=1)                 # a width that fits no 16-byte piece


def test_router_groups_and_negative_choice_scores(ops):
    """Experts outside the kept groups are never chosen, also where every choice score inside is negative; a group's
    strength is the sum of its two largest scores, not its largest; weights leave the correction out, add up to the scale,
    and come with the largest choice score first."""
    E, C, top = 8, 16, 3
    dev = lambda t: t.to(ops.device)
    for dtype in act_types(ops):
        x = rnd(40, C, seed=1).to(dtype)
        weight = rnd(E + 1, C, seed=2, scale=0.3).to(dtype)
        correction = torch.tensor([-3.0, -3.0, -3.1, -3.2, 0.9, -9.0, -0.2, -0.3])
        rule = RouteRule(dev(correction), 2, 1, 2.5, True)
        experts, gates = ops.route_topk(dev(x), dev(weight), None, top, "sigmoid_share", rule)
        s = torch.sigmoid(x.to(F) @ weight.to(F).T)
        for t in range(len(x)):
            choice = s[t, :E] + correction.to(F)
            want = plain.choose(s[t, :E], choice, {"experts": E, "top": top, "scale": 2.5, "groups": {"count": 2, "keep": 1}})
            assert experts[t].tolist() == list(want), t
            assert all(e >= 4 for e in want)
            close(gates[t, :top].cpu(), torch.tensor(list(want.values()), dtype=F), torch.float32, "weights")
            assert abs(float(gates[t, :top].sum()) - 2.5) < 1e-5
        close(gates[:, top], s[:, E], torch.float32, "the shared expert's gate", slack=2.0)
        # both kept groups negative throughout: the best of them, not a zero of a closed group
        low = RouteRule(dev(torch.tensor([-5.0, -5.0, -6.0, -6.0, -7.0, -7.0, -8.0, -8.0])), 4, 2, 1.0, True)
        experts, _ = ops.route_topk(dev(x), dev(weight), None, 4, "sigmoid_share", low)
        assert {tuple(sorted(row)) for row in experts.tolist()} == {(0, 1, 2, 3)}
        # one large score does not make a strong group
        pair = RouteRule(dev(torch.tensor([2.0, -9.0, 0.9, 0.9])), 2, 1, 1.0, False)
        experts, _ = ops.route_topk(dev(x), dev(weight[:4].contiguous()), None, 1, "sigmoid_share", pair)
        assert set(experts.view(-1).tolist()) <= {2, 3}


def test_residual_multiplier_is_part_of_the_norm(ops):
    norm = build_part("norm", PartSpec("rmsnorm", "", {"size": 24, "eps": 1e-5, "weight_name": "w", "gain": 0.37}))
    weight = (1 + rnd(24, seed=1, scale=0.3)).to(torch.bfloat16)
    norm.load({"w": weight.to(ops.device)})
    assert norm.weight.dtype == torch.float32
    x, residual = rnd(5, 24, seed=2), rnd(5, 24, seed=3)
    held = residual.clone().to(ops.device)
    ops.add_normed(held, x.to(ops.device), norm.weight, norm.eps)
    close(held, residual.to(F) + 0.37 * plain.rms(x.to(F), 1e-5) * weight.to(F), torch.float32)


def test_what_the_surface_refuses():
    """On the host, before anything is launched: chunks with a window, with borrowed keys; groups that leave fewer experts
    than are chosen; a gate for a shared expert that is not there."""
    attention = dict(hidden_size=8, num_heads=2, num_kv_heads=1, head_dim=8, output_gate=False)
    for broken in (dict(chunk=4, window=4), dict(chunk=0), dict(chunk=4, kv_from=0)):
        with pytest.raises(ValueError):
            build_part("mixer", PartSpec("conv_gated_attention", "", {**attention, **broken}))
    experts = dict(hidden_size=8, num_experts=6, top=3, expert_size=4, router_bias=False, scoring="sigmoid_share", route_in_hidden=True)
    for broken in (dict(groups=3, groups_kept=1), dict(groups=4, groups_kept=4), dict(shared_gate=True),
                   dict(shared_size=4), dict(scoring="sigmoid", correction=True)):
        with pytest.raises(ValueError):
            build_part("feed_forward", PartSpec("routed_experts", "", {**experts, **broken}))
    with pytest.raises(ValueError):
        build_part("mixer", PartSpec("gated_delta_rule", "", dict(hidden_size=8, num_heads=3, num_kv_heads=2, head_dim=4,
                                                                  conv_taps=2, eps=1e-5)))
    with pytest.raises(ValueError):
        build_part("mixer", PartSpec("retention", "", dict(hidden_size=8, num_heads=2, head_dim=4, eps=1e-5, decay=(0.5,))))
