"""The Fogorax design on the GPU kernels against the plain float64 form of its equations (oracle/fogorax.py): every mechanism
alone, then the model — prompts, decoding, portions, batches, slots — and greedy generation through the scheduler."""
import math

import pytest
import torch

from oracle import fogorax as O
import fogorax_cases as C

pytestmark = pytest.mark.gpu
DEV = "cuda"
LIMIT = {torch.float32: 1e-4, torch.bfloat16: 6e-2}      # rows of logits (C.row_errors)
OP = {torch.float32: 2e-5, torch.bfloat16: 1e-2}         # operators, relative to the size of the result
DTYPES = [torch.float32, torch.bfloat16]
BF = torch.bfloat16


def lim(dtype):
    return LIMIT[dtype]


def rnd(shape, seed, dtype, scale=1.0):
    return (torch.randn(shape, generator=torch.Generator().manual_seed(seed)) * scale).to(dtype)


def close(got, want, tol):
    got, want = got.double().cpu(), want.double()
    err = (got - want).norm() / want.norm()
    worst = (got - want).abs().max() / want.abs().max()
    assert err < tol and worst < 4 * tol, (float(err), float(worst))


def cache_of(layers, slots, capacity, dtype, starts):
    """a slot cache whose sequences (slot -> tokens it holds already) are taken in this order"""
    from timeviper_amd.model.llm import SlotStateCache
    c = SlotStateCache(layers, slots, dtype, DEV, capacity)
    for _ in range(slots):
        c.alloc()
    for s, n in starts.items():
        c._len[s] = n
    return c


# ------------------------------------------------------------------ embedding, norm, shift, gated products
@pytest.mark.parametrize("dtype", DTYPES)
def test_embedding_with_positions(dtype):
    from timeviper_amd import kernels as K
    table, pos = rnd((11, 76), 1, dtype), rnd((40, 76), 2, dtype)
    starts, counts = {3: 0, 1: 17, 0: 39}, [5, 3, 1]
    c = cache_of([("tokens", 4)], 4, 40, dtype, starts)
    ids = torch.tensor([4, 0, 10, 4, 2, 7, 7, 1, 9])
    x, h = K.embed_scaled(ids.to(DEV), table.to(DEV), positions=pos.to(DEV), plan=c.plan(list(starts), counts))
    places = [0, 1, 2, 3, 4, 17, 18, 19, 39]
    want = table.float()[ids] + pos.float()[places]
    assert torch.equal(x.cpu(), want) and torch.equal(h.cpu(), want.to(dtype))      # the stream is 32-bit
    p = c.plan([1, 0], [1, 1])                                # single tokens: the places come from the device
    x, _ = K.embed_scaled(ids[:2].to(DEV), table.to(DEV), positions=pos.to(DEV), plan=p)
    assert torch.equal(x.cpu(), table.float()[ids[:2]] + pos.float()[[17, 39]])


def shift_case(D, counts, starts, dtype, seed):
    x, y = rnd((sum(counts), D), seed, torch.float32), rnd((sum(counts), D), seed + 1, dtype, 0.3)
    gain, w, s = rnd((), seed + 2, dtype, 0.2) + 1.3, rnd((D,), seed + 3, dtype, 0.3) + 1, rnd((D,), seed + 4, dtype, 0.5)
    state = rnd((len(counts) + 2, 3, 2, D), seed + 5, torch.float32)
    return x, y, gain.to(dtype), w.to(dtype), s, state


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("D", [76, 512, 1000, 2048, 4096, 8192, 9000])
@pytest.mark.parametrize("waits", [True, False])
def test_norm_and_token_shift_over_a_ragged_step(D, dtype, waits):
    """First tokens of sequences, continued ones with odd and even places, portions of 1 .. 70 tokens; what waits is added first."""
    from timeviper_amd import kernels as K
    eps, counts = 1e-5, [1, 2, 70, 5, 1, 2, 3, 66]
    starts = {4: 0, 8: 7, 2: 0, 0: 12, 1: 33, 6: 8, 9: 1, 3: 64}
    x, y, gain, w, s, state = shift_case(D, counts, starts, dtype, 10)
    c = cache_of([("state", (3, 2, D))], 10, 200, dtype, starts)
    c.state(0).copy_(state)
    plan = c.plan(list(starts), counts)
    x1, h, hs = K.norm_shift(x.to(DEV), gain.to(DEV), eps, *((y.to(DEV), w.to(DEV)) if waits else (None, None)), shift=s.to(DEV),
                             state=c.state(0)[:, 1], plan=plan)
    xs = x.double() + (O.rms(y.double(), eps) * w.double() if waits else 0)
    want = O.norm_scalar(xs, gain.double(), eps)
    close(x1, xs, 2e-6)
    close(h, want, OP[dtype])
    at, new = 0, state.clone().double()
    for (slot, st), n in zip(starts.items(), counts):
        hh = want[at:at + n]
        front = state[slot, 1, (st - 1) & 1].double() if st else torch.zeros(D).double()
        sh = O.token_shift(torch.cat([front[None], hh]), s.double())[1:]
        close(hs[at:at + n], sh, OP[dtype])
        new[slot, 1, (st + n - 1) & 1] = hh[-1]
        at += n
    close(c.state(0), new, 2e-6)                              # the last h of every sequence in 32 bits; nobody else's rows


@pytest.mark.parametrize("D,T", [(256, 9000), (2048, 2500), (4096, 8200)])
def test_norm_and_token_shift_of_long_prompts(D, T):
    """Several rows a wave: the edges between the groups."""
    from timeviper_amd import kernels as K
    x, y, gain, w, s, state = shift_case(D, [T - 3, 3], {0: 0, 1: 0}, BF, 30)
    c = cache_of([("state", (3, 2, D))], 4, T, BF, {0: 0, 1: 0})
    plan = c.plan([0, 1], [T - 3, 3])
    x1, h, hs = (t.float() for t in K.norm_shift(x.to(DEV), gain.to(DEV), 1e-6, y.to(DEV), w.to(DEV), s.to(DEV), c.state(0)[:, 2], plan))
    xd, yd = x.to(DEV), y.to(DEV).float()
    xs = xd + yd * torch.rsqrt(yd.pow(2).mean(-1, keepdim=True) + 1e-6) * w.to(DEV).float()
    want = xs * torch.rsqrt(xs.pow(2).mean(-1, keepdim=True) + 1e-6) * gain.to(DEV).float()
    front = torch.cat([torch.zeros(1, D, device=DEV), want[:-1]])
    front[T - 3] = 0
    sh = want + (front - want) * s.to(DEV).float()
    for got, ref, tol in ((x1, xs, 1e-5), (h, want, 1e-2), (hs, sh, 1e-2)):
        assert float(((got - ref).abs().amax(-1) / ref.abs().amax(-1)).max()) < tol
    assert float((c.state(0)[0, 2, (T - 4) & 1] - want[T - 4]).abs().max()) < 1e-4


def test_eps_is_inside_the_root_and_the_shift_reads_the_unshifted_h():
    from timeviper_amd import kernels as K
    x = torch.full((3, 64), 1e-3, device=DEV)
    x[1] *= 2
    c = cache_of([("state", (1, 2, 64))], 1, 8, torch.float32, {})
    one = torch.ones((), device=DEV)
    _, h, hs = K.norm_shift(x, one, 1e-6, shift=torch.ones(64, device=DEV), state=c.state(0)[:, 0], plan=c.plan([0], [3]))
    assert abs(float(h[0, 0]) - 1e-3 / math.sqrt(2e-6)) < 1e-6
    assert float(hs[0].abs().max()) == 0 and torch.allclose(hs[1:], h[:-1], atol=1e-6)      # shift 1: the previous token's h, as it was


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("n", [10, 24, 264])
def test_gated_products(dtype, n):
    from timeviper_amd import kernels as K
    a, b, table = rnd((7, 2 * n), 40, dtype, 3.0), rnd((7, n), 41, dtype), rnd((13, 3 * n), 42, dtype)
    ids = torch.tensor([12, 0, 5, 5, 1, 7, 3])
    out = torch.zeros((7, 3 * n), dtype=dtype, device=DEV)
    K.gated_mul(a.to(DEV)[:, n:], b.to(DEV), K.ACT_SIGMOID, out=out[:, n:2 * n])
    close(out[:, n:2 * n], O.sigmoid(a[:, n:].double()) * b.double(), OP[dtype])
    assert float(out[:, :n].abs().max()) == 0 and float(out[:, 2 * n:].abs().max()) == 0
    got = K.gated_mul(a.to(DEV)[:, :n], table.to(DEV)[:, n:2 * n], K.ACT_GELU_TANH, ids=ids.to(DEV))
    close(got, O.gelu_tanh(a[:, :n].double()) * table[ids, n:2 * n].double(), OP[dtype])
    x = rnd((7, n), 43, torch.float32)
    s, h = K.residual_add(x.to(DEV), a.to(DEV)[:, :n])
    close(s, x.double() + a[:, :n].double(), 1e-6)
    assert torch.equal(h, s.to(dtype))
    buf = torch.zeros((9, n), dtype=dtype, device=DEV)
    K.scatter_rows(a.to(DEV)[:3, n:], torch.tensor([8, 0, 4], dtype=torch.int32, device=DEV), buf)
    assert torch.equal(buf[[8, 0, 4]].cpu(), a[:3, n:]) and float(buf[[1, 2, 3, 5, 6, 7]].abs().max()) == 0


# ------------------------------------------------------------------ attention in a window
SHAPES = [(6, 3, 18, 22), (8, 2, 64, 96), (4, 4, 96, 40), (8, 4, 128, 128), (12, 1, 128, 64), (2, 1, 192, 256), (2, 2, 40, 8), (7, 1, 64, 128), (20, 1, 32, 24),
          (10, 1, 128, 200)]


def attention_case(H, G, d, e, starts, counts, capacity, dtype, seed=50):
    T, W = sum(counts), G * (d + e)
    return rnd((T, H * d), seed, dtype), rnd((T, H * e), seed + 1, dtype), rnd((max(starts) + 2, capacity, W), seed + 2, dtype)


def attention_want(q, g, cache, H, G, d, e, starts, counts, scale, window, keep):
    out, at = [], 0
    for (slot, st), n in zip(starts.items(), counts):
        k, v = cache[slot, :st + n].double().split([G * d, G * e], dim=1)
        o = O.window_attention(q[at:at + n].double().view(n, H, d), k.reshape(-1, G, d), v.reshape(-1, G, e), scale, window, keep, start=st)
        out.append(o.reshape(n, H * e) * O.sigmoid(g[at:at + n].double()))
        at += n
    return torch.cat(out)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,G,d,e", SHAPES)
@pytest.mark.parametrize("window,keep", [(1, 0), (33, 5), (96, 97), (500, 3)])
def test_window_attention_of_a_ragged_step(H, G, d, e, window, keep, dtype):
    """Whole prompts and portions behind earlier tokens; windows shorter and longer than tiles and sequences; a gate; results into
    a slice of a wider row."""
    from timeviper_amd import kernels as K
    starts, counts = {2: 0, 0: 140, 3: 97, 1: 0}, [1, 33, 4, 150]
    q, g, kv = attention_case(H, G, d, e, starts, counts, 190, dtype)
    c = cache_of([("tokens", G * (d + e))], 5, 190, dtype, starts)
    c.tokens(0).copy_(kv)
    plan, scale = c.plan(list(starts), counts), 0.7 * d ** -0.5
    out = torch.zeros((sum(counts), H * e + 16), dtype=dtype, device=DEV)
    K.attention_window(q.to(DEV).view(-1, H, d), c.tokens(0), plan, G, scale, window, keep, gate=g.to(DEV).view(-1, H, e),
                       out=out[:, :H * e].unflatten(1, (H, e)))
    close(out[:, :H * e], attention_want(q, g, kv, H, G, d, e, starts, counts, scale, window, keep), OP[dtype])
    assert float(out[:, H * e:].abs().max()) == 0


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,G,d,e", SHAPES)
@pytest.mark.parametrize("window,keep", [(1, 0), (40, 5), (130, 70), (900, 0), (2000, 900)])
def test_window_attention_of_single_tokens(H, G, d, e, window, keep, dtype):
    """Few and many keys for the splits, the newest key from the step's own rows (which reach the cache, and only there)."""
    from timeviper_amd import kernels as K
    starts = {1: 0, 4: 22, 0: 63, 2: 64, 5: 250, 3: 801, 6: 16}
    B = len(starts)
    q, g, kv = attention_case(H, G, d, e, starts, [1] * B, 810, dtype)
    c = cache_of([("tokens", G * (d + e))], max(starts) + 2, 810, dtype, starts)
    new = rnd((B, G * (d + e)), 60, dtype)
    want_kv = kv.clone()
    for b, (s, st) in enumerate(starts.items()):
        want_kv[s, st] = new[b]
    plan, scale = c.plan(list(starts), [1] * B), 0.8 * d ** -0.5
    want = attention_want(q, g, want_kv, H, G, d, e, starts, [1] * B, scale, window, keep)
    for fresh in (True, False):                               # without: another layer's rows, in the cache already
        c.tokens(0).copy_(kv if fresh else want_kv)
        o = K.attention_window_decode(q.to(DEV).view(B, H, d), c.tokens(0), plan, G, scale, window, keep, gate=g.to(DEV).view(B, H, e),
                                      fresh=new.to(DEV) if fresh else None)
        close(o.reshape(B, H * e), want, OP[dtype])
        assert torch.equal(c.tokens(0).cpu(), want_kv)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("d,e", [(64, 64), (128, 96), (18, 22)])
@pytest.mark.parametrize("key", [0, 6, 7, 95, 96, 191, 383, 384, 500])
def test_one_key_that_stands_out_is_seen_exactly_in_its_window(d, e, key, dtype):
    """One huge score: every query that sees the key returns its value, every other one does not.  Window 96, 7 kept; queries in a
    prompt, in portions and one by one."""
    from timeviper_amd import kernels as K
    H, G, n, window, keep = 2, 1, 520, 96, 7
    q, kv = torch.full((n, H * d), 1.0), rnd((1, n, d + e), 70, torch.float32, 0.01)
    kv[0, key, :d] = 3.0
    kv[0, :, d:] = 0.0
    kv[0, key, d:] = 1.0
    q, kv = q.to(dtype), kv.to(dtype)
    sees = torch.tensor([key <= i and (i - key < window or key < keep) for i in range(n)])

    def check(o, lo):
        v = o.float().cpu().view(-1, H * e)
        s = sees[lo:lo + len(v)]
        assert bool((v[s] > 0.99).all()) and bool((v[~s] == 0).all()), (key, lo)

    for cuts in ([n], [96, 1, 190, 97, 2, 134]):
        c = cache_of([("tokens", d + e)], 1, n, dtype, {})
        c.tokens(0).copy_(kv)
        at = 0
        for m in cuts:
            plan = c.plan([0], [m])
            f = K.attention_window_decode if plan.decode else K.attention_window
            check(f(q[at:at + m].to(DEV).view(m, H, d), c.tokens(0), plan, G, 0.5, window, keep), at)
            c.commit(plan)
            at += m
    for lo in {key, key + window - 1, key + window, n - 1}:   # single tokens around the window's edge
        if lo < n:
            c._len[0], c._decode_plan = lo, None
            check(K.attention_window_decode(q[lo:lo + 1].to(DEV).view(1, H, d), c.tokens(0), c.plan([0], [1]), G, 0.5, window, keep), lo)


def test_far_key_among_thousands():
    """A kept key far back and one just inside a long window, in a prompt and for a single token."""
    from timeviper_amd import kernels as K
    H, G, d, n, window, keep = 4, 2, 128, 6000, 2048, 3
    kv = rnd((1, n, G * 2 * d), 71, torch.float32, 0.3)
    kv[0, [2, n - window], :d] = 2.0                          # key head 0 only
    kv, q = kv.to(BF), torch.full((n, H * d), 0.5).to(BF)
    c = cache_of([("tokens", G * 2 * d)], 1, n, BF, {0: n - 300})
    c.tokens(0).copy_(kv)
    plan = c.plan([0], [300])
    o = K.attention_window(q[:300].to(DEV).view(-1, H, d), c.tokens(0), plan, G, 0.2, window, keep).float().cpu()
    v = kv[0, :, G * d:G * d + d].float()
    want_last, want_next = (v[2] + v[n - window]) / 2, v[2]
    assert float((o[299, :2] - want_last).abs().max()) < 1e-2
    c._len[0] = n - 1
    for w, want in ((window, want_last), (window - 1, want_next)):
        o1 = K.attention_window_decode(q[:1].to(DEV).view(1, H, d), c.tokens(0), c.plan([0], [1]), G, 0.2, w, keep).float().cpu()
        assert float((o1[0, :2] - want).abs().max()) < 1e-2
        c._decode_plan = None


# ------------------------------------------------------------------ fused decode operators
@pytest.mark.parametrize("M,D,n1,ff", [(1, 64, 24, 0), (2, 384, 70, 33), (4, 2048, 513, 512), (3, 4096, 63, 1), (1, 8192, 33, 40), (4, 4096, 1, 3000),
                                       (1, 9000, 5, 9), (2, 2056, 4097, 700), (1, 2048, 5120, 5632), (4, 2560, 3072, 6000)])
def test_input_products_of_one_launch(M, D, n1, ff):
    from timeviper_amd import kernels as K
    x, x2 = rnd((M, D), 80, BF), rnd((M, D), 81, BF)
    weight, bias = rnd((n1 + 2 * ff, D), 86, BF, D ** -0.5), rnd((2 * ff,), 87, BF)
    u = torch.zeros((M, ff + 16), dtype=BF, device=DEV)
    y = K.gemv_pair(x.to(DEV), x2.to(DEV), weight.to(DEV), n1, bias.to(DEV) if ff else None, act_out=u[:, 8:8 + ff])
    close(y, x.double() @ weight[:n1].double().T, 1e-2)
    if ff:
        z, v = (x2.double() @ weight[n1:].double().T + bias.double()).split(ff, dim=1)
        close(u[:, 8:8 + ff], O.gelu_tanh(z) * v, 1e-2)
    assert float(u[:, :8].abs().max()) == 0 and float(u[:, 8 + ff:].abs().max()) == 0


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("D", [76, 384, 2048, 4096])
def test_norm_and_token_shift_of_single_tokens(D, dtype):
    """One row per sequence, first tokens among them, step after step on one plan; against the whole sequences."""
    from timeviper_amd import kernels as K
    starts, steps = {2: 0, 0: 3, 5: 0}, 7
    c = cache_of([("state", (2, 2, D))], 6, 32, dtype, {})
    gain, s, w = rnd((), 1, dtype) + 1.2, rnd((D,), 2, dtype, 0.5), rnd((D,), 3, dtype) + 1
    gain = gain.to(dtype)
    xs = {b: rnd((n + steps, D), 10 + b, torch.float32) for b, n in starts.items()}
    ys = {b: rnd((n + steps, D), 20 + b, dtype) for b, n in starts.items()}
    run = lambda plan, x, y: K.norm_shift(x.to(DEV), gain.to(DEV), 1e-5, y.to(DEV), w.to(DEV), s.to(DEV), c.state(0)[:, 1], plan)
    p = c.plan([0], [3])
    run(p, xs[0][:3], ys[0][:3])
    c.commit(p)
    got = []
    for t in range(steps):
        p = c.plan(list(starts), [1] * 3)
        got.append(run(p, *(torch.stack([v[b][n + t] for b, n in starts.items()]) for v in (xs, ys))))
        c.commit(p)
    for i, (b, n) in enumerate(starts.items()):
        x = xs[b].double() + O.rms(ys[b].double(), 1e-5) * w.double()
        h = O.norm_scalar(x, gain.double(), 1e-5)
        for j, ref in ((0, x), (1, h), (2, O.token_shift(h, s.double()))):
            close(torch.stack([g[j][i] for g in got]), ref[n:], 2e-6 if j == 0 else OP[dtype])


@pytest.mark.parametrize("M,D,N", [(1, 64, 40), (2, 512, 70), (4, 7680, 513), (1, 7680, 2048), (1, 13312, 100), (4, 15104, 30), (3, 16384, 384)])
def test_output_product_on_the_stream(M, D, N):
    from timeviper_amd import kernels as K
    x, weight, bias, res = rnd((M, D), 90, BF), rnd((N, D), 92, BF, D ** -0.5), rnd((N,), 93, BF), rnd((M, N), 94, torch.float32)
    for b in (bias, None):
        xs, hs = K.gemv_add(x.to(DEV), weight.to(DEV), res.to(DEV), None if b is None else b.to(DEV))
        close(xs, res.double() + x.double() @ weight.double().T + (0 if b is None else b.double()), 2e-6)
        assert torch.equal(hs, xs.to(BF))


@pytest.mark.parametrize("M,n,N", [(3, 24, 384), (4, 256, 2048), (1, 8, 64), (2, 128, 4096)])
def test_product_of_token_rows(M, n, N):
    from timeviper_amd import kernels as K
    z, u, weight, table = rnd((M, n), 95, BF, 2.0), rnd((M, n), 96, BF), rnd((N, n), 97, BF, n ** -0.5), rnd((9, 3 * n), 98, BF)
    ids = torch.tensor([8, 0, 3, 3][:M])
    for rows, by, got in ((u, None, K.gemv_glu(z.to(DEV), u.to(DEV), weight.to(DEV))),
                          (table[:, n:2 * n], ids, K.gemv_glu(z.to(DEV), table.to(DEV)[:, n:2 * n], weight.to(DEV), ids=ids.to(DEV)))):
        f = (O.gelu_tanh(z.double()) * (rows if by is None else rows[by]).double()).to(BF).double()
        close(got, f @ weight.double().T, 1e-2)


# ------------------------------------------------------------------ the model
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", list(C.CONFIGS))
def test_prompt_against_the_equations(name, dtype, tmp_path):
    from timeviper_amd.model.llm import TextEngine
    cfg, tensors, llm = C.build(name, dtype, DEV, tmp_path)
    toks = C.prompt(cfg, min(cfg["max_positions"], 230), 5)
    want = O.model(cfg, tensors, toks)
    err = C.row_errors(C.run(TextEngine(llm), 0, toks, []), want)
    assert float(err.max()) < lim(dtype) and float(err.median()) < lim(dtype) / 2, (float(err.max()), float(err.median()))
    cut = len(toks) // 2
    err = C.row_errors(C.run(TextEngine(llm), 0, toks, [cut] + [1] * (len(toks) - cut)), want)
    assert float(err.max()) < lim(dtype) and float(err.median()) < lim(dtype) / 2, (float(err.max()), float(err.median()))


@pytest.mark.parametrize("name", ["odd", "large"])
def test_stream_behind_every_layer(name, tmp_path):
    cfg, tensors, llm = C.build(name, torch.float32, DEV, tmp_path, seed=3)
    toks, want = C.prompt(cfg, 50, 9), []
    O.model(cfg, tensors, toks, trace=want)
    out = llm(input_ids=torch.tensor([toks], device=DEV), output_hidden_states=True)
    assert len(out.hidden_states) == len(want) + 1 and out.logits.shape == (1, 1, cfg["vocab"])
    for got, w in zip(out.hidden_states[1:], want):
        close(got, w, 2e-5)


@pytest.mark.parametrize("name,dtype", [("odd", torch.float32), ("tiles", torch.float32), ("large", torch.float32), ("tiles", BF), ("large", BF),
                                        ("mixed", BF)])
@pytest.mark.parametrize("cuts", [[2] * 30, [1] * 70, [64, 1, 1, 3], [7, 2, 2, 1, 33, 5], [127, 2]])
def test_portions_of_a_prompt(name, dtype, cuts, tmp_path):
    from timeviper_amd.model.llm import TextEngine
    cfg, _, llm = C.build(name, dtype, DEV, tmp_path, seed=5)
    toks = C.prompt(cfg, 140, 17)
    whole = C.run(TextEngine(llm), 0, toks, [])
    assert float(C.row_errors(C.run(TextEngine(llm), 0, toks, cuts), whole).max()) < lim(dtype)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["odd", "tiles", "large"])
def test_unequal_requests_together_and_slots_used_again(name, dtype, tmp_path):
    """Batches of unequal prompts decoded together, requests that end early and others that take their slots, against each
    request alone."""
    from timeviper_amd.model.llm import TextEngine
    cfg, _, llm = C.build(name, dtype, DEV, tmp_path, seed=6)
    lens = {"a": 1, "b": 37, "c": 130, "d": 64, "e": 3, "f": 65}
    toks = {r: C.prompt(cfg, n + 12, 200 + n) for r, n in lens.items()}
    alone = {r: C.run(TextEngine(llm), r, toks[r], []) for r in lens}
    eng, got, at = TextEngine(llm), {r: [] for r in lens}, {r: 0 for r in lens}

    def step(parts):
        lg = eng.step([(r, toks[r][at[r]:at[r] + n], range(n)) for r, n in parts]).cpu()
        for r, n in parts:
            got[r].append(lg[:n])
            lg, at[r] = lg[n:], at[r] + n

    step([(r, lens[r]) for r in "abc"])
    for _ in range(4):
        step([(r, 1) for r in "abc"])
    eng.end("b")                                              # b leaves, d and e take its slot and a new one
    step([("d", lens["d"]), ("e", lens["e"])])
    for _ in range(5):
        step([(r, 1) for r in "ecda"])                        # another order
    eng.end("a"), eng.end("c")
    step([("f", lens["f"]), ("d", 1), ("e", 2)])              # a prompt, a single token and a portion in one step
    for _ in range(3):
        step([("f", 1), ("d", 1)])
    for r in lens:
        lg = torch.cat(got[r])
        err = C.row_errors(lg, alone[r][:len(lg)])
        assert float(err.max()) < lim(dtype), (r, err.topk(min(3, len(err))))


@pytest.mark.parametrize("name,dtype", [("odd", torch.float32), ("tiles", torch.float32), ("tiles", BF)])
def test_long_decoding(name, dtype, tmp_path):
    """Hundreds of single tokens, to the last position: the cache grows, windows pass over decoded keys; against the whole sequence
    in one step."""
    from timeviper_amd.model.llm import TextEngine
    cfg, _, llm = C.build(name, dtype, DEV, tmp_path, seed=7)
    toks = C.prompt(cfg, cfg["max_positions"], 31)
    whole = C.run(TextEngine(llm), 0, toks, [])
    eng = TextEngine(llm)
    assert float(C.row_errors(C.run(eng, 0, toks, [3] + [1] * (len(toks) - 3)), whole).max()) < lim(dtype)
    with pytest.raises(ValueError):
        eng.step([(0, [1], [0])])


@pytest.mark.parametrize("B", [2, 4, 5, 17])
def test_batched_decoding_fused_and_general(B, tmp_path, monkeypatch):
    """Batches on the fused kernels (up to four sequences) and beyond them, against each sequence in one step."""
    from timeviper_amd.model.llm import TextEngine
    cfg, _, llm = C.build("large", BF, DEV, tmp_path, seed=12)
    toks = [C.prompt(cfg, 5 + 7 * i % 40 + 6, 400 + i) for i in range(B)]
    alone = [C.run(TextEngine(llm), 0, t, [])[-4:] for t in toks]
    for fused in ("1", "0"):
        monkeypatch.setenv("TV_DECODE_FUSED", fused)
        eng = TextEngine(llm, slots=2)
        rows = [eng.step([(i, t[:-3], [len(t) - 4]) for i, t in enumerate(toks)]).cpu()]
        for k in (3, 2, 1):
            rows.append(eng.step([(i, [t[-k]], [0]) for i, t in enumerate(toks)]).cpu())
        err = torch.stack([C.row_errors(torch.stack([r[i] for r in rows]), alone[i]) for i in range(B)])
        assert float(err.max()) < lim(BF), (fused, err.flatten().topk(5))


@pytest.mark.parametrize("graph", ["1", "0"])
@pytest.mark.parametrize("name,dtype", [("odd", torch.float32), ("tiles", torch.float32), ("tiles", BF), ("large", BF)])
def test_greedy_generation_through_the_scheduler(name, dtype, graph, tmp_path, monkeypatch):
    """More prompts than the batch takes, an end token for some of them; every chosen token is (nearly) the best of the
    equations' logits.  Replayed steps (hipGraph) and eager ones."""
    from timeviper_amd.model.llm import GenericLLMBackbone
    monkeypatch.setenv("TV_DECODE_GRAPH", graph)
    cfg = C.CONFIGS[name]
    tensors = O.random_tensors(cfg, 8)
    bb = GenericLLMBackbone.from_folder(C.write_folder(tmp_path / name, cfg, tensors), dtype, DEV)
    prompts = [C.prompt(cfg, n, 300 + n) for n in (1, 9, 40, 5, 17)]
    first = bb.generate(prompts, max_new_tokens=12, eos_token_id=[], max_batch=3)
    eos = first[1][6]
    new = bb.generate(prompts, max_new_tokens=12, eos_token_id=[eos], max_batch=3)
    slack = 1e-3 if dtype == torch.float32 else 0.15
    for p, f, ids in zip(prompts, first, new):
        assert len(f) == 12
        if dtype == torch.float32:
            assert ids == (f[:f.index(eos) + 1] if eos in f else f)
        lg = O.model(cfg, tensors, p + ids)[len(p) - 1:-1]
        behind = lg.max(-1).values - lg.gather(1, torch.tensor(ids)[:, None])[:, 0]
        assert float(behind.max()) < slack * float(lg.std()) * 4, behind


def test_replayed_decode_steps_equal_eager_ones(tmp_path):
    """The captured step replayed with eager work between the replays: every replay's logits against the eager step's."""
    from timeviper_amd.model.llm.decode_graph import GraphedDecodeStep
    cfg, _, llm = C.build("large", BF, DEV, tmp_path, seed=13)
    ids = torch.tensor([C.prompt(cfg, 40, 1), C.prompt(cfg, 40, 2)], device=DEV)
    nxt = torch.tensor(C.prompt(cfg, 2 * 12, 3), device=DEV).view(12, 2, 1)
    with torch.inference_mode():
        a, b = llm.new_cache(2), llm.new_cache(2)
        llm(input_ids=ids, past_key_values=a), llm(input_ids=ids, past_key_values=b)
        a.begin_static_decode(12)
        step = GraphedDecodeStep(lambda i: llm(input_ids=i, past_key_values=a).logits, a, 2, DEV)
        for t in range(12):
            step.step(nxt[t])
            got = step.logits.clone()
            want = llm(input_ids=nxt[t], past_key_values=b).logits[:, -1]
            torch.cuda.synchronize()
            assert float(C.row_errors(got, want.cpu()).max()) < 2e-2, t
        assert step.graph is not None and a.get_seq_length() == b.get_seq_length() == 52


def test_batch_call_with_padding(tmp_path):
    """The (batch, tokens) call: padding on either side is left out."""
    cfg, tensors, llm = C.build("tiles", torch.float32, DEV, tmp_path, seed=10)
    a, b = C.prompt(cfg, 20, 1), C.prompt(cfg, 13, 2)
    ids = torch.zeros((2, 20), dtype=torch.long)
    mask = torch.ones((2, 20), dtype=torch.long)
    ids[0], ids[1, 7:] = torch.tensor(a), torch.tensor(b)
    mask[1, :7] = 0
    with torch.no_grad():
        out = llm(input_ids=ids.to(DEV), attention_mask=mask.to(DEV), logits_to_keep=0)
    assert float(C.row_errors(out.logits[0], O.model(cfg, tensors, a)).max()) < 1e-4
    assert float(C.row_errors(out.logits[1, 7:], O.model(cfg, tensors, b)).max()) < 1e-4
    nxt = torch.tensor([[3], [4]], device=DEV)
    with torch.no_grad():
        step = llm(input_ids=nxt, past_key_values=out.past_key_values)
    assert float(C.row_errors(step.logits[1], O.model(cfg, tensors, b + [4])[-1:]).max()) < 1e-4


def test_trace_runner_and_generate_commands(tmp_path):
    """bin/trace_run and the generate command as a user calls them."""
    import json
    import subprocess
    import sys
    from pathlib import Path

    import numpy as np
    root = Path(__file__).resolve().parent.parent
    cfg = C.CONFIGS["tiles"]
    tensors = O.random_tensors(cfg, 11)
    folder = C.write_folder(tmp_path / "m", cfg, tensors)
    p = C.prompt(cfg, 12, 5)
    steps = [{"step": 0, "entries": [{"id": "x", "tokens": p[:10], "want": [9, 0]}, {"id": "y", "tokens": p[:4], "want": []}], "end": ["y"]},
             {"step": 1, "entries": [{"id": "x", "tokens": [p[10]], "want": []}], "end": []},
             {"step": 2, "entries": [{"id": "x", "tokens": [p[11]], "want": [0]}], "end": ["x"]}]
    r = subprocess.run([str(root / "bin" / "trace_run"), "--model", str(folder), "--dtype", "float32", "--out", str(tmp_path), "--max-tokens", "64"],
                       input="\n".join(json.dumps(s) for s in steps) + "\n", capture_output=True, text=True, timeout=110)
    assert r.returncode == 0, r.stderr[-2000:]
    assert [ln for ln in r.stdout.splitlines() if ln.startswith("done")] == ["done 0", "done 1", "done 2"]
    want = O.model(cfg, tensors, p)
    got = np.fromfile(tmp_path / "0.f32", dtype="<f4").reshape(2, -1)
    assert float(C.row_errors(torch.from_numpy(got), want[[9, 0]]).max()) < 1e-4
    assert not (tmp_path / "1.f32").exists()
    got = np.fromfile(tmp_path / "2.f32", dtype="<f4").reshape(1, -1)
    assert float(C.row_errors(torch.from_numpy(got), want[[11]]).max()) < 1e-4
    r = subprocess.run([sys.executable, "-m", "timeviper_amd.generate", "--model", str(folder), "--dtype", "float32", "--max-new-tokens", "1",
                        "--prompt", " ".join(map(str, p))], cwd=root, capture_output=True, text=True, timeout=110)
    assert r.returncode == 0 and int(r.stdout.split()[-1]) == int(want[-1].argmax()), r.stderr[-2000:]
