"""GPU: the operators behind Sozarax, each alone, against the plain float64 restatement in oracle/sozarax.py."""
import pytest
import torch

from op_harness import bounds, i32, limit, op, padded_rows, paged_case, rel
from oracle import sozarax as O

pytestmark = pytest.mark.gpu
DTYPES = [torch.float32, torch.bfloat16]
D = torch.float64


# ---------------------------------------------------------------------------------------------------- residual, norms, activations
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rows,n,parts", [(5, 72, 1), (3, 1024, 3), (2, 101, 2), (4, 2048, 1), (1, 10000, 2), (130, 640, 4)])
def test_add_norm_norm(gpu, dtype, rows, n, parts):
    g = torch.Generator().manual_seed(n + parts)
    x, y = torch.randn((rows, n), generator=g), torch.randn((rows * parts, n), generator=g).to(dtype)
    wo, wi = (torch.randn(n, generator=g).to(dtype) for _ in range(2))
    res = x.clone().to(gpu)
    out = op("add_norm_norm")(res, y.to(gpu), wo.to(gpu), wi.to(gpu), 1e-4)
    want = x.to(D) + O.norm(y.to(D).view(rows, parts, n).sum(1), wo.to(D), 1e-4)
    assert rel(res, want) < 1e-6
    assert rel(out, O.norm(want, wi.to(D), 1e-4)) < limit(dtype)


@pytest.mark.parametrize("dtype", DTYPES)
def test_scaled_embedding_and_squared_relu(gpu, dtype):
    g = torch.Generator().manual_seed(3)
    for width in (64, 70):
        t = torch.randn((33, width), generator=g).to(dtype)
        ids = torch.tensor([4, 0, 32, 4, 99])
        res, act = op("embed_residual")(ids.to(gpu), t.to(gpu), 2.7)
        want = torch.cat((t[ids[:4]].to(D) * 2.7, torch.zeros((1, width), dtype=D)))
        assert rel(res, want) < 1e-6 and rel(act, want) < limit(dtype)
        res2, none = op("embed_residual")(ids.to(gpu), t.to(gpu), 2.7, need_act=False)
        assert none is None and torch.equal(res, res2)
    for n in (64, 37):
        x = torch.randn((9, n + 16), generator=g).to(dtype)
        assert rel(op("squared_relu")(x.to(gpu)[:, :n]), O.squared_relu(x[:, :n].to(D))) < limit(dtype)


# ---------------------------------------------------------------------------------------------------- time mixing
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("width", [64, 75])
def test_token_mix(gpu, dtype, width):
    """Portions and single tokens; the row in front comes from the slot unless the sequence starts, whatever the slot holds."""
    g = torch.Generator().manual_seed(width)
    counts, starts, slots = [1, 1, 1, 2, 7, 5], [0, 3, 9, 6, 0, 4], [2, 5, -1, 0, 6, 3]
    T = sum(counts)
    x, mu, before = torch.randn((T, width), generator=g).to(dtype), torch.rand((5, width), generator=g), torch.randn((7, width), generator=g).to(dtype)
    before[2], before[6] = float("nan"), float("inf")      # of sequences that start
    cu = bounds(counts)
    seq = [i for i, n in enumerate(counts) for _ in range(n)]

    def wanted(i):
        prev = None if starts[i] == 0 or slots[i] < 0 else before[slots[i]].to(D)
        return torch.stack([O.token_mix(x[cu[i]:cu[i + 1]].to(D), mu[p].to(D), prev) for p in range(5)])

    b = before.clone().to(gpu)
    out = op("token_mix")(x.to(gpu), mu.to(gpu), b, i32(starts, gpu), i32(slots, gpu), i32(seq, gpu), i32(cu, gpu))
    assert rel(out, torch.cat([wanted(i) for i in range(6)], dim=1)) < limit(dtype)
    after = before.clone()
    for i, s in enumerate(slots):
        if s >= 0:
            after[s] = x[cu[i + 1] - 1]
    assert torch.equal(b.cpu()[[0, 2, 3, 5, 6]], after[[0, 2, 3, 5, 6]]) and torch.equal(b.cpu()[[1, 4]], before[[1, 4]])
    b = before.clone().to(gpu)      # a decode step: no cu_seqlens
    out = op("token_mix")(x[:3].to(gpu), mu.to(gpu), b, i32(starts[:3], gpu), i32(slots[:3], gpu))
    assert rel(out, torch.cat([wanted(i) for i in range(3)], dim=1)) < limit(dtype)
    assert torch.equal(b.cpu()[[2, 5]], x[:2])


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("tokens,channels,rank", [(1, 64, 16), (70, 300, 5), (129, 256, 64), (3, 33, 1), (65, 520, 100), (2, 64, 300)])
def test_low_rank_decay(gpu, dtype, tokens, channels, rank):
    g = torch.Generator().manual_seed(rank)
    z, w2 = torch.randn((tokens, rank + 3), generator=g).to(dtype), (torch.randn((channels, rank), generator=g) * rank ** -0.5).to(dtype)
    w0 = torch.randn(channels, generator=g) * 2 - 2
    got = op("low_rank_decay")(z.to(gpu)[:, :rank], w2.to(gpu), w0.to(gpu))
    assert got.dtype == torch.float32
    want = torch.log(O.channel_decay(z[:, :rank].to(D), torch.eye(rank, dtype=D), w2.to(D), w0.to(D)))
    assert rel(got, want) < limit(dtype, 3e-6, 4e-3)


def run_recurrence(gpu, which, dtype, H, d, vd, counts, starts, log_decay, seed=0, wanted=768, far=False, slots=None):
    """Largest relative errors of outputs and states over the sequences."""
    from nano_vllm_ninetoothed_amd.mops.hip import recurrent_ops as R
    g = torch.Generator().manual_seed(seed)
    T, B, cu = sum(counts), len(counts), bounds(counts)
    r, k, v = (torch.randn((T, H * n), generator=g).to(dtype) for n in (d, d, vd))
    lw = log_decay(g, (T, H * d))
    if far:      # the first token of the longest sequence stands out of everything behind it, if it is kept
        t = cu[max(range(B), key=lambda i: counts[i])]
        k[t] *= 64
    u = torch.randn(H * d, generator=g)
    S0 = torch.randn((B, H, d, vd), generator=g)
    slots = list(range(B, 0, -1)) if slots is None else slots
    state = torch.full((B + 2, H, vd, R.recurrence_state_pitch(d)), float("nan"))
    for b in range(B):
        if starts[b] and slots[b] >= 0:
            state[slots[b], :, :, :d] = S0[b].transpose(1, 2)
            state[slots[b], :, :, d:] = 0
    state, out = state.to(gpu), torch.full((T, H * vd), float("nan"), dtype=dtype, device=gpu)
    args = [r.to(gpu), k.to(gpu), v.to(gpu), out, state, i32(slots, gpu), i32(starts, gpu), H, H, d, vd]
    options = dict(channel_decay=lw.to(gpu), bonus=u.to(gpu), cu_seqlens=i32(cu, gpu))
    if which == "chunks":
        segs, ends = R.channel_segments(counts, H, vd, wanted)
        op("channel_chunks")(*args, i32(segs, gpu), i32(ends, gpu), **options)
    else:
        if max(counts) == 1:
            del options["cu_seqlens"]
        op("decayed_recurrence")(*args, **options)
    worst = [0.0, 0.0]
    for b in range(B):
        if slots[b] < 0:
            continue
        f = lambda x: x[cu[b]:cu[b + 1]].to(D).view(counts[b], H, -1)      # noqa: E731
        o, S = O.channel_recurrence(f(r), f(k), f(v), torch.exp(f(lw)), u.to(D).view(H, d), S0[b].to(D) if starts[b] else None)
        worst[0] = max(worst[0], rel(out[cu[b]:cu[b + 1]].view(counts[b], H, vd), o))
        worst[1] = max(worst[1], rel(state[slots[b], :, :, :d].transpose(1, 2), S))
    return worst


def usual(g, shape):
    return -torch.exp(torch.randn(shape, generator=g) * 1.5 - 3)


def strong(g, shape):      # decays down to e^-400 beside some near one
    return -torch.exp(torch.randn(shape, generator=g) * 3 + 1)


def weak(g, shape):
    return -torch.exp(torch.randn(shape, generator=g) * 0.5 - 9)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,d,vd", [(3, 64, 64), (2, 20, 20), (1, 128, 128), (2, 33, 70), (1, 300, 24), (2, 16, 8)])
def test_channel_recurrence_token_by_token(gpu, dtype, H, d, vd):
    for decay in (usual, strong, weak):
        o, S = run_recurrence(gpu, "plain", dtype, H, d, vd, [1] * 7, [0, 4, 1, 9, 0, 7, 2], decay, slots=[3, 1, -1, 0, 2, 8, 5])
        assert o < limit(dtype, 2e-6) and S < 1e-6
        o, S = run_recurrence(gpu, "plain", dtype, H, d, vd, [40, 2, 19], [0, 4, 1], decay, far=True)
        assert o < limit(dtype, 2e-6) and S < 2e-6


@pytest.mark.parametrize("H,d,vd", [(3, 64, 64), (2, 20, 20), (1, 128, 128), (2, 33, 70), (1, 256, 200), (2, 16, 8), (1, 48, 130)])
def test_channel_recurrence_in_chunks(gpu, H, d, vd):
    """Portions shorter and longer than chunks, and one that is cut into segments; far tokens that are kept; all strengths of decay."""
    for seed, decay in enumerate((usual, strong, weak)):
        for counts, starts in (([2, 37, 16, 1, 100], [0, 5, 3, 2, 0]), ([17], [4]), ([400, 33], [0, 7])):
            o, S = run_recurrence(gpu, "chunks", torch.bfloat16, H, d, vd, counts, starts, decay, seed=seed, far=True)
            assert o < 3e-3 and S < 2e-5, (decay.__name__, counts, o, S)


def test_channel_chunks_leave_padding_slots_alone(gpu):
    o, S = run_recurrence(gpu, "chunks", torch.bfloat16, 2, 64, 64, [20, 20, 20], [0, 3, 1], usual, slots=[2, -1, 0])
    assert o < 3e-3 and S < 2e-5


# ---------------------------------------------------------------------------------------------------- attention
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,G,d,v", [(4, 2, 64, 64), (6, 3, 20, 13), (1, 1, 8, 24), (16, 8, 128, 128)])
def test_attention_prepare(gpu, dtype, H, G, d, v):
    from nano_vllm_ninetoothed_amd.layers import Rotary
    from nano_vllm_ninetoothed_amd.mops.hip.attention_ops import padded
    g = torch.Generator().manual_seed(d)
    n = (H + G) * d + G * v
    x = torch.randn((9, (n + 7) // 8 * 8), generator=g).to(dtype)
    wq, wk = torch.randn(H * d, generator=g).to(dtype), torch.randn(G * d, generator=g).to(dtype)
    pos, slots = [0, 5, 6, 7, 12, 13, 14, 40, 200], [3, -1, 8, 9, 31, 0, 16, 15, 20]
    kp, vp = (torch.full((2, 16, G, padded(s)), float("nan"), dtype=dtype, device=gpu) for s in (d, v))
    factor = Rotary(256, gpu).steps(0.3, 7)
    q = op("attention_prepare")(x.to(gpu), wq.to(gpu), wk.to(gpu), 1e-5, i32(pos, gpu), i32(slots, gpu), kp, vp, H, G, d, v, q_factor=factor)
    t = O.query_temperature(torch.tensor(pos), 0.3, 7)
    assert t[0] == 1 and t[1] == 1 and t[2] > 1 and t[3] == t[2] and t[5] > t[4]      # the step lies between positions 5 and 6, 12 and 13
    want = (O.norm(x[:, :H * d].to(D), wq.to(D), 1e-5) * t[:, None]).view(9, H, d)
    assert rel(q[..., :d], want) < limit(dtype) and (q[..., d:] == 0).all()
    keys, values = O.norm(x[:, H * d:(H + G) * d].to(D), wk.to(D), 1e-5).view(9, G, d), x[:, (H + G) * d:n].view(9, G, v)
    ok = [i for i, s in enumerate(slots) if s >= 0]
    at = [slots[i] for i in ok]
    kf, vf = kp.view(32, G, -1)[at].cpu(), vp.view(32, G, -1)[at].cpu()
    assert rel(kf[..., :d], keys[ok]) < limit(dtype) and (kf[..., d:] == 0).all()
    assert torch.equal(vf[..., :v], values[ok]) and (vf[..., v:] == 0).all()
    rest = [s for s in range(32) if s not in at]
    assert kp.view(32, -1)[rest].isnan().all() and vp.view(32, -1)[rest].isnan().all()


SIZES = [(8, 2, 64, 64), (6, 3, 20, 13), (1, 1, 8, 40), (20, 1, 128, 128), (4, 4, 200, 24), (3, 1, 24, 256), (16, 8, 128, 128)]


@pytest.mark.parametrize("H,G,d,v", SIZES)
@pytest.mark.parametrize("kind", ["rows float32", "rows bfloat16", "decode"])
def test_single_rows(gpu, kind, H, G, d, v):
    """Rows of several sequences at once, also several of one sequence; contexts of one token, around stages and pages, empty ones."""
    dtype = torch.float32 if kind == "rows float32" else torch.bfloat16
    name = "biased_decode" if kind == "decode" else "biased_attention_rows"
    slopes = O.distance_slopes(H)
    for bs, lens, far in ((32, [1, 31, 32, 33, 64, 300], (0,)), (64, [65, 2, 700], (3, 63, 64, 640)), (32, [500], (31, 32, 95, 96))):
        seqs, kp, vp, table = paged_case(gpu, dtype, H, G, d, v, lens, bs, H + bs, far)
        rows = [(i, c) for i, n in enumerate(lens) for c in sorted({1, 2, n // 2 + 1, max(1, n - 1), n} & set(range(1, n + 1)))]
        rows.insert(2, (0, 0))
        q = torch.stack([seqs[i][0][max(c - 1, 0)] for i, c in rows])
        args = (kp, vp, d, v, i32([c for _, c in rows], gpu), table, 0.3 * d ** -0.5)
        got = op(name)(padded_rows(q, d).to(gpu), *args, slopes=slopes.float().to(gpu), row_seq=i32([i for i, _ in rows], gpu)).cpu()
        assert got.shape == (len(rows), H, v) and (got[2] == 0).all()
        for j, (i, c) in enumerate(rows):
            if c:
                qq, k, val = (t[:c].to(D) for t in seqs[i])
                want = O.biased_attention(qq, k, val, 0.3 * d ** -0.5, slopes)[-1]
                assert rel(got[j], want) < limit(dtype, 2e-6, 4e-3), (bs, i, c)
    plain = op(name)(padded_rows(q, d).to(gpu), *args, row_seq=i32([i for i, _ in rows], gpu)).cpu()      # without a bias
    i, c = rows[-1]
    assert rel(plain[-1], O.biased_attention(*(t[:c].to(D) for t in seqs[i]), 0.3 * d ** -0.5, torch.zeros(H))[-1]) < limit(dtype, 2e-6, 4e-3)


def test_decode_with_many_rows(gpu):
    """More rows than the run search has lanes, of very different lengths, one row per sequence."""
    H, G, d, v = 4, 2, 64, 32
    g = torch.Generator().manual_seed(1)
    lens = [int(x) for x in torch.randint(1, 130, (150,), generator=g)]
    lens[70] = 1500
    seqs, kp, vp, table = paged_case(gpu, torch.bfloat16, H, G, d, v, lens, 32, 5)
    got = op("biased_decode")(torch.stack([s[0][-1] for s in seqs]).to(gpu), kp, vp, d, v, i32(lens, gpu), table, 0.1, slopes=O.distance_slopes(H).float().to(gpu))
    for i in (0, 1, 63, 64, 69, 70, 71, 149):
        want = O.biased_attention(*(t.to(D) for t in seqs[i]), 0.1, O.distance_slopes(H))[-1]
        assert rel(got[i], want) < 4e-3, i


@pytest.mark.parametrize("H,G,d,v", SIZES)
def test_long_portions(gpu, H, G, d, v):
    """Portions behind cached tokens and from the start, packed behind rows that the launch must leave alone."""
    from nano_vllm_ninetoothed_amd.mops.hip.attention_ops import biased_prefill_tiles
    slopes = O.distance_slopes(H)
    for bs, lens, counts in ((32, [130, 64, 300], [130, 33, 70]), (64, [513, 1], [200, 1]), (48, [97], [96])):
        seqs, kp, vp, table = paged_case(gpu, torch.bfloat16, H, G, d, v, lens, bs, d + bs, far=(0, 63, 64, 127, 128))
        starts = [n - c for n, c in zip(lens, counts)]
        skip = 3
        q = torch.cat([torch.randn((skip, H, d)).bfloat16()] + [s[0][a:] for s, a in zip(seqs, starts)])
        out = torch.full((q.shape[0], H, v), 7.0, dtype=torch.bfloat16, device=gpu)
        context = torch.zeros(q.shape[0], dtype=torch.int32, device=gpu)
        op("biased_prefill")(padded_rows(q, d).to(gpu), kp, vp, d, v, i32(biased_prefill_tiles(counts, starts, skip, 0), gpu), table, 0.3 * d ** -0.5, context,
                             slopes=slopes.float().to(gpu), out=out)
        assert (out[:skip] == 7).all()
        at = skip
        for s, a, n in zip(seqs, starts, counts):
            want = O.biased_attention(*(t.to(D) for t in s), 0.3 * d ** -0.5, slopes)[a:]
            err = (out[at:at + n].double().cpu() - want).flatten(1).norm(dim=1) / want.flatten(1).norm(dim=1)
            assert err.max() < 5e-3, (bs, a, n, err.argmax())
            at += n


# ---------------------------------------------------------------------------------------------------- mixture of experts
@pytest.mark.parametrize("dtype,block", [(torch.float32, 32), (torch.bfloat16, 32), (torch.bfloat16, 128)])
@pytest.mark.parametrize("tokens,width,ff,experts,top", [(1, 64, 32, 4, 1), (70, 72, 24, 5, 2), (300, 256, 136, 16, 4), (40, 50, 17, 3, 3), (33, 128, 40, 130, 2),
                                                         (129, 96, 64, 1, 1), (257, 64, 200, 33, 1), (2500, 64, 32, 20, 3), (2111, 48, 16, 7, 2)])
def test_mixture(gpu, dtype, block, tokens, width, ff, experts, top):
    g = torch.Generator().manual_seed(experts)
    h, router = torch.randn((tokens, width), generator=g).to(dtype), (torch.randn((experts, width), generator=g) * 4 * width ** -0.5).to(dtype)
    if experts > 2:
        router[1] = 0      # most tokens have a preference; none has this one, and some expert stays empty
    routing = op("moe_route")(h.to(gpu), router.to(gpu), top, block)
    chosen, score = O.route(h.to(D), router.to(D), top)
    got = routing.chosen.cpu().long()
    z = torch.sigmoid(h.to(D) @ router.to(D).T)
    assert rel(z.gather(1, got), score) < 1e-5 and rel(routing.score, z.gather(1, got)) < 1e-5      # a tie may go either way
    assert all(len(set(r)) == top for r in got.tolist())
    rows = routing.rows.cpu().long()
    assert sorted(rows.tolist()) == list(range(tokens * top)) and (got.flatten()[rows].diff() >= 0).all()
    n_tiles = int(routing.tiles[0])
    tiles = routing.tiles[1:1 + 3 * n_tiles].view(-1, 3).cpu()
    assert int(tiles[:, 2].sum()) == tokens * top and (tiles[:, 2] <= block).all() and (tiles[:, 2] > 0).all()
    assert all((got.flatten()[rows[r:r + n]] == e).all() for e, r, n in tiles.tolist())
    pad = -ff % 8
    gu, down = torch.zeros((experts, 2, ff + pad, width)).to(dtype), torch.zeros((experts, width, ff + pad)).to(dtype)
    gu[:, :, :ff] = torch.randn((experts, 2, ff, width), generator=g) * width ** -0.5 * 2
    down[:, :, :ff] = torch.randn((experts, width, ff), generator=g) * ff ** -0.5
    y = op("moe_gate_up")(h.to(gpu), gu.to(gpu), routing)
    s, e = z.gather(1, got).flatten()[rows], got.flatten()[rows]
    x = h.to(D)[rows // top] * s[:, None]
    hidden = O.silu(torch.einsum("ck,cnk->cn", x, gu[:, 0].to(D)[e])) * torch.einsum("ck,cnk->cn", x, gu[:, 1].to(D)[e])
    assert rel(y, hidden) < limit(dtype, 2e-6, 4e-3)
    out = op("moe_down")(y, down.to(gpu), routing)
    want = torch.empty((tokens * top, width), dtype=D)
    want[rows] = torch.einsum("ck,cnk->cn", y.double().cpu(), down.to(D)[e])
    assert rel(out, want) < limit(dtype, 2e-6)
    assert rel(out.view(tokens, top, width).double().sum(1), O.mixture(h.to(D), {"router": router.to(D), **{
        f"e{i}.{n}": t[:, :ff] if n == "down" else t[:ff] for i in range(experts) for n, t in (("gate", gu[i, 0].to(D)), ("up", gu[i, 1].to(D)), ("down", down[i].to(D)))}},
        {"router": {"experts": experts, "top": top}})) < limit(dtype, 3e-6, 8e-3)


def test_all_tokens_on_one_expert_and_replay(gpu):
    """The largest block of one expert; a captured route and product replayed on other inputs."""
    width, ff, experts, top, tokens = 64, 32, 8, 2, 200
    g = torch.Generator().manual_seed(0)
    router, h = torch.randn((experts, width), generator=g).bfloat16(), torch.randn((tokens, width), generator=g).abs().bfloat16()
    router[3] = 1.0
    r = op("moe_route")(h.to(gpu), router.to(gpu), top)
    assert (r.chosen[:, 0] == 3).all()
    w = torch.randn((experts, 2, ff, width), generator=g).bfloat16().to(gpu)
    x, rt = h.to(gpu), router.to(gpu)
    torch.cuda.synchronize()
    graph = torch.cuda.CUDAGraph()
    with torch.cuda.graph(graph):
        routing = op("moe_route")(x, rt, top)
        y = op("moe_gate_up")(x, w, routing)
    for seed in range(3):
        x.copy_(torch.randn((tokens, width), generator=torch.Generator().manual_seed(seed)).bfloat16())
        graph.replay()
        eager = op("moe_route")(x, rt, top)
        ye = op("moe_gate_up")(x, w, eager)
        torch.cuda.synchronize()
        assert torch.equal(routing.chosen, eager.chosen) and torch.equal(routing.score, eager.score)
        a, b = torch.empty_like(y), torch.empty_like(ye)
        a[routing.rows.long()], b[eager.rows.long()] = y, ye
        assert torch.equal(a, b)


@pytest.mark.parametrize("groups,tokens,n,k,last", [(4, 1, 64, 64, 16), (4, 70, 132, 72, 5), (3, 256, 256, 320, 256), (2, 33, 50, 44, None), (4, 16, 1024, 1024, 32)])
def test_grouped_linear(gpu, groups, tokens, n, k, last):
    g = torch.Generator().manual_seed(n)
    x, w = torch.randn((groups + (last is not None), tokens, k), generator=g).bfloat16(), torch.randn((groups, n, k), generator=g).bfloat16()
    wl = None if last is None else torch.randn((last, k), generator=g).bfloat16()
    got = op("grouped_linear")(x.to(gpu), w.to(gpu), None if wl is None else wl.to(gpu))
    y = got if last is None else got[0]
    assert rel(y, torch.stack([x[i].to(D) @ w[i].to(D).T for i in range(groups)])) < 3e-3
    if last is not None:
        assert rel(got[1], x[-1].to(D) @ wl.to(D).T) < 3e-3
