"""GPU: the operators behind Lulizen, each alone, against the plain float64 restatement in oracle/lulizen.py."""
import pytest
import torch

from op_harness import bounds, i32, limit, op, padded_rows, paged_case, rel
from oracle import lulizen as O

pytestmark = pytest.mark.gpu
DTYPES = [torch.float32, torch.bfloat16]
D = torch.float64


# ---------------------------------------------------------------------------------------------------- embedding, norms, activations
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("width,mul_prev,mul_cur,buckets", [(64, 29, 11, 53), (75, 1000003, -99991, 20), (640, 1, 1, 1)])
def test_embedding_of_pairs(gpu, dtype, width, mul_prev, mul_cur, buckets):
    """Portions and single tokens; the token in front comes from the slot unless the sequence starts, whatever the slot holds."""
    g = torch.Generator().manual_seed(width)
    vocab = 90
    table, pairs = torch.randn((vocab, width), generator=g).to(dtype), torch.randn((buckets + 1, width), generator=g).to(dtype)
    counts, starts, slots = [1, 1, 1, 2, 7, 5], [0, 3, 9, 6, 0, 4], [2, 5, 1, 0, 6, 3]
    ids = torch.randint(0, vocab, (sum(counts),), generator=g)
    before = torch.randint(0, vocab, (8,), generator=g).to(torch.int32)
    before[2] = -77                                                     # of a sequence that starts
    cu = bounds(counts)
    seq = [i for i, n in enumerate(counts) for _ in range(n)]
    bigram = {"buckets": buckets, "mul_prev": mul_prev, "mul_cur": mul_cur}

    def wanted(i):
        mine = ids[cu[i]:cu[i + 1]].tolist()
        front = [int(before[slots[i]])] if starts[i] else []
        return O.embedding(front + mine, table.to(D), pairs.to(D), bigram)[len(front):]

    b = before.clone().to(gpu)
    got = op("embed_pairs")(ids.to(gpu), table.to(gpu), pairs.to(gpu), mul_prev, mul_cur, b, i32(starts, gpu), i32(slots, gpu), i32(seq, gpu), i32(cu, gpu))
    assert got.dtype == torch.float32 and rel(got, torch.cat([wanted(i) for i in range(6)])) < 1e-6
    after = before.clone()
    for i, s in enumerate(slots):
        after[s] = ids[cu[i + 1] - 1]
    assert torch.equal(b.cpu(), after)
    b = before.clone().to(gpu)      # a decode step: no cu_seqlens; a padding row leaves every slot alone
    got = op("embed_pairs")(ids[:3].to(gpu), table.to(gpu), pairs.to(gpu), mul_prev, mul_cur, b, i32(starts[:3], gpu), i32([2, 5, -1], gpu), scale=0.5)
    want = torch.stack([wanted(0)[0], wanted(1)[0], table[ids[2]].to(D) + pairs[buckets].to(D)]) - 0.5 * table[ids[:3]].to(D)
    assert rel(got, want) < 1e-6
    after = before.clone()
    after[[2, 5]] = ids[:2].to(torch.int32)
    assert torch.equal(b.cpu(), after)


def test_rows_of_pairs_are_those_of_exact_arithmetic(gpu):
    """Large token ids and factors, negative ones too."""
    vocab, buckets = 150000, 4099
    table, pairs = torch.zeros((vocab, 8), dtype=torch.float32), torch.arange(buckets + 1, dtype=torch.float32)[:, None].repeat(1, 8)
    ids = torch.randint(0, vocab, (300,), generator=torch.Generator().manual_seed(1))
    for mul_prev, mul_cur in ((2 ** 31 - 1, 2 ** 31 - 1), (-2 ** 31 + 1, 5), (12345, -678)):
        got = op("embed_pairs")(ids.to(gpu), table.to(gpu), pairs.to(gpu), mul_prev, mul_cur, torch.zeros(1, dtype=torch.int32, device=gpu), i32([0], gpu), i32([0], gpu),
                                i32([0] * 300, gpu), i32([0, 300], gpu))
        assert got[:, 3].long().tolist() == O.bigram_rows(ids.tolist(), buckets, mul_prev, mul_cur)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rows,n,parts,more", [(5, 72, 1, False), (3, 1024, 3, True), (2, 101, 2, True), (4, 2048, 1, True), (1, 10000, 2, False), (130, 640, 4, True), (2, 700, 1, False),
                                               (3, 8, 1, False), (2, 2504, 1, True)])
def test_layer_norms(gpu, dtype, rows, n, parts, more):
    """Rows whose mean is far larger than their spread."""
    g = torch.Generator().manual_seed(n + parts)
    x, y = torch.randn((rows, n), generator=g) + 30, (torch.randn((rows * parts, n), generator=g) - 3).to(dtype)
    extra = (torch.randn((rows, n), generator=g) + 5).to(dtype) if more else None
    wo, wi = (torch.randn(n, generator=g).to(dtype) for _ in range(2))
    assert rel(op("layer_norm_f32")(x.to(gpu), wi.to(gpu), 1e-4), O.layer_norm(x.to(D), wi.to(D), 1e-4)) < limit(dtype, 3e-6)
    res = x.clone().to(gpu)
    out = op("add_norm_norm")(res, y.to(gpu), wo.to(gpu), wi.to(gpu), 1e-4, center=True, extra=None if extra is None else extra.to(gpu))
    total = y.to(D).view(rows, parts, n).sum(1) + (0 if extra is None else extra.to(D))
    want = x.to(D) + O.layer_norm(total, wo.to(D), 1e-4)
    assert rel(res, want) < 1e-6
    assert rel(out, O.layer_norm(want, wi.to(D), 1e-4)) < limit(dtype, 3e-6)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("n", [64, 37])
def test_gelu_unit(gpu, dtype, n):
    g = torch.Generator().manual_seed(n)
    p = 4 * torch.randn((9, 2 * n + 6), generator=g)
    p[0, :4], p[1, :2] = torch.tensor([-60.0, 60.0, 0.0, -1e-3]), torch.tensor([-1e4, 1e4])
    p = p.to(dtype)
    gate, up = p[:, :n], p[:, n:2 * n]
    got = op("gelu_glu")(p.to(gpu)[:, :n], p.to(gpu)[:, n:2 * n])
    want = O.gelu_tanh(gate.to(D)) * up.to(D)
    assert rel(got[2:], want[2:]) < limit(dtype) and (got.double().cpu() - want).abs().max() <= limit(dtype, 2e-6, 8e-3) * want.abs().max()
    small = (gate.abs() < 20) & (gate != 0)
    assert ((got.double().cpu() - want).abs() <= limit(dtype, 1e-5, 8e-3) * (want.abs() + 1e-6))[small].all()


# ---------------------------------------------------------------------------------------------------- attention
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,G,d,v,rot,norms", [(4, 2, 64, 64, 64, True), (6, 3, 22, 13, 14, False), (1, 1, 8, 24, 2, True), (16, 8, 128, 128, 64, True), (3, 1, 48, 40, 48, True),
                                               (2, 1, 256, 128, 32, False), (2, 2, 96, 96, 0, True), (2, 1, 320, 8, 160, True), (5, 1, 24, 264, 16, True), (2, 2, 80, 72, 24, True)])
def test_rotary_prepare(gpu, dtype, H, G, d, v, rot, norms):
    from nano_vllm_ninetoothed_amd.layers import Rotary
    from nano_vllm_ninetoothed_amd.mops.hip.attention_ops import padded
    g = torch.Generator().manual_seed(d)
    n = (H + G) * d + G * v
    x = torch.randn((9, (n + 5 + 7) // 8 * 8), generator=g).to(dtype)      # something behind the values
    wq, wk = ((torch.randn(d, generator=g).to(dtype) for _ in range(2)) if norms else (None, None))
    pos, slots = [0, 5, 6, 7, 12, 13, 14, 40, 200], [3, -1, 8, 9, 31, 0, 16, 15, 20]
    kp, vp = (torch.full((2, 16, G, padded(s)), float("nan"), dtype=dtype, device=gpu) for s in (d, v))
    on = lambda t: None if t is None else t.to(gpu)      # noqa: E731
    q = op("rotary_prepare")(x.to(gpu), i32(pos, gpu), i32(slots, gpu), kp, vp, H, G, d, v, cos_sin=Rotary(256, gpu).table(3e3, rot) if rot else None,
                             q_weight=on(wq), k_weight=on(wk), eps=1e-5)

    def turned(part, heads, w):
        y = part.to(D).view(9, heads, d)
        return O.rotate(y if w is None else O.rms_norm(y, w.to(D), 1e-5), torch.tensor(pos), 3e3, rot) if rot else (y if w is None else O.rms_norm(y, w.to(D), 1e-5))
    assert rel(q[..., :d], turned(x[:, :H * d], H, wq)) < limit(dtype) and (q[..., d:] == 0).all()
    keys, values = turned(x[:, H * d:(H + G) * d], G, wk), x[:, (H + G) * d:n].view(9, G, v)
    ok = [i for i, s in enumerate(slots) if s >= 0]
    at = [slots[i] for i in ok]
    kf, vf = kp.view(32, G, -1)[at].cpu(), vp.view(32, G, -1)[at].cpu()
    assert rel(kf[..., :d], keys[ok]) < limit(dtype) and (kf[..., d:] == 0).all()
    assert torch.equal(vf[..., :v], values[ok]) and (vf[..., v:] == 0).all()
    rest = [s for s in range(32) if s not in at]
    assert kp.view(32, -1)[rest].isnan().all() and vp.view(32, -1)[rest].isnan().all()


def scores(gpu, softcap, chunk=0, window=0, keep=0, sinks=None):
    from nano_vllm_ninetoothed_amd.mops.hip.attention_ops import Scores
    return Scores(softcap=softcap, window=window, chunk=chunk, keep_first=keep, sinks=None if sinks is None else sinks.float().to(gpu))


def oracle_mask(n, chunk=0, window=0, keep=0):
    return O.chunk_mask(n, chunk) if chunk else O.window_mask(n, window or n, keep)


MASKS = [dict(chunk=190), dict(chunk=64), dict(chunk=7), dict(chunk=1), dict(window=70, keep=18), dict(window=33, keep=40), dict(window=64), dict(window=1, keep=1), dict(window=5000, keep=3),
         dict(window=128, keep=64), dict(window=10, keep=170)]
SIZES = [(8, 2, 64, 64, 20.0, True, False), (6, 3, 20, 13, 5.0, False, True), (20, 1, 128, 128, 100.0, True, True), (3, 1, 24, 256, 3.0, False, False), (16, 8, 128, 128, 30.0, True, True)]


@pytest.mark.parametrize("H,G,d,v,cap,sink,gated", SIZES)
@pytest.mark.parametrize("kind", ["rows float32", "rows bfloat16", "decode"])
def test_single_rows(gpu, kind, H, G, d, v, cap, sink, gated):
    """Rows of several sequences at once, at edges of pages, stages, chunks and windows, with keys that stand out just inside and just
    outside of what the last row sees, and among the first tokens."""
    dtype = torch.float32 if kind == "rows float32" else torch.bfloat16
    name = "biased_decode" if kind == "decode" else "biased_attention_rows"
    g = torch.Generator().manual_seed(H)
    sinks, scale = torch.randn(H, generator=g) * 2 if sink else None, 1.5 * d ** -0.5
    for m, mask in enumerate(MASKS):
        bs, lens = ((32, [300, 1, 33, 201]), (64, [700, 65]), (32, [401]))[m % 3]
        see = oracle_mask(max(lens), **mask)
        last = see[lens[0] - 1].nonzero().flatten().tolist()
        edges = {last[0], last[-1], *[j for a, b in zip(last, last[1:]) if b != a + 1 for j in (a, a + 1, b - 1, b)], max(0, last[0] - 1)}
        seqs, kp, vp, table = paged_case(gpu, dtype, H, G, d, v, lens, bs, H + m, sorted(edges))
        rows = [(i, c) for i, n in enumerate(lens) for c in sorted({1, 2, n // 2 + 1, max(1, n - 1), n, 64, 65, 71, 89, 191} & set(range(1, n + 1)))]
        rows.insert(2, (0, 0))
        q = torch.stack([seqs[i][0][max(c - 1, 0)] for i, c in rows])
        gate = torch.randn((len(rows), H + 3), generator=g).to(dtype).to(gpu)[:, 1:1 + H] if gated else None
        got = op(name)(padded_rows(q, d).to(gpu), kp, vp, d, v, i32([c for _, c in rows], gpu), table, scale, row_seq=i32([i for i, _ in rows], gpu),
                       scores=scores(gpu, cap, sinks=sinks, **mask), gate=gate).cpu()
        assert got.shape == (len(rows), H, v) and (got[2] == 0).all()
        for j, (i, c) in enumerate(rows):
            if c:
                qq, k, val = (t[:c].to(D) for t in seqs[i])
                want = O.masked_attention(qq[-1:], k, val, scale, cap, oracle_mask(c, **mask)[-1:], None if sinks is None else sinks.float().to(D))[0]
                if gated:
                    want = want * O.sigmoid(gate[j].to(D).cpu())[:, None]
                assert rel(got[j], want) < limit(dtype, 2e-6, 5e-3), (mask, i, c)


@pytest.mark.parametrize("H,G,d,v,cap,sink,gated", SIZES)
def test_long_portions(gpu, H, G, d, v, cap, sink, gated):
    """Portions behind cached tokens and from the start, packed behind rows that the launch must leave alone."""
    from nano_vllm_ninetoothed_amd.mops.hip.attention_ops import biased_prefill_tiles
    g = torch.Generator().manual_seed(d)
    sinks, scale = torch.randn(H, generator=g) * 2 if sink else None, 1.5 * d ** -0.5
    for m, mask in enumerate(MASKS):
        bs, lens, counts = ((32, [130, 64, 300], [130, 33, 70]), (64, [513, 1], [300, 1]), (48, [397], [396]))[m % 3]
        seqs, kp, vp, table = paged_case(gpu, torch.bfloat16, H, G, d, v, lens, bs, d + m, far=(0, 17, 18, 63, 64, 127, 128, 189, 190))
        starts = [n - c for n, c in zip(lens, counts)]
        skip = 3
        q = torch.cat([torch.randn((skip, H, d)).bfloat16()] + [s[0][a:] for s, a in zip(seqs, starts)])
        gate = torch.randn((q.shape[0], H + 3), generator=g).bfloat16().to(gpu)[:, 1:1 + H] if gated else None
        out = torch.full((q.shape[0], H, v), 7.0, dtype=torch.bfloat16, device=gpu)
        op("biased_prefill")(padded_rows(q, d).to(gpu), kp, vp, d, v, i32(biased_prefill_tiles(counts, starts, skip, 0), gpu), table, scale,
                             torch.zeros(q.shape[0], dtype=torch.int32, device=gpu), out=out, scores=scores(gpu, cap, sinks=sinks, **mask), gate=gate)
        assert (out[:skip] == 7).all()
        at = skip
        for s, a, n in zip(seqs, starts, counts):
            want = O.masked_attention(*(t.to(D) for t in s), scale, cap, oracle_mask(a + n, **mask), None if sinks is None else sinks.float().to(D))[a:]
            if gated:
                want = want * O.sigmoid(gate[at:at + n].to(D).cpu())[:, :, None]
            err = (out[at:at + n].double().cpu() - want).flatten(1).norm(dim=1) / want.flatten(1).norm(dim=1)
            assert err.max() < 6e-3, (mask, a, n, err.argmax())
            at += n


@pytest.mark.parametrize("kind", ["rows float32", "decode", "prefill"])
@pytest.mark.parametrize("mask,distances", [(dict(window=70, keep=18), (69, 70)), (dict(window=64, keep=32), (63, 64)), (dict(window=100), (99, 100)), (dict(chunk=96), (1, 95, 96)),
                                            (dict(chunk=50), (49, 50))])
def test_every_query_at_an_edge(gpu, kind, mask, distances):
    """For every query the key at one distance stands out far above all others: it takes nearly all the weight where it is visible, and
    none where it is not.  The first tokens' last visible key and the one behind it stand out for all."""
    from nano_vllm_ninetoothed_amd.mops.hip.attention_ops import biased_prefill_tiles
    dtype = torch.float32 if kind == "rows float32" else torch.bfloat16
    H, G, d, v, n, bs, cap = 2, 1, 128, 16, 330, 32, 25.0
    g = torch.Generator().manual_seed(1)
    for distance in distances:
        seqs, kp, vp, table = paged_case(gpu, dtype, H, G, d, v, [n], bs, distance)
        q, k = 0.1 * torch.randn((n, H, d), generator=g), 0.1 * torch.randn((n, G, d), generator=g)
        for i in range(n):
            q[i, :, i % 120] = 4
            k[i, :, (i + distance) % 120] = 4
            q[i, :, 125] = 4
        for j in (mask.get("keep", 0) - 1, mask.get("keep", 0)):
            if 0 <= j:
                k[j, :, 125] = 4
        q, k, val = q.to(dtype), k.to(dtype), seqs[0][2]
        for b in range(-(-n // bs)):
            m = min(bs, n - b * bs)
            kp[table[0, b], :m] = k[b * bs:b * bs + m].to(gpu)
        s = scores(gpu, cap, **mask)
        if kind == "prefill":
            out = torch.empty((n, H, v), dtype=dtype, device=gpu)
            op("biased_prefill")(q.to(gpu), kp, vp, d, v, i32(biased_prefill_tiles([n], [0], 0, 0), gpu), table, 1.0, torch.zeros(n, dtype=torch.int32, device=gpu), out=out, scores=s)
        else:
            out = op("biased_decode" if kind == "decode" else "biased_attention_rows")(q.to(gpu), kp, vp, d, v, i32(list(range(1, n + 1)), gpu), table, 1.0,
                                                                                       row_seq=i32([0] * n, gpu), scores=s)
        want = O.masked_attention(q.to(D), k.to(D), val.to(D), 1.0, cap, oracle_mask(n, **mask))
        err = (out.double().cpu() - want).flatten(1).norm(dim=1) / want.flatten(1).norm(dim=1)
        assert err.max() < limit(dtype, 1e-5, 6e-3), (distance, int(err.argmax()))


def test_a_sink_that_outweighs_everything_and_one_that_weighs_nothing(gpu):
    H, G, d, v, n = 4, 2, 64, 32, 100
    sinks = torch.tensor([300.0, -300.0, 60.0, 0.0])
    seqs, kp, vp, table = paged_case(gpu, torch.bfloat16, H, G, d, v, [n], 32, 0)
    q, k, val = seqs[0]
    for cap in (20.0, 90.0):
        want = O.masked_attention(q.to(D), k.to(D), val.to(D), 0.2, cap, O.chunk_mask(n, 1000), sinks.to(D))
        got = op("biased_decode")(q.to(gpu), kp, vp, d, v, i32(list(range(1, n + 1)), gpu), table, 0.2, row_seq=i32([0] * n, gpu), scores=scores(gpu, cap, sinks=sinks))
        assert torch.isfinite(got).all() and (got[:, 0].abs() < 1e-30).all() and rel(got[:, 1:], want[:, 1:]) < 5e-3
        assert rel(got[:, 2], want[:, 2]) < 1e-2


def test_decode_with_many_rows(gpu):
    """More rows than the run search has lanes, of very different lengths, some cut over several runs."""
    H, G, d, v = 4, 2, 64, 32
    g = torch.Generator().manual_seed(1)
    lens = [int(x) for x in torch.randint(1, 130, (150,), generator=g)]
    lens[70] = 1500
    seqs, kp, vp, table = paged_case(gpu, torch.bfloat16, H, G, d, v, lens, 32, 5)
    sinks = torch.randn(H, generator=g)
    for mask in (dict(chunk=1024), dict(chunk=60), dict(window=900, keep=70), dict(window=40, keep=33)):
        got = op("biased_decode")(torch.stack([s[0][-1] for s in seqs]).to(gpu), kp, vp, d, v, i32(lens, gpu), table, 0.3, scores=scores(gpu, 10.0, sinks=sinks, **mask))
        for i in (0, 1, 63, 64, 69, 70, 71, 149):
            q, k, val = (t.to(D) for t in seqs[i])
            want = O.masked_attention(q[-1:], k, val, 0.3, 10.0, oracle_mask(lens[i], **mask)[-1:], sinks.to(D))[0]
            assert rel(got[i], want) < 5e-3, (mask, i)


def test_pages_beyond_what_a_row_sees_do_not_matter(gpu):
    """Not even when they hold no numbers."""
    from nano_vllm_ninetoothed_amd.mops.hip.attention_ops import biased_prefill_tiles
    H, G, d, v, n = 4, 2, 64, 64, 512
    seqs, kp, vp, table = paged_case(gpu, torch.bfloat16, H, G, d, v, [n], 32, 0)
    for mask, dead in ((dict(window=64, keep=32), range(2, 12)), (dict(chunk=128), range(0, 12))):
        s = scores(gpu, 10.0, **mask)
        q = seqs[0][0][448:]
        run = lambda: (op("biased_decode")(q.to(gpu), kp, vp, d, v, i32(list(range(449, 513)), gpu), table, 0.3, row_seq=i32([0] * 64, gpu), scores=s),      # noqa: E731
                       op("biased_prefill")(q.to(gpu), kp, vp, d, v, i32(biased_prefill_tiles([64], [448], 0, 0), gpu), table, 0.3, i32([0] * 64, gpu), scores=s))
        clean = run()
        kp[table[0, list(dead)].long()], vp[table[0, list(dead)].long()] = float("nan"), float("nan")
        for a, b in zip(clean, run()):
            assert torch.equal(a, b)


# ---------------------------------------------------------------------------------------------------- mixture of experts
@pytest.mark.parametrize("dtype,block", [(torch.float32, 32), (torch.bfloat16, 32), (torch.bfloat16, 128)])
@pytest.mark.parametrize("tokens,width,ff,experts,top,count,keep", [(1, 64, 32, 4, 1, 2, 1), (70, 72, 24, 6, 2, 3, 2), (300, 256, 136, 16, 4, 4, 2), (40, 50, 17, 3, 2, 3, 2), (33, 128, 40, 130, 2, 65, 30),
                                                                    (129, 96, 64, 1, 1, 1, 1), (257, 64, 200, 33, 1, 3, 1), (2500, 64, 32, 20, 3, 1, 1), (2111, 48, 16, 8, 8, 2, 2),
                                                                    (35, 64, 24, 14, 5, 2, 1), (20, 64, 24, 256, 6, 8, 3)])
def test_weighted_mixture(gpu, dtype, block, tokens, width, ff, experts, top, count, keep):
    from nano_vllm_ninetoothed_amd.mops.hip.mixture_ops import Weighted
    g = torch.Generator().manual_seed(experts)
    h, router = torch.randn((tokens, width), generator=g).to(dtype), (torch.randn((experts, width), generator=g) * 2 * width ** -0.5).to(dtype)
    correction = torch.randn(experts, generator=g) * 0.4 - 0.8      # most choice scores are negative
    m = {"top": top, "groups": {"count": count, "keep": keep}, "scale": 1.3}
    routing = op("moe_route")(h.to(gpu), router.to(gpu), top, block, weighted=Weighted(correction.to(gpu), count, keep, 1.3))
    with O.watching_choices() as margins:
        chosen, weight = O.route(h.to(D), router.to(D), correction.to(D), m)
    clear = margins[0] > 1e-5
    assert clear.float().mean() > 0.97
    got = routing.chosen.cpu().long()
    assert torch.equal(got[clear].sort(1).values, chosen[clear].sort(1).values)
    s = O.sigmoid(h.to(D) @ router.to(D).T).gather(1, got)
    assert all(len(set(r)) == top for r in got.tolist()) and rel(routing.score, s / (s.sum(1, keepdim=True) + 1e-20) * 1.3) < 1e-5
    c = (O.sigmoid(h.to(D) @ router.to(D).T) + correction.to(D)).gather(1, got)
    assert (c.diff(dim=1) <= 1e-5).all()      # the best first
    rows = routing.rows.cpu().long()
    assert sorted(rows.tolist()) == list(range(tokens * top)) and (got.flatten()[rows].diff() >= 0).all()
    pad = -ff % 8
    gu, down = torch.zeros((experts, 2, ff + pad, width)).to(dtype), torch.zeros((experts, width, ff + pad)).to(dtype)
    gu[:, :, :ff] = torch.randn((experts, 2, ff, width), generator=g) * width ** -0.5 * 2
    down[:, :, :ff] = torch.randn((experts, width, ff), generator=g) * ff ** -0.5
    y = op("moe_gate_up")(h.to(gpu), gu.to(gpu), routing, 1.5)
    z = op("moe_down")(y, down.to(gpu), routing)
    want = torch.empty((tokens, top, width), dtype=D)
    for t in range(tokens):
        for p in range(top):
            e = int(got[t, p])
            unit = {"gate": gu[e, 0, :ff].to(D), "up": gu[e, 1, :ff].to(D), "down": down[e, :, :ff].to(D)}
            want[t, p] = O.clamped_unit(h[t:t + 1].to(D), unit, 1.5)[0] * routing.score[t, p].double().cpu()
        if t >= 300:
            break
    n = min(tokens, 301)
    assert rel(z.view(tokens, top, width)[:n], want[:n]) < limit(dtype, 3e-6, 8e-3)


@pytest.mark.parametrize("tokens,width,ff,experts,top,shared", [(1, 64, 32, 4, 1, 72), (70, 72, 24, 6, 2, 17), (33, 256, 136, 16, 4, 300), (64, 100, 16, 3, 2, 8), (150, 64, 24, 16, 2, 1030)])
def test_a_shared_unit_in_the_launches_of_the_experts(gpu, tokens, width, ff, experts, top, shared):
    from nano_vllm_ninetoothed_amd.mops.hip.mixture_ops import CommonUnit, Weighted
    g = torch.Generator().manual_seed(shared)
    rnd = lambda *s: (torch.randn(s, generator=g) * s[-1] ** -0.5).bfloat16().to(gpu)      # noqa: E731
    h, pad, half = torch.randn((tokens, width), generator=g).bfloat16().to(gpu), (ff + 7) // 8 * 8, (shared + 7) // 8 * 8
    gu, down, cg, cd = 2 * rnd(experts, 2, pad, width), rnd(experts, width, pad), 2 * rnd(half + (shared + 7) // 8 * 8, width), rnd(width, shared)
    gu[:, :, ff:], down[:, :, ff:] = 0, 0
    routing = op("moe_route")(h, rnd(experts, width), top, 32, weighted=Weighted(torch.randn(experts, generator=g).to(gpu), 1, 1, 1.0))
    assert routing.takes_common
    unit = CommonUnit(cg, cd, shared, half, 0.7)
    y, yc = op("moe_gate_up")(h, gu, routing, 1.5, common=unit)
    z, zc = op("moe_down")(y, down, routing, unit, yc)
    assert torch.equal(y, op("moe_gate_up")(h, gu, routing, 1.5)) and torch.equal(z, op("moe_down")(y, down, routing))
    w = {"gate": cg[:shared].double().cpu(), "up": cg[half:half + shared].double().cpu(), "down": cd.double().cpu()}
    assert yc.shape == (tokens, shared) and rel(zc, O.clamped_unit(h.double().cpu(), w, 0.7)) < 8e-3
    big = op("moe_route")(h, rnd(experts, width), top, 128, weighted=Weighted(torch.randn(experts, generator=g).to(gpu), 1, 1, 1.0))
    assert not big.takes_common
    with pytest.raises(Exception):
        op("moe_gate_up")(h, gu, big, 1.5, common=unit)


def test_groups_that_lose_are_out_even_with_the_best_expert(gpu):
    """The single best expert stands in a group whose two best add up to less; negative choice scores are still taken from kept groups."""
    from nano_vllm_ninetoothed_amd.mops.hip.mixture_ops import Weighted
    router = torch.zeros((6, 8))
    correction = torch.tensor([0.4, -0.9, 0.1, 0.1, -2.0, -2.0])      # every sigmoid is a half: groups of two score 0.5, 1.2, -3
    for dtype in DTYPES:
        args = torch.ones((3, 8), dtype=dtype, device=gpu), router.to(dtype).to(gpu)
        r = op("moe_route")(*args, 2, weighted=Weighted(correction.to(gpu), 3, 1, 2.0))
        assert r.chosen.tolist() == [[2, 3]] * 3 and torch.allclose(r.score, torch.ones(3, 2, device=gpu))
        r = op("moe_route")(*args, 4, weighted=Weighted(correction.to(gpu), 3, 2, 2.0))
        assert r.chosen.tolist() == [[0, 2, 3, 1]] * 3 and torch.allclose(r.score, torch.full((3, 4), 0.5, device=gpu))


def test_weighted_routing_replays(gpu):
    from nano_vllm_ninetoothed_amd.mops.hip.mixture_ops import Weighted
    width, ff, experts, top, tokens = 64, 32, 8, 2, 200
    g = torch.Generator().manual_seed(0)
    router, w = torch.randn((experts, width), generator=g).bfloat16().to(gpu), torch.randn((experts, 2, ff, width), generator=g).bfloat16().to(gpu)
    down = torch.randn((experts, width, ff), generator=g).bfloat16().to(gpu)
    form = Weighted(torch.randn(experts, generator=g).to(gpu), 4, 2, 2.5)
    x = torch.randn((tokens, width), generator=g).bfloat16().to(gpu)

    def run():
        routing = op("moe_route")(x, router, top, weighted=form)
        return routing, op("moe_down")(op("moe_gate_up")(x, w, routing, 1.0), down, routing)
    run()
    torch.cuda.synchronize()
    graph = torch.cuda.CUDAGraph()
    with torch.cuda.graph(graph):
        routing, z = run()
    for seed in range(3):
        x.copy_(torch.randn((tokens, width), generator=torch.Generator().manual_seed(seed)).bfloat16())
        graph.replay()
        eager, ze = run()
        torch.cuda.synchronize()
        assert torch.equal(routing.chosen, eager.chosen) and torch.equal(routing.score, eager.score) and torch.equal(z, ze)
