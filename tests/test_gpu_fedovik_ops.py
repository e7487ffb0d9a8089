"""GPU: the operators of Fedovik models, each alone, against oracle/fedovik.py in float64."""
import pytest
import torch

from op_harness import bounds, i32, limit, op, padded_rows, paged_case, rel
from oracle import fedovik as O

pytestmark = pytest.mark.gpu
D = torch.float64
DTYPES = [torch.float32, torch.bfloat16]


# ---------------------------------------------------------------------------------------------------- rows
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rows,n", [(5, 72), (3, 1024), (2, 101), (4, 2048), (1, 10000), (2, 700), (3, 8), (2, 2504)])
def test_add_norm(gpu, dtype, rows, n):
    """Rows whose mean is far larger than their spread; sums, replacements, plain copies into wider rows."""
    g = torch.Generator().manual_seed(n)
    x, y = torch.randn((rows, n), generator=g) + 30, (torch.randn((rows, n + 8), generator=g) - 3).to(dtype)[:, :n]
    shift = torch.randn(n, generator=g) * 2
    w, b = (torch.randn(n, generator=g).to(dtype) for _ in range(2))
    for use_y, use_shift, replace in ((True, True, False), (True, False, False), (False, True, False), (False, False, False), (True, True, True), (True, False, True)):
        total = (0 if replace else x.to(D)) + (y.to(D) if use_y else 0) + (shift.to(D) if use_shift else 0)
        for norm in ("layer", "rms", "none"):
            res, wide = x.clone().to(gpu), torch.full((rows, 2 * n), 7.0, dtype=dtype, device=gpu)
            out = op("add_norm")(res, y.to(gpu) if use_y else None, shift.to(gpu) if use_shift else None, replace, None if norm == "none" else w.to(gpu),
                                 b.to(gpu) if norm == "layer" else None, 1e-4, center=norm == "layer", out=wide[:, n:] if norm == "none" else None)
            want = {"layer": O.layer_norm(total, w.to(D), b.to(D), 1e-4), "rms": O.over_rms(total, 1e-4) * w.to(D), "none": total}[norm]
            assert rel(res, total) < 1e-6 and rel(out, want) < limit(dtype, 4e-6), (norm, use_y, use_shift, replace)
            assert norm != "none" or (wide[:, :n] == 7).all()


@pytest.mark.parametrize("dtype", DTYPES)
def test_embedding_copy_into_wider_rows(gpu, dtype):
    g = torch.Generator().manual_seed(0)
    for width in (64, 41):
        table, ids = torch.randn((50, width), generator=g).to(dtype), torch.randint(0, 50, (9,), generator=g)
        pair = torch.full((9, 2 * width), 7.0, dtype=dtype, device=gpu)
        res, _ = op("embed_residual")(ids.to(gpu), table.to(gpu), 3.5, need_act=False, act=pair[:, width:])
        assert rel(res, table[ids].to(D) * 3.5) < 1e-6 and rel(pair[:, width:], table[ids].to(D) * 3.5) < limit(dtype) and (pair[:, :width] == 7).all()


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("groups,size", [(6, 48), (3, 64), (1, 128), (4, 300), (5, 13), (2, 1030)])
def test_gated_group_norm_with_a_sigmoid(gpu, dtype, groups, size):
    """Weights for the whole row or shared by the groups, a factor, rows of a wider matrix as result."""
    g = torch.Generator().manual_seed(size)
    n = groups * size
    y, z = torch.randn((7, n), generator=g).to(dtype), torch.randn((7, n + 16), generator=g).to(dtype)[:, 8:8 + n]
    for shared in (False, True):
        w = torch.randn(size if shared else n, generator=g).to(dtype)
        wide = torch.full((7, n + 24), 7.0, dtype=dtype, device=gpu)
        op("gated_group_norm")(y.to(gpu), z.to(gpu), groups, 1e-3, weight=w.to(gpu), activation="sigmoid", scale=1.3, out=wide[:, 8:8 + n])
        want = O.over_rms(y.to(D).view(7, groups, size), 1e-3).reshape(7, n) * (w.to(D).repeat(groups) if shared else w.to(D)) * O.sigmoid(z.to(D)) * 1.3
        assert rel(wide[:, 8:8 + n], want) < limit(dtype) and (wide[:, :8] == 7).all() and (wide[:, 8 + n:] == 7).all()


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("n", [256, 41])
def test_relu_glu(gpu, dtype, n):
    p = torch.randn((5, 2 * n), generator=torch.Generator().manual_seed(n)).to(dtype)
    wide = torch.zeros((5, n + 8), dtype=dtype, device=gpu)
    op("relu_glu")(p.to(gpu)[:, :n], p.to(gpu)[:, n:], out=wide[:, 8:])
    assert rel(wide[:, 8:], p[:, :n].to(D).clamp(min=0) * p[:, n:].to(D)) < limit(dtype) and (wide[:, :8] == 0).all()


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("tokens,heads,dim,rank", [(5, 4, 64, 24), (70, 3, 20, 16), (3, 1, 300, 300), (2100, 2, 32, 9)])
def test_low_rank_decay_with_a_rate(gpu, dtype, tokens, heads, dim, rank):
    """Decays from nearly one, whose logarithms must keep their digits, to nearly nothing."""
    g = torch.Generator().manual_seed(rank)
    z, w2 = torch.randn((tokens, (rank + 7) // 8 * 8), generator=g).to(dtype), (torch.randn((heads * dim, rank), generator=g) * rank ** -0.5).to(dtype)
    a_log = torch.randn(heads, generator=g)
    for at in (-14.0, -5.0, 0.0, 30.0):
        bias = torch.randn(heads * dim, generator=g) + at
        got = op("low_rank_decay")(z.to(gpu)[:, :rank], w2.to(gpu), bias.to(gpu), rate=-torch.exp(a_log).to(gpu))
        want = torch.log(O.channel_decays(z[:, :rank].to(D) @ w2.to(D).T, a_log.to(D), bias.to(D), heads)).reshape(tokens, -1)
        err = ((got.double().cpu() - want) / want).abs().max()
        assert got.dtype == torch.float32 and err < 6e-5, at


@pytest.mark.parametrize("dtype", DTYPES)
def test_short_convolution_without_a_bias(gpu, dtype):
    g = torch.Generator().manual_seed(3)
    for channels, taps, n in ((64, 4, 300), (41, 4, 20), (24, 1, 9), (16, 6, 40), (64, 2, 270)):
        x, w = torch.randn((n, channels), generator=g).to(dtype), torch.randn((channels, taps), generator=g).to(dtype)
        ring = torch.full((2, taps, channels), float("nan"), dtype=dtype, device=gpu)
        cut, slots, want = n // 3, i32([1], gpu), O.short_convolution(x.to(D), w.to(D))
        got = []
        for a, b in ((0, cut), (cut, n)):
            part, cu, start = x[a:b].to(gpu), i32([0, b - a], gpu), i32([a], gpu)
            got.append(op("short_conv")(part, w.float().t().contiguous().to(gpu), None, ring, i32([0] * (b - a), gpu), cu, start, slots))
            op("short_conv_update")(part, ring, cu, start, slots)
        assert rel(torch.cat(got), want) < limit(dtype)


# ---------------------------------------------------------------------------------------------------- attention
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,G,d,v,rot,norms", [(8, 4, 64, 32, 64, False), (6, 3, 20, 13, 14, False), (2, 1, 24, 8, 8, True), (4, 4, 128, 128, 0, True), (3, 1, 272, 40, 100, True),
                                              (2, 2, 6, 40, 2, False)])
def test_rotary_prepare_with_neighbours_and_biases(gpu, dtype, H, G, d, v, rot, norms):
    from nano_vllm_ninetoothed_amd.layers import Rotary
    from nano_vllm_ninetoothed_amd.mops.hip.attention_ops import padded
    g = torch.Generator().manual_seed(d)
    n = (H + G) * d + G * v
    x, bias = torch.randn((9, (n + 12) // 8 * 8), generator=g).to(dtype), torch.randn(n, generator=g).to(dtype)
    wq, wk = ((torch.randn(d, generator=g).to(dtype) for _ in range(2)) if norms else (None, None))
    pos, slots = [0, 5, 6, 7, 12, 13, 14, 40, 200], [3, -1, 8, 9, 31, 0, 16, 15, 20]
    kp, vp = (torch.full((2, 16, G, padded(s)), float("nan"), dtype=dtype, device=gpu) for s in (d, v))
    on = lambda t: None if t is None else t.to(gpu)      # noqa: E731
    q = op("rotary_prepare")(x.to(gpu), i32(pos, gpu), i32(slots, gpu), kp, vp, H, G, d, v, cos_sin=Rotary(256, gpu).table(3e3, rot) if rot else None,
                             q_weight=on(wq), k_weight=on(wk), eps=1e-5, bias=bias.to(gpu), neighbours=True)
    full = x[:, :n].to(D) + bias.to(D)

    def turned(part, heads, w):
        y = part.reshape(9, heads, d)
        y = y if w is None else O.over_rms(y, 1e-5) * w.to(D)
        return O.rotate_neighbours(y, torch.tensor(pos), 3e3, rot) if rot else y
    assert rel(q[..., :d], turned(full[:, :H * d], H, wq)) < limit(dtype) and (q[..., d:] == 0).all()
    ok = [i for i, s in enumerate(slots) if s >= 0]
    at = [slots[i] for i in ok]
    kf, vf = kp.view(32, G, -1)[at].cpu(), vp.view(32, G, -1)[at].cpu()
    assert rel(kf[..., :d], turned(full[:, H * d:(H + G) * d], G, wk)[ok]) < limit(dtype) and (kf[..., d:] == 0).all()
    assert rel(vf[..., :v], full[ok][:, (H + G) * d:].reshape(-1, G, v)) < limit(dtype) and (vf[..., v:] == 0).all()
    rest = [s for s in range(32) if s not in at]
    assert kp.view(32, -1)[rest].isnan().all() and vp.view(32, -1)[rest].isnan().all()


class Kind:
    """A kind of attention: what the operators take, and the oracle's outputs for a whole sequence."""

    def __init__(self, gpu, kind, H, seed):
        from nano_vllm_ninetoothed_amd.mops.hip.attention_ops import Scores
        g = torch.Generator().manual_seed(seed)
        self.name, self.window = kind[0], kind[1]
        if self.name == "sigmoid":
            self.bias = torch.randn(H, generator=g) * 2 - 2
            self.scores = Scores(weight_bias=self.bias.to(gpu))
        else:
            self.rate, self.step = torch.rand(H, generator=g) * 2, torch.rand(H, generator=g) * 3
            self.step[0] = 0 if H > 1 else 0.5
            self.scores = Scores(window=self.window, log_distance=(self.rate.to(gpu), self.step.to(gpu)))

    def __call__(self, q, k, v, scale):
        s = O.scores(q.to(D), k.to(D), scale)
        if self.name == "sigmoid":
            return O.weighted(O.sigmoid_weights(s, self.bias.to(D)), v.to(D))
        return O.weighted(O.log_distance_weights(s, self.rate.to(D), self.step.to(D), self.window), v.to(D))


KINDS = [("sigmoid", 0), ("log distance", 72), ("log distance", 64), ("log distance", 1), ("log distance", 33), ("log distance", 5000), ("log distance", 190)]
SIZES = [(8, 2, 64, 64), (6, 3, 20, 13), (20, 1, 128, 128), (3, 1, 24, 256), (16, 8, 128, 128), (4, 4, 64, 32), (6, 2, 64, 128), (2, 1, 40, 1)]


def edge_positions(n, kind):
    """Just inside and just outside of what the last row sees."""
    return sorted({max(0, n - 1 - w) for w in (kind[1] - 1, kind[1])} | {0, n // 2}) if kind[1] else [0, 1, n // 3]


@pytest.mark.parametrize("H,G,d,v", SIZES)
@pytest.mark.parametrize("kind", ["rows float32", "rows bfloat16", "decode"])
def test_single_rows(gpu, kind, H, G, d, v):
    """Rows of several sequences at once, around pages, stages and windows, with keys that stand out; gates per element and per head, a
    factor, and results into rows of a wider matrix."""
    dtype = torch.float32 if kind == "rows float32" else torch.bfloat16
    name = "biased_decode" if kind == "decode" else "biased_attention_rows"
    g = torch.Generator().manual_seed(H)
    scale = 1.2 * d ** -0.5
    for m, form in enumerate(KINDS):
        bs, lens = ((32, [300, 1, 33, 201]), (64, [700, 65]), (32, [401]))[m % 3]
        attention = Kind(gpu, form, H, m)
        seqs, kp, vp, table = paged_case(gpu, dtype, H, G, d, v, lens, bs, H + m, edge_positions(lens[0], form))
        rows = [(i, c) for i, n in enumerate(lens) for c in sorted({1, 2, n // 2 + 1, max(1, n - 1), n, 64, 65, 71, 73, 191} & set(range(1, n + 1)))]
        rows.insert(2, (0, 0))
        q = torch.stack([seqs[i][0][max(c - 1, 0)] for i, c in rows])
        columns = {0: H * v, 1: H, 2: 0}[m % 3]
        gate = torch.randn((len(rows), columns + 16), generator=g).to(dtype).to(gpu)[:, 8:8 + columns] if columns else None
        wide = torch.full((len(rows), H * v + 16), 7.0, dtype=dtype, device=gpu)
        op(name)(padded_rows(q, d).to(gpu), kp, vp, d, v, i32([c for _, c in rows], gpu), table, scale, row_seq=i32([i for i, _ in rows], gpu),
                 scores=attention.scores, gate=gate, out=wide[:, 8:8 + H * v], out_scale=0.6)
        assert (wide[:, :8] == 7).all() and (wide[:, 8 + H * v:] == 7).all()
        got = wide[:, 8:8 + H * v].reshape(-1, H, v)
        assert (got[2] == 0).all()
        for j, (i, c) in enumerate(rows):
            if c:
                want = 0.6 * attention(*(t[:c] for t in seqs[i]), scale)[-1]
                if columns:
                    want = want * O.sigmoid(gate[j].to(D).cpu().view(H, -1))
                assert rel(got[j], want) < limit(dtype, 3e-6, 6e-3), (form, i, c)


@pytest.mark.parametrize("H,G,d,v", SIZES)
def test_long_portions(gpu, H, G, d, v):
    """Portions behind cached tokens and from the start, packed behind rows that the launch must leave alone."""
    from nano_vllm_ninetoothed_amd.mops.hip.attention_ops import biased_prefill_tiles
    g = torch.Generator().manual_seed(d)
    scale, skip = 1.2 * d ** -0.5, 3
    for m, form in enumerate(KINDS):
        bs, lens, counts = ((32, [130, 64, 300], [130, 33, 70]), (64, [513, 1], [300, 1]), (48, [397], [396]))[m % 3]
        attention = Kind(gpu, form, H, m)
        seqs, kp, vp, table = paged_case(gpu, torch.bfloat16, H, G, d, v, lens, bs, d + m, far=(0, 17, 63, 64, 71, 72, 127, 128, 189, 190))
        starts = [n - c for n, c in zip(lens, counts)]
        q = torch.cat([torch.randn((skip, H, d)).bfloat16()] + [s[0][a:] for s, a in zip(seqs, starts)])
        columns = {0: H * v, 1: H, 2: 0}[m % 3]
        gate = torch.randn((q.shape[0], columns + 16), generator=g).bfloat16().to(gpu)[:, 8:8 + columns] if columns else None
        wide = torch.full((q.shape[0], H * v + 16), 7.0, dtype=torch.bfloat16, device=gpu)
        op("biased_prefill")(padded_rows(q, d).to(gpu), kp, vp, d, v, i32(biased_prefill_tiles(counts, starts, skip, 0), gpu), table, scale,
                             torch.zeros(q.shape[0], dtype=torch.int32, device=gpu), out=wide[:, 8:8 + H * v], scores=attention.scores, gate=gate, out_scale=1.1)
        assert (wide[:skip] == 7).all() and (wide[:, :8] == 7).all() and (wide[:, 8 + H * v:] == 7).all()
        at = skip
        for s, a, n in zip(seqs, starts, counts):
            want = 1.1 * attention(*s, scale)[a:]
            if columns:
                want = want * O.sigmoid(gate[at:at + n].to(D).cpu().view(n, H, -1))
            err = (wide[at:at + n, 8:8 + H * v].double().cpu() - want.flatten(1)).norm(dim=1) / want.flatten(1).norm(dim=1)
            assert err.max() < 7e-3, (form, a, n, err.argmax())
            at += n


@pytest.mark.parametrize("kind", ["rows float32", "decode", "prefill"])
@pytest.mark.parametrize("window,distances", [(72, (71, 72)), (64, (63, 64)), (100, (99, 100)), (33, (32, 33))])
def test_every_query_at_the_edge_of_a_window(gpu, kind, window, distances):
    """For every query the key at one distance stands out far above all others: it takes nearly all the weight where it is visible, and
    none where it is not."""
    from nano_vllm_ninetoothed_amd.mops.hip.attention_ops import biased_prefill_tiles
    dtype = torch.float32 if kind == "rows float32" else torch.bfloat16
    H, G, d, v, n, bs = 2, 1, 128, 16, 330, 32
    g = torch.Generator().manual_seed(1)
    attention = Kind(gpu, ("log distance", window), H, 3)
    for distance in distances:
        seqs, kp, vp, table = paged_case(gpu, dtype, H, G, d, v, [n], bs, distance)
        q, k = 0.1 * torch.randn((n, H, d), generator=g), 0.1 * torch.randn((n, G, d), generator=g)
        for i in range(n):
            q[i, :, i % 120] = 5
            k[i, :, (i + distance) % 120] = 5
        q, k, val = q.to(dtype), k.to(dtype), seqs[0][2]
        for b in range(-(-n // bs)):
            m = min(bs, n - b * bs)
            kp[table[0, b], :m] = k[b * bs:b * bs + m].to(gpu)
        if kind == "prefill":
            out = torch.empty((n, H, v), dtype=dtype, device=gpu)
            op("biased_prefill")(q.to(gpu), kp, vp, d, v, i32(biased_prefill_tiles([n], [0], 0, 0), gpu), table, 1.0, torch.zeros(n, dtype=torch.int32, device=gpu),
                                 out=out, scores=attention.scores)
        else:
            out = op("biased_decode" if kind == "decode" else "biased_attention_rows")(q.to(gpu), kp, vp, d, v, i32(list(range(1, n + 1)), gpu), table, 1.0,
                                                                                       row_seq=i32([0] * n, gpu), scores=attention.scores)
        want = attention(q, k, val, 1.0)
        err = (out.double().cpu() - want).flatten(1).norm(dim=1) / want.flatten(1).norm(dim=1)
        assert err.max() < limit(dtype, 1e-5, 6e-3), (distance, int(err.argmax()))


def test_sigmoid_weights_far_from_zero(gpu):
    """Scores whose exponentials overflow either way: weights of one and of nothing."""
    from nano_vllm_ninetoothed_amd.mops.hip.attention_ops import Scores, biased_prefill_tiles
    H, G, d, v, n = 4, 2, 64, 32, 100
    bias = torch.tensor([200.0, -200.0, -8.0, 3.0])
    seqs, kp, vp, table = paged_case(gpu, torch.bfloat16, H, G, d, v, [n], 32, 0)
    q, k, val = seqs[0]
    for scale in (0.1, 20.0):
        want = O.weighted(O.sigmoid_weights(O.scores(q.to(D), k.to(D), scale), bias.to(D)), val.to(D))
        rows = op("biased_decode")(q.to(gpu), kp, vp, d, v, i32(list(range(1, n + 1)), gpu), table, scale, row_seq=i32([0] * n, gpu), scores=Scores(weight_bias=bias.to(gpu)))
        tiles = op("biased_prefill")(q.to(gpu), kp, vp, d, v, i32(biased_prefill_tiles([n], [0], 0, 0), gpu), table, scale, torch.zeros(n, dtype=torch.int32, device=gpu),
                                     scores=Scores(weight_bias=bias.to(gpu)))
        for got in (rows, tiles):
            assert torch.isfinite(got).all() and rel(got[:, [0, 2, 3]], want[:, [0, 2, 3]]) < 8e-3
            assert scale > 1 or (got[:, 1].abs() < 1e-30).all()


def test_decode_with_many_rows(gpu):
    """More rows than the run search has lanes, of very different lengths, some cut over several runs."""
    H, G, d, v = 4, 2, 64, 32
    lens = [int(x) for x in torch.randint(1, 130, (150,), generator=torch.Generator().manual_seed(1))]
    lens[70] = 1500
    seqs, kp, vp, table = paged_case(gpu, torch.bfloat16, H, G, d, v, lens, 32, 5)
    gate = torch.randn((150, H * v), generator=torch.Generator().manual_seed(2)).bfloat16().to(gpu)
    for form in (("sigmoid", 0), ("log distance", 900), ("log distance", 40)):
        attention = Kind(gpu, form, H, 7)
        got = op("biased_decode")(torch.stack([s[0][-1] for s in seqs]).to(gpu), kp, vp, d, v, i32(lens, gpu), table, 0.3, scores=attention.scores, gate=gate)
        for i in (0, 1, 63, 64, 69, 70, 71, 149):
            want = attention(*seqs[i], 0.3)[-1] * O.sigmoid(gate[i].to(D).cpu().view(H, v))
            assert rel(got[i], want) < 6e-3, (form, i)


# ---------------------------------------------------------------------------------------------------- gated delta rule
def usual(g, shape):
    return -torch.exp(torch.randn(shape, generator=g) * 1.5 - 3)


def strong(g, shape):      # decays down to e^-400 beside some near one
    return -torch.exp(torch.randn(shape, generator=g) * 3 + 1)


def weak(g, shape):
    return -torch.exp(torch.randn(shape, generator=g) * 0.5 - 9)


def run_delta(gpu, which, dtype, H, G, d, vd, counts, starts, log_decay, seed=0, slots=None, alike=0.0, beta_at=0.0, wanted=256):
    """Largest relative errors of outputs and states over the sequences.  alike: how much of a key all keys of a head share."""
    from nano_vllm_ninetoothed_amd.mops.hip import recurrent_ops as R
    g = torch.Generator().manual_seed(seed)
    T, B, cu = sum(counts), len(counts), bounds(counts)
    wide = torch.randn((T, 2 * G * d + H * vd + 8), generator=g)
    wide[:, G * d:2 * G * d] += alike * torch.randn(G * d, generator=g)
    wide = wide.to(dtype)
    q, k, v = wide[:, :G * d], wide[:, G * d:2 * G * d], wide[:, 2 * G * d:2 * G * d + H * vd]
    lw = log_decay(g, (T, H * d))
    beta = (2 * torch.randn((T, H + 3), generator=g) + beta_at).to(dtype)
    S0 = torch.randn((B, H, d, vd), generator=g)
    slots = list(range(B, 0, -1)) if slots is None else slots
    state = torch.full((B + 2, H, vd, R.recurrence_state_pitch(d)), float("nan"))
    for b in range(B):
        if starts[b] and slots[b] >= 0:
            state[slots[b], :, :, :d] = S0[b].transpose(1, 2)
            state[slots[b], :, :, d:] = 0
    state, out = state.to(gpu), torch.full((T, H * vd + 8), float("nan"), dtype=dtype, device=gpu)[:, :H * vd]
    on = wide.to(gpu)
    args = [on[:, :G * d], on[:, G * d:2 * G * d], on[:, 2 * G * d:2 * G * d + H * vd], out, state, i32(slots, gpu), i32(starts, gpu), H, G, d, vd]
    options = dict(log_decay=lw.to(gpu), beta=beta.to(gpu)[:, :H], q_scale=d ** -0.5, unit_eps=1e-6, cu_seqlens=i32(cu, gpu))
    if which == "chunks":
        cuts = R.delta_cuts(counts, H, vd, wanted)
        op("delta_chunks")(*args, *(i32(x, gpu) for x in cuts), **options)
    else:
        if max(counts) == 1:
            del options["cu_seqlens"]
        op("delta_rule")(*args, **options)
    worst = [0.0, 0.0]
    for b in range(B):
        if slots[b] < 0:
            continue
        f = lambda x, heads: x[cu[b]:cu[b + 1]].to(D).reshape(counts[b], heads, -1)      # noqa: E731
        o, S = O.delta_rule(O.unit(f(q, G)) * d ** -0.5, O.unit(f(k, G)), f(v, H), torch.exp(f(lw, H)), O.sigmoid(beta[cu[b]:cu[b + 1], :H].to(D)),
                            S0[b].to(D) if starts[b] else None)
        worst[0] = max(worst[0], rel(out[cu[b]:cu[b + 1]].reshape(counts[b], H, vd), o))
        worst[1] = max(worst[1], rel(state[slots[b], :, :, :d].transpose(1, 2), S))
    return worst


DELTA_SIZES = [(4, 4, 64, 64), (6, 2, 32, 48), (2, 1, 20, 20), (2, 2, 128, 128), (3, 1, 33, 70), (1, 1, 256, 200), (2, 2, 16, 8), (2, 1, 48, 130), (1, 1, 8, 1)]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,G,d,vd", DELTA_SIZES + [(1, 1, 300, 24)])
def test_delta_rule_token_by_token(gpu, dtype, H, G, d, vd):
    for decay in (usual, strong, weak):
        o, S = run_delta(gpu, "plain", dtype, H, G, d, vd, [1] * 7, [0, 4, 1, 9, 0, 7, 2], decay, slots=[3, 1, -1, 0, 2, 8, 5])
        assert o < limit(dtype, 2e-6, 4e-3) and S < 1e-6
        o, S = run_delta(gpu, "plain", dtype, H, G, d, vd, [40, 2, 19], [0, 4, 1], decay, alike=1.0)
        assert o < limit(dtype, 4e-6, 4e-3) and S < 4e-6


@pytest.mark.parametrize("H,G,d,vd", DELTA_SIZES)
def test_delta_rule_in_chunks(gpu, H, G, d, vd):
    """Portions shorter and longer than chunks, and some that are cut into segments; all strengths of decay; keys that are nearly the same throughout, so that every write
    answers all those in front of it."""
    for seed, decay in enumerate((usual, strong, weak)):
        for counts, starts, alike in (([2, 37, 16, 1, 100], [0, 5, 3, 2, 0], 0.0), ([17], [4], 6.0), ([300, 33], [0, 7], 2.0), ([64], [0], 30.0), ([290, 517], [9, 0], 0.0), ([700], [3], 1.0)):
            o, S = run_delta(gpu, "chunks", torch.bfloat16, H, G, d, vd, counts, starts, decay, seed=seed, alike=alike, beta_at=2.0 if alike else 0.0)
            assert o < 4e-3 and S < 1e-4, (decay.__name__, counts, o, S)


def test_delta_chunks_leave_padding_slots_alone(gpu):
    o, S = run_delta(gpu, "chunks", torch.bfloat16, 2, 2, 64, 64, [20, 20, 20], [0, 3, 1], usual, slots=[2, -1, 0])
    assert o < 4e-3 and S < 1e-4


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,G,d,vd,taps", [(4, 2, 32, 24, 4), (3, 3, 20, 70, 2), (2, 1, 64, 8, 1), (1, 1, 16, 150, 6)])
def test_delta_decode_with_its_convolutions(gpu, dtype, H, G, d, vd, taps):
    """Single tokens one after the other with the convolution inside the step, against the convolution of the whole sequence."""
    from nano_vllm_ninetoothed_amd.mops.hip import recurrent_ops as R
    g = torch.Generator().manual_seed(d)
    n, at = 23, (0, G * d, 2 * G * d)
    channels = 2 * G * d + H * vd
    x, w = torch.randn((n, channels), generator=g).to(dtype), torch.randn((channels, taps), generator=g).to(dtype)
    lw, beta = usual(g, (n, H * d)), torch.randn((n, H), generator=g).to(dtype)
    state = torch.full((3, H, vd, R.recurrence_state_pitch(d)), float("nan"), device=gpu)
    ring = torch.full((3, taps, channels), float("nan"), dtype=dtype, device=gpu)
    out = torch.empty((n, H * vd), dtype=dtype, device=gpu)
    conv_w = w.float().t().contiguous().to(gpu)
    for t in range(n):
        row = x[t:t + 1].to(gpu)
        op("delta_rule")(row[:, :at[1]], row[:, at[1]:at[2]], row[:, at[2]:], out[t:t + 1], state, i32([1], gpu), i32([t], gpu), H, G, d, vd,
                         log_decay=lw[t:t + 1].to(gpu), beta=beta[t:t + 1].to(gpu), q_scale=d ** -0.5, unit_eps=1e-6, conv=(conv_w, ring, at))
    c = O.short_convolution(x.to(D), w.to(D))
    o, _ = O.delta_rule(O.unit(c[:, :at[1]].view(n, G, d)) * d ** -0.5, O.unit(c[:, at[1]:at[2]].view(n, G, d)), c[:, at[2]:].view(n, H, vd),
                        torch.exp(lw.to(D).view(n, H, d)), O.sigmoid(beta.to(D)))
    assert rel(out.view(n, H, vd), o) < limit(dtype, 3e-6, 6e-3)


# ---------------------------------------------------------------------------------------------------- matrix memory
def run_memory(gpu, which, dtype, H, d, vd, counts, starts, cap, gates_at, seed=0, slots=None, wanted=512):
    """Largest relative errors of outputs, states, normalizers and the largest absolute one of the running maxima."""
    from nano_vllm_ninetoothed_amd.mops.hip import recurrent_ops as R
    g = torch.Generator().manual_seed(seed)
    T, B, cu, copies, pitch = sum(counts), len(counts), bounds(counts), R.matrix_memory_copies(vd), R.recurrence_state_pitch(d)
    q, k, v = (torch.randn((T, H * n), generator=g) for n in (d, d, vd))
    # n . q of either sign, but well away from zero: a denominator that cancels would make any rounding large
    q, k, v = (q.abs() * torch.randn((T, 1), generator=g).sign()).to(dtype), k.abs().to(dtype), v.to(dtype)
    both = torch.randn((T, 2 * H + 6), generator=g)
    both[:, :H] = 3 * both[:, :H] + gates_at[0]
    both[:, H:2 * H] = 3 * both[:, H:2 * H] + gates_at[1]
    both = both.to(dtype)
    bi, bf = torch.randn(H, generator=g), torch.randn(H, generator=g)
    S0, n0, m0 = torch.randn((B, H, d, vd), generator=g), 3 * torch.randn((B, H, d), generator=g).abs(), torch.randn((B, H), generator=g)
    slots = list(range(B, 0, -1)) if slots is None else slots
    state, top = torch.full((B + 2, H, vd + copies, pitch), float("nan")), torch.full((B + 2, H, copies), float("nan"))
    for b in range(B):
        if starts[b] and slots[b] >= 0:
            state[slots[b], :, :, d:] = 0
            state[slots[b], :, :vd, :d] = S0[b].transpose(1, 2)
            state[slots[b], :, vd:, :d] = n0[b][:, None]
            top[slots[b]] = m0[b][:, None]
    state, top, out = state.to(gpu), top.to(gpu), torch.full((T, H * vd), float("nan"), dtype=dtype, device=gpu)
    on = both.to(gpu)
    gates = R.MemoryGates(on[:, :H], on[:, H:2 * H], bi.to(gpu), bf.to(gpu), cap, top, d ** -0.5)
    args = [q.to(gpu), k.to(gpu), v.to(gpu), out, state, i32(slots, gpu), i32(starts, gpu), H, H, d, vd]
    options = dict(gates=gates, cu_seqlens=i32(cu, gpu))
    if which == "chunks":
        segs, ends = R.recurrence_segments(counts, H, H, vd, wanted)
        op("decayed_chunks")(*args, i32(segs, gpu), i32(ends, gpu), **options)
    else:
        if max(counts) == 1:
            del options["cu_seqlens"]
        op("decayed_recurrence")(*args, **options)
    worst = [0.0] * 4
    for b in range(B):
        if slots[b] < 0:
            continue
        f = lambda x: x[cu[b]:cu[b + 1]].to(D).view(counts[b], H, -1)      # noqa: E731
        i, fg = O.log_gates(both[cu[b]:cu[b + 1], :H].to(D) + bi.to(D), both[cu[b]:cu[b + 1], H:2 * H].to(D) + bf.to(D), cap)
        o, (S, n, m) = O.matrix_memory(f(q) * d ** -0.5, f(k), f(v), i, fg, (S0[b].to(D), n0[b].to(D), m0[b].to(D)) if starts[b] else None)
        s = state[slots[b]]
        worst[0] = max(worst[0], rel(out[cu[b]:cu[b + 1]].view(counts[b], H, vd), o))
        worst[1] = max(worst[1], rel(s[:, :vd, :d].transpose(1, 2), S))
        worst[2] = max(worst[2], *(rel(s[:, vd + c, :d], n) for c in range(copies)))
        worst[3] = max(worst[3], (top[slots[b]].double().cpu() - m[:, None]).abs().max().item())
    return worst


MEMORY_SIZES = [(6, 32, 48), (2, 64, 64), (1, 128, 128), (3, 20, 20), (2, 33, 70), (1, 256, 200), (2, 16, 8), (1, 48, 130), (1, 8, 1)]
GATES = [(15.0, (0.0, 2.0)), (15.0, (-14.0, 14.0)), (3.0, (10.0, -10.0)), (40.0, (30.0, 0.0)), (15.0, (-9.0, -3.0))]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,d,vd", MEMORY_SIZES + [(1, 300, 24)])
def test_matrix_memory_token_by_token(gpu, dtype, H, d, vd):
    for cap, at in GATES:
        o, S, n, m = run_memory(gpu, "plain", dtype, H, d, vd, [1] * 7, [0, 4, 1, 9, 0, 7, 2], cap, at, slots=[3, 1, -1, 0, 2, 8, 5])
        assert o < limit(dtype, 4e-6, 4e-3) and S < 4e-6 and n < 4e-6 and m < 1e-5, (cap, at)
        o, S, n, m = run_memory(gpu, "plain", dtype, H, d, vd, [40, 2, 19], [0, 4, 1], cap, at)
        assert o < limit(dtype, 3e-5, 4e-3) and S < 2e-5 and n < 2e-5 and m < 1e-5, (cap, at)


@pytest.mark.parametrize("H,d,vd", MEMORY_SIZES)
def test_matrix_memory_in_chunks(gpu, H, d, vd):
    """Portions shorter and longer than chunks, and some that are cut into segments; gates that forget nothing and all, that take in
    nothing and all; denominators from the normalizer and from the running maximum."""
    for seed, (cap, at) in enumerate(GATES):
        for counts, starts in (([2, 37, 64, 1, 100], [0, 5, 3, 2, 0]), ([65], [4]), ([600, 33], [0, 7])):
            o, S, n, m = run_memory(gpu, "chunks", torch.bfloat16, H, d, vd, counts, starts, cap, at, seed=seed)
            assert o < 6e-3 and S < 1e-4 and n < 1e-4 and m < 1e-4, (cap, at, counts, o, S, n, m)


def test_memory_chunks_leave_padding_slots_alone(gpu):
    o, S, n, m = run_memory(gpu, "chunks", torch.bfloat16, 2, 64, 64, [20, 20, 20], [0, 3, 1], 15.0, (0.0, 2.0), slots=[2, -1, 0])
    assert o < 6e-3 and S < 1e-4 and n < 1e-4 and m < 1e-4
