"""GPU: the operators behind recurrent layers, latent attention and the float32 residual stream, each alone against the plain
float64 restatement in oracle/nepulix.py."""
import math

import pytest
import torch

from nano_vllm_ninetoothed_amd import mops
from nano_vllm_ninetoothed_amd.mops.hip import recurrent_ops as R
from oracle import nepulix as O

pytestmark = pytest.mark.gpu
DTYPES = [torch.float32, torch.bfloat16]
TOL = {torch.float32: 3e-6, torch.bfloat16: 8e-3}     # of the largest magnitude in the result


def op(name):
    return mops.get_op(name, "hip")


def rnd(g, *shape, dtype=torch.float32, std=1.0):
    """Random values that are exact in bfloat16."""
    return (torch.randn(shape, generator=g) * std).bfloat16().to(dtype)


def close(got, want, dtype, what="", factor=1.0):
    got, want = got.double().cpu(), want.double()
    assert torch.isfinite(got).all(), f"{what}: not finite"
    err = (got - want).abs().max().item() / max(want.abs().max().item(), 1e-9)
    assert err <= factor * TOL[dtype], f"{what}: {err:.3g} > {factor * TOL[dtype]:.3g}"


# ------------------------------------------------------------------------------------------------ norms, embedding, glu
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("n", [8, 77, 320, 1024, 1032, 5000])
def test_residual_norms(gpu, dtype, n):
    g = torch.Generator().manual_seed(n)
    x, y, w = torch.randn((5, n), generator=g), rnd(g, 5, n, dtype=dtype), rnd(g, n, dtype=dtype, std=0.3)
    y[3] *= 1e-3            # eps matters here
    for off in (0.0, 1.0):
        want = x.double() + O.rms(y.double(), 1e-5) * (off + w.double())
        res = x.to(gpu)
        act = op("norm_residual_add")(res, y.to(gpu), w.to(gpu), 1e-5, off)
        close(res, want, torch.float32, "residual")
        close(act, want, dtype, "activation copy")
        close(op("rms_norm_f32")(x.to(gpu), w.to(gpu), 1e-5, off), O.rms(x.double(), 1e-5) * (off + w.double()), dtype, "norm")
    # a strided y
    wide = torch.zeros((5, n + 24), dtype=dtype)
    wide[:, 8:8 + n] = y
    res = x.to(gpu)
    op("norm_residual_add")(res, wide.to(gpu)[:, 8:8 + n], w.to(gpu), 1e-5, 1.0)
    close(res, x.double() + O.norm_unit_offset(y.double(), w.double(), 1e-5), torch.float32, "strided")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("width", [33, 128])
def test_embed_residual(gpu, dtype, width):
    g = torch.Generator().manual_seed(3)
    table, ids = rnd(g, 50, width, dtype=dtype), torch.tensor([0, 49, 7, 7, 50, -1])
    res, act = op("embed_residual")(ids.to(gpu), table.to(gpu))
    want = torch.zeros(6, width)
    want[:4] = table[ids[:4]].float()
    assert torch.equal(res.cpu(), want) and torch.equal(act.cpu().float(), want)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("groups,size", [(1, 17), (3, 40), (8, 64), (2, 2504)])
def test_gated_group_norm(gpu, dtype, groups, size):
    g = torch.Generator().manual_seed(size)
    n = groups * size
    y, both, w = rnd(g, 9, n, dtype=dtype), rnd(g, 9, 2 * n, dtype=dtype), rnd(g, n, dtype=dtype)
    y[:, :size] *= 50       # groups differ in scale
    gate = both[:, n:]
    yd, gd = y.double(), gate.double()
    got = op("gated_group_norm")(y.to(gpu), both.to(gpu)[:, n:], groups, 1e-6)
    close(got, O.group_rms(yd, groups, 1e-6) * O.silu(gd), dtype, "norm first")
    got = op("gated_group_norm")(y.to(gpu), both.to(gpu)[:, n:], groups, 1e-6, weight=w.to(gpu), gate_first=True)
    close(got, O.group_rms(yd * O.silu(gd), groups, 1e-6) * w.double(), dtype, "gate first")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("n", [13, 96])
def test_clamped_glu(gpu, dtype, n):
    g = torch.Generator().manual_seed(n)
    p = rnd(g, 11, 2 * n, dtype=dtype, std=3.0)
    for limit in (0.5, 1.0, 7.0):
        gt, up = p[:, :n].double().clamp(max=limit), p[:, n:].double().clamp(-limit, limit)
        close(op("clamped_glu")(p.to(gpu)[:, :n], p.to(gpu)[:, n:], limit), gt / (1 + torch.exp(-1.702 * gt)) * (up + 1), dtype, f"limit {limit}")


# ------------------------------------------------------------------------------------------------ recurrences
def recurrence_case(g, heads, groups, d, vd, T, dtype, kind, rot):
    q, k = rnd(g, T, groups * d, dtype=dtype), rnd(g, T, groups * d, dtype=dtype)
    v = rnd(g, T, heads * vd, dtype=dtype)
    case = dict(q=q, k=k, v=v, k_scale=d ** -0.5)
    if kind == "const":
        decay = torch.tensor([1.0 - 0.5 ** (1 + 1.7 * i) if i else 1.0 for i in range(heads)], dtype=torch.float64)
        case.update(decay=decay.float(), log_decay=decay.log().float())
        a, s, skip = decay.float().double()[None].expand(T, heads), torch.ones(T, heads, dtype=torch.float64), torch.zeros(heads)
    else:
        dt = rnd(g, T, heads, dtype=dtype, std=2.0)
        dt[T // 2] = 25.0                     # a step that wipes the state of fast heads out
        bias, neg_a, skip = torch.randn(heads, generator=g) - 1, -torch.exp(torch.randn(heads, generator=g)), torch.randn(heads, generator=g)
        case.update(dt=dt, dt_bias=bias, neg_a=neg_a, skip=skip)
        s = O.softplus(dt.double() + bias.double())
        a = torch.exp(neg_a.double() * s)
    qd, kd, vdd = q.double().view(T, groups, d), k.double().view(T, groups, d), v.double().view(T, heads, vd)
    if rot:
        pos = torch.arange(T)
        qd, kd = O.rotate_half(qd, pos, 7e3, rot), O.rotate_half(kd, pos, 7e3, rot)
        from nano_vllm_ninetoothed_amd.layers import Rotary
        case["cos_sin"] = Rotary(T + 5, "cpu").table(7e3, rot)
    rep = heads // groups
    o, S = O.decayed_recurrence(qd.repeat_interleave(rep, 1), (kd * d ** -0.5).repeat_interleave(rep, 1), vdd * s[..., None], a)
    o = o + skip.double()[None, :, None] * vdd
    return case, o.reshape(T, -1), S


def run_recurrence(gpu, case, heads, groups, d, vd, cuts, chunked, segment=None, slots=3, slot=1):
    """Runs the tokens in portions ending at `cuts`; returns (out, state [H, d, vd])."""
    T = case["q"].shape[0]
    c = {k: (t.to(gpu) if isinstance(t, torch.Tensor) else t) for k, t in case.items()}
    state = torch.full((slots, heads, vd, R.recurrence_state_pitch(d)), 1e4, device=gpu)      # what another sequence left
    out = torch.full((T, heads * vd), float("nan"), dtype=c["v"].dtype, device=gpu)
    i32 = lambda x: torch.tensor(x, dtype=torch.int32, device=gpu)   # noqa: E731
    at = 0
    opts = {k: c[k] for k in ("decay", "log_decay", "dt_bias", "neg_a", "skip", "cos_sin", "k_scale") if k in c}
    for end in cuts:
        n = end - at
        if "dt" in c:
            opts["dt"] = c["dt"][at:end]
        args = (c["q"][at:end], c["k"][at:end], c["v"][at:end], out[at:end], state, i32([slot]), i32([at]), heads, groups, d, vd)
        if n == 1 and not chunked:
            op("decayed_recurrence")(*args, **opts)
        elif chunked:
            seg = [(0, b, min(n, b + (segment or n))) for b in range(0, n, segment or n)]
            op("decayed_chunks")(*args, i32(seg), i32([0, len(seg)]), cu_seqlens=i32([0, n]), **opts)
        else:
            op("decayed_recurrence")(*args, cu_seqlens=i32([0, n]), **opts)
        at = end
    assert at == T
    assert float(state[0].min()) == 1e4 and float(state[2].max()) == 1e4, "another slot was written"
    return out, state[slot, :, :, :d].transpose(1, 2)


SIZES = [(1, 1, 16, 16), (4, 2, 24, 40), (3, 3, 42, 25), (2, 1, 64, 64), (2, 2, 128, 130), (2, 1, 200, 32), (8, 2, 32, 24), (4, 1, 48, 27), (2, 2, 256, 300)]


@pytest.mark.parametrize("kind", ["const", "steps"])
@pytest.mark.parametrize("sizes", SIZES)
@pytest.mark.parametrize("dtype", DTYPES)
def test_recurrence_token_by_token_form(gpu, dtype, sizes, kind):
    heads, groups, d, vd = sizes
    rot = 0 if kind == "steps" else (d // 2 - d // 2 % 2 if d > 24 else d)
    case, want, S = recurrence_case(torch.Generator().manual_seed(d), heads, groups, d, vd, 37, dtype, kind, rot)
    for cuts in ([37], [2, 5, 36, 37], list(range(1, 38))):
        out, state = run_recurrence(gpu, case, heads, groups, d, vd, cuts, False)
        close(out, want, dtype, f"out {cuts[:3]}", 4)
        close(state, S, torch.float32, f"state {cuts[:3]}", 4)


@pytest.mark.parametrize("kind", ["const", "steps"])
@pytest.mark.parametrize("sizes", SIZES)
def test_recurrence_in_chunks(gpu, sizes, kind):
    heads, groups, d, vd = sizes
    rot = 0 if kind == "steps" else (d if d % 16 == 0 else d // 2 - d // 2 % 2)
    T = 333
    case, want, S = recurrence_case(torch.Generator().manual_seed(d + 1), heads, groups, d, vd, T, torch.bfloat16, kind, rot)
    scale = want.abs().max()
    for cuts, segment in (([T], None), ([T], 64), ([T], 128), ([2, 64, 65, 128, 131, T], None), ([63, 200, T], 64)):
        out, state = run_recurrence(gpu, case, heads, groups, d, vd, cuts, True, segment)
        err = (out.double().cpu() - want).abs().max() / scale
        assert err < 1e-2, f"{cuts} {segment}: {err}"
        # k and q are rounded to bf16 after rotation and scaling, nothing else of the state is
        serr = (state.double().cpu() - S).norm() / S.norm()
        assert serr < (4e-3 if rot or kind == "const" else 3e-3), f"state {cuts} {segment}: {serr}"


def test_chunked_state_keeps_more_than_sixteen_bits(gpu):
    """Values that only a 32-bit state carries: a large constant part and small increments, over many chunks without decay."""
    T, d, vd = 640, 32, 32
    k = torch.zeros(T, d)
    k[:, 0] = 1.0
    v = torch.full((T, vd), 1.0)
    v[0] = 1024.0
    q = torch.zeros(T, d)
    q[:, 0] = 1.0
    case = dict(q=q.bfloat16(), k=k.bfloat16(), v=v.bfloat16(), k_scale=1.0, decay=torch.ones(1), log_decay=torch.zeros(1))
    for segment in (None, 128):
        _, state = run_recurrence(gpu, case, 1, 1, d, vd, [T], True, segment)
        assert torch.equal(state[0, 0].cpu(), torch.full((vd,), 1024.0 + T - 1))


def test_chunks_of_several_sequences_and_padding_slots(gpu):
    """Unequal portions in one launch, each against itself alone; a slot of -1 is left out."""
    g = torch.Generator().manual_seed(8)
    heads, d, vd = 2, 48, 72
    lens, starts = [130, 2, 77, 64], [0, 5, 0, 64]
    cu = [0]
    for n in lens:
        cu.append(cu[-1] + n)
    q, k, v = (rnd(g, cu[-1], heads * x, dtype=torch.bfloat16).to(gpu) for x in (d, d, vd))
    decay = torch.tensor([0.99, 0.8], dtype=torch.float64)
    opts = dict(decay=decay.float().to(gpu), log_decay=decay.log().float().to(gpu), k_scale=d ** -0.5)
    i32 = lambda x: torch.tensor(x, dtype=torch.int32, device=gpu)   # noqa: E731
    init = torch.randn((6, heads, vd, R.recurrence_state_pitch(d)), generator=g).to(gpu)
    slots = [4, 0, -1, 2]
    segs, bounds = R.recurrence_segments(lens, heads, heads, vd)
    for cut in (1, 64):
        state, out = init.clone(), torch.zeros((cu[-1], heads * vd), dtype=torch.bfloat16, device=gpu)
        if cut == 64:
            segs, bounds = [], [0]
            for i, n in enumerate(lens):
                segs += [(i, cu[i] + b, cu[i] + min(n, b + 64)) for b in range(0, n, 64)]
                bounds.append(len(segs))
        op("decayed_chunks")(q, k, v, out, state, i32(slots), i32(starts), heads, heads, d, vd, i32(segs), i32(bounds), cu_seqlens=i32(cu), **opts)
        for i, n in enumerate(lens):
            if slots[i] < 0:
                continue
            s1, o1 = init.clone(), torch.zeros((n, heads * vd), dtype=torch.bfloat16, device=gpu)
            sl = slice(cu[i], cu[i + 1])
            op("decayed_recurrence")(q[sl], k[sl], v[sl], o1, s1, i32([slots[i]]), i32([starts[i]]), heads, heads, d, vd, cu_seqlens=i32([0, n]), **opts)
            close(out[sl], o1.double().cpu(), torch.bfloat16, f"sequence {i}", 2)
            assert ((state[slots[i]] - s1[slots[i]]).norm() / s1[slots[i]].norm()) < 4e-3
        for s in (1, 3, 5):
            assert torch.equal(state[s], init[s])


def test_segments_cover_every_portion():
    for counts in ([5000], [64], [2, 3, 700], [100] * 40, [16384, 1000]):
        segs, bounds = R.recurrence_segments(counts, 4, 2, 64)
        at = 0
        for i, n in enumerate(counts):
            mine = segs[bounds[i]:bounds[i + 1]]
            assert mine[0][1] == at and mine[-1][2] == at + n and all(s[0] == i for s in mine)
            assert all(a[2] == b[1] and (a[2] - a[1]) % 64 == 0 for a, b in zip(mine, mine[1:]))
            at += n


# ------------------------------------------------------------------------------------------------ short convolution
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("channels,taps", [(40, 4), (37, 3), (24, 1), (16, 7)])
def test_short_conv_in_portions(gpu, dtype, channels, taps):
    g = torch.Generator().manual_seed(taps)
    T = 41
    x, w, b = rnd(g, T, channels + 8, dtype=dtype), torch.randn((channels, taps), generator=g), torch.randn(channels, generator=g)
    want = O.silu(O.causal_conv(x[:, 8:].double(), w.double(), b.double()))
    wt, xg = w.t().contiguous().to(gpu), x.to(gpu)[:, 8:]
    i32 = lambda t: torch.tensor(t, dtype=torch.int32, device=gpu)   # noqa: E731
    for cuts in ([T], [2, 4, 7, 30, 31, T], list(range(1, T + 1))):
        ring = torch.full((2, taps, channels), 99.0, dtype=dtype, device=gpu)
        at = 0
        for end in cuts:
            n = end - at
            meta = (i32([0, n]), i32([at]), i32([1]))
            got = op("short_conv")(xg[at:end], wt, b.to(gpu), ring, i32([0] * n), *meta)
            close(got, want[at:end], dtype, f"{cuts[:2]} at {at}", 2)
            op("short_conv_update")(xg[at:end], ring, *meta)
            at = end
        assert float(ring[0].min()) == 99.0


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("taps", [2, 3, 4, 5])
def test_short_conv_of_many_tokens(gpu, dtype, taps):
    """Unequal portions packed into one long launch, some behind earlier tokens."""
    g = torch.Generator().manual_seed(taps + 40)
    channels, lens, before = 48, [100, 1, 2, 3, 17, 260], [0, 7, 1, 2, 0, 31]
    w, b = torch.randn((channels, taps), generator=g), torch.randn(channels, generator=g)
    i32 = lambda t: torch.tensor(t, dtype=torch.int32, device=gpu)   # noqa: E731
    ring = torch.full((7, taps, channels), 99.0, dtype=dtype, device=gpu)
    slots, cu, xs, wants = [3, 6, 0, 5, 1, 2], [0], [], []
    for n, p, s in zip(lens, before, slots):
        full = rnd(g, p + n, channels, dtype=dtype)
        wants.append(O.silu(O.causal_conv(full.double(), w.double(), b.double()))[p:])
        op("short_conv_update")(full[:p].to(gpu), ring, i32([0, p]), i32([0]), i32([s])) if p else None
        xs.append(full[p:])
        cu.append(cu[-1] + n)
    seqs = [i for i, n in enumerate(lens) for _ in range(n)]
    got = op("short_conv")(torch.cat(xs).to(gpu), w.t().contiguous().to(gpu), b.to(gpu), ring, i32(seqs), i32(cu), i32(before), i32(slots))
    close(got, torch.cat(wants), dtype, f"{taps} taps", 2)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("sizes", [(4, 2, 16, 24, 4), (6, 3, 20, 70, 3), (2, 1, 128, 64, 1)])
def test_decode_step_with_the_convolution_inside(gpu, dtype, sizes):
    """One launch per token against convolution, then recurrence, in float64; two sequences at different positions."""
    heads, groups, n, vd, taps = sizes
    g = torch.Generator().manual_seed(vd)
    inner, gn = heads * vd, groups * n
    ch, T = inner + 2 * gn, 19
    w, b = torch.randn((ch, taps), generator=g) * 0.5, torch.randn(ch, generator=g) * 0.3
    bias, neg_a, skip = torch.randn(heads, generator=g), -torch.exp(torch.randn(heads, generator=g)), torch.randn(heads, generator=g)
    xs = [rnd(g, T, ch + heads, dtype=dtype) for _ in range(2)]
    wants = []
    for x in xs:
        c = O.silu(O.causal_conv(x[:, :ch].double(), w.double(), b.double()))
        v, B, C = c[:, :inner].reshape(T, heads, vd), c[:, inner:inner + gn].reshape(T, groups, n), c[:, inner + gn:].reshape(T, groups, n)
        s = O.softplus(x[:, ch:].double() + bias.double())
        rep = heads // groups
        o, _ = O.decayed_recurrence(C.repeat_interleave(rep, 1), B.repeat_interleave(rep, 1), v * s[..., None], torch.exp(neg_a.double() * s))
        wants.append((o + skip.double()[None, :, None] * v).reshape(T, inner))
    f = lambda t: t.float().contiguous().to(gpu)   # noqa: E731
    i32 = lambda t: torch.tensor(t, dtype=torch.int32, device=gpu)   # noqa: E731
    ring = torch.full((3, taps, ch), 7.0, dtype=dtype, device=gpu)
    state = torch.full((3, heads, vd, R.recurrence_state_pitch(n)), 50.0, device=gpu)
    conv = (f(w.t()), f(b), ring, (inner + gn, inner, 0))
    got = [[], []]
    for step in range(T + 3):                       # the second sequence starts three steps later
        live = [i for i in (0, 1) if 0 <= step - 3 * i < T]
        pos = [step - 3 * i for i in live]
        x = torch.stack([xs[i][p] for i, p in zip(live, pos)] + [xs[0][0]]).to(gpu)        # and a padding row
        out = torch.empty((len(live) + 1, inner), dtype=dtype, device=gpu)
        op("decayed_recurrence")(x[:, inner + gn:ch], x[:, inner:inner + gn], x[:, :inner], out, state, i32([2 * i for i in live] + [-1]), i32(pos + [0]),
                                 heads, groups, n, vd, dt=x[:, ch:], dt_bias=f(bias), neg_a=f(neg_a), skip=f(skip), conv=conv)
        assert float(out[-1].abs().max()) == 0.0
        for j, i in enumerate(live):
            got[i].append(out[j].cpu())
    for i in (0, 1):
        close(torch.stack(got[i]), wants[i], dtype, f"sequence {i}", 4)
    assert float(ring[1].min()) == 7.0 and float(state[1].min()) == 50.0


# ------------------------------------------------------------------------------------------------ latent attention
LATENT = [(1, 8, 2, 8, 16), (5, 22, 6, 37, 44), (16, 64, 32, 64, 128), (18, 128, 64, 128, 512), (3, 40, 24, 144, 200)]    # heads, dim, rot, vdim, kv_rank


def latent_case(gpu, sizes, lens, dtype, bs, seed, spikes=()):
    """Random caches for sequences of `lens` tokens in shuffled pages; spikes: (sequence, key position) whose latent is scaled
    up so that one score stands out."""
    heads, dim, rot, vdim, kr = sizes
    g = torch.Generator().manual_seed(seed)
    from nano_vllm_ninetoothed_amd.layers import Rotary
    need = [(n + bs - 1) // bs for n in lens]
    perm = torch.randperm(sum(need) + 2, generator=g).tolist()
    table = torch.full((len(lens), max(max(need), 1) + 1), -1, dtype=torch.int32)
    pitch = (kr + rot + 7) // 8 * 8
    cache = torch.full((sum(need) + 2, bs, pitch), 1e4, dtype=dtype)       # what others left in the pages
    cs, ks = [], []
    for s, n in enumerate(lens):
        c, k = rnd(g, n, kr, std=0.5), rnd(g, n, rot)
        for ss, p in spikes:
            if ss == s and p < n:
                c[p] = (c[p] * 6).bfloat16().float()
        for i in range(need[s]):
            table[s, i] = perm.pop()
            rows = slice(i * bs, min(n, (i + 1) * bs))
            m = rows.stop - rows.start
            cache[table[s, i], :m, :kr], cache[table[s, i], :m, kr:kr + rot] = c[rows].to(dtype), k[rows].to(dtype)
            cache[table[s, i], :m, kr + rot:] = 0
        cs.append(c.double())
        ks.append(k.double())
    cos_sin = Rotary(max(lens) + 3, "cpu").table(3e3, rot)
    return g, cache.to(gpu), table.to(gpu), cs, ks, cos_sin.to(gpu)


def rows_reference(ql, qr, pos, c, kr, scale):
    """One query row in float64: latent attention in the latent space."""
    n = pos + 1
    qr = O.rotate_interleaved(qr[None], torch.tensor([pos]), 3e3, qr.shape[-1])[0]
    s = (ql @ c[:n].T + qr @ kr[:n].T) * scale
    p = torch.exp(s - s.max(dim=-1, keepdim=True).values)
    return (p / p.sum(dim=-1, keepdim=True)) @ c[:n]


@pytest.mark.parametrize("form", ["plain f32", "plain bf16", "matrix"])
@pytest.mark.parametrize("sizes", LATENT)
def test_latent_rows(gpu, sizes, form):
    heads, dim, rot, vdim, kr = sizes
    dtype = torch.float32 if form == "plain f32" else torch.bfloat16
    run = op("latent_decode" if form == "matrix" else "latent_attention_rows")
    for bs in (32, 256):
        lens = [1, 31, 32, 33, 64, 65, 300, 257]
        spikes = [(2, 31), (3, 32), (4, 0), (5, 64), (6, 0), (7, 255), (6, 256)]
        g, cache, table, cs, ks, cos_sin = latent_case(gpu, sizes, lens, dtype, bs, 5, spikes)
        rows = [(s, n - 1) for s, n in enumerate(lens)] + [(6, 299), (6, 256), (6, 255), (6, 31), (6, 0), (5, 63)]
        ql, q = rnd(g, len(rows) + 1, heads, kr, std=0.7), rnd(g, len(rows) + 1, heads, dim + rot)
        scale = (dim + rot) ** -0.5
        i32 = lambda t: torch.tensor(t, dtype=torch.int32, device=gpu)   # noqa: E731
        got = run(ql.to(dtype).to(gpu), q.to(dtype).to(gpu)[..., dim:], cache, cos_sin, i32([p + 1 for _, p in rows] + [0]), table, scale,
                  i32([s for s, _ in rows] + [0]))
        assert float(got[-1].abs().max()) == 0.0
        for i, (s, p) in enumerate(rows):
            close(got[i], rows_reference(ql[i].double(), q[i, :, dim:].double(), p, cs[s], ks[s], scale), dtype, f"{form} bs {bs} row {i}", 3)
        # without a row -> sequence map
        got2 = run(ql[:8].to(dtype).to(gpu), q[:8].to(dtype).to(gpu)[..., dim:], cache, cos_sin, i32(lens), table, scale)
        assert torch.equal(got2, got[:8]) or (got2.float() - got[:8].float()).abs().max() < 2e-2


@pytest.mark.parametrize("n_rows,ctx", [(1, 5000), (2, 2049), (600, 100)])
def test_latent_decode_in_runs(gpu, n_rows, ctx):
    """Contexts that are split over workgroups; a spike at the first and last key of runs decides the result."""
    sizes = (4, 32, 16, 32, 64)
    heads, dim, rot, _, kr = sizes
    spikes = [(0, p) for p in (0, 63, 64, 1023, 1024, ctx - 1)]
    g, cache, table, cs, ks, cos_sin = latent_case(gpu, sizes, [ctx], torch.bfloat16, 64, 6, spikes)
    ql, q = rnd(g, n_rows, heads, kr), rnd(g, n_rows, heads, dim + rot)
    i32 = lambda t: torch.tensor(t, dtype=torch.int32, device=gpu)   # noqa: E731
    pos = [max(0, ctx - 1 - 7 * i) if n_rows < 10 else i % ctx for i in range(n_rows)]
    got = op("latent_decode")(ql.bfloat16().to(gpu), q.bfloat16().to(gpu)[..., dim:], cache, cos_sin, i32([p + 1 for p in pos]), table, 0.2, i32([0] * n_rows))
    for i in range(0, n_rows, max(1, n_rows // 20)):
        close(got[i], rows_reference(ql[i].double(), q[i, :, dim:].double(), pos[i], cs[0], ks[0], 0.2), torch.bfloat16, f"row {i}", 2)


@pytest.mark.parametrize("sizes", LATENT)
def test_latent_prefill(gpu, sizes):
    """Portions behind cached tokens against dense attention; spikes at tile, page and portion borders."""
    heads, dim, rot, vdim, kr = sizes
    counts, starts = [130, 64, 200, 1], [0, 63, 129, 0]
    lens = [s + n for s, n in zip(starts, counts)]
    spikes = [(0, 0), (0, 63), (0, 64), (0, 129), (1, 62), (1, 126), (2, 128), (2, 0), (2, 255)]
    g, cache, table, cs, ks, cos_sin = latent_case(gpu, sizes, lens, torch.bfloat16, 64, 9, spikes)
    T = 3 + sum(counts)                              # three rows of other sequences in front
    q = rnd(g, T, heads, dim + rot, std=1.5)
    uk, uv = rnd(g, heads * dim, kr, std=kr ** -0.5 * 2), rnd(g, heads * vdim, kr, std=kr ** -0.5 * 2)
    row_seq, row_pos, tiles = R.latent_prefill_plan(counts, starts, 3, 0)
    i32 = lambda t: torch.tensor(t, dtype=torch.int32, device=gpu)   # noqa: E731
    c, kpart = op("latent_gather")(cache, table, i32(row_seq), i32(row_pos), kr, rot)
    pad, dp, rp = -kr % 8, (dim + 7) // 8 * 8, (rot + 7) // 8 * 8
    assert c.shape[1] == kr + pad and kpart.shape[1] == rp and float(kpart[:, rot:].abs().sum()) == 0.0
    lin = op("linear")
    F = torch.nn.functional
    k = lin(c, F.pad(uk.view(heads, dim, kr), (0, pad, 0, dp - dim)).reshape(heads * dp, -1).bfloat16().to(gpu))
    vt = lin(F.pad(uv.bfloat16().to(gpu), (0, pad)).contiguous(), c)
    out = torch.full((T, heads, vdim), 3.0, dtype=torch.bfloat16, device=gpu)
    scale = (dim + rot) ** -0.5
    qp = torch.cat((F.pad(q[..., :dim], (0, dp - dim)), F.pad(q[..., dim:], (0, rp - rot))), -1).bfloat16().to(gpu)
    positions = i32([0, 0, 0] + [p for n, st in zip(counts, starts) for p in range(st, st + n)])
    op("rotate_pairs")(qp[3:, :, dp:dp + rot], positions[3:], cos_sin)
    assert torch.equal(qp[:3, :, dp:dp + rot].cpu(), q[:3, :, dim:].bfloat16())
    op("latent_prefill")(qp, k, kpart, vt, i32(tiles), scale, out)
    assert float(out[:3].float().min()) == 3.0
    at = 3
    for s, (n, start) in enumerate(zip(counts, starts)):
        qq = q[at:at + n].double()
        qr = O.rotate_interleaved(qq[..., dim:], torch.arange(start, start + n), 3e3, rot)
        ku, vv = (cs[s] @ uk.double().T).view(-1, heads, dim), (cs[s] @ uv.double().T).view(-1, heads, vdim)
        sc = (torch.einsum("ihd,jhd->hij", qq[..., :dim], ku) + torch.einsum("ihd,jd->hij", qr, ks[s])) * scale
        mask = torch.arange(lens[s])[None, :] > torch.arange(start, start + n)[:, None]
        p = torch.softmax(sc.masked_fill(mask, -math.inf), dim=-1)
        close(out[at:at + n], torch.einsum("hij,jhd->ihd", p, vv), torch.bfloat16, f"sequence {s}", 4)
        at += n


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("sizes", [(16, 24, 8, 24), (51, 44, 6, 7), (192, 512, 64, 3)])      # q_rank, kv_rank, rot, tokens
def test_latent_prepare(gpu, dtype, sizes):
    qr, kr, rot, T = sizes
    from nano_vllm_ninetoothed_amd.layers import Rotary
    g = torch.Generator().manual_seed(qr)
    down, wq, wk = rnd(g, T, qr + kr + rot + 3, dtype=dtype), rnd(g, qr, dtype=dtype), rnd(g, kr, dtype=dtype)
    pitch = (kr + rot + 7) // 8 * 8
    cache = torch.full((3, 32, pitch), 5.0, dtype=dtype, device=gpu)
    slots = torch.randperm(96, generator=g)[:T].to(torch.int32)
    slots[1] = -1
    pos = torch.randint(0, 2000, (T,), generator=g).to(torch.int32)
    cq = op("latent_prepare")(down.to(gpu), wq.to(gpu), wk.to(gpu), 1e-5, Rotary(2000, gpu).table(1e4, rot), pos.to(gpu), slots.to(gpu), cache, qr, kr, rot)
    d = down.double()
    close(cq, O.rms(d[:, :qr], 1e-5) * wq.double(), dtype, "query latent")
    c = O.rms(d[:, qr:qr + kr], 1e-5) * wk.double()
    k = O.rotate_interleaved(d[:, None, qr + kr:qr + kr + rot], pos.long(), 1e4, rot)[:, 0]
    rows = cache.view(96, pitch).cpu().double()
    keep = slots >= 0
    close(rows[slots[keep].long(), :kr], c[keep], dtype, "latent row")
    close(rows[slots[keep].long(), kr:kr + rot], k[keep], dtype, "key part", 2)
    assert float(rows[slots[keep].long(), kr + rot:].abs().sum()) == 0.0
    untouched = torch.ones(96, dtype=torch.bool)
    untouched[slots[keep].long()] = False
    assert float(rows[untouched].min()) == 5.0


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("sizes", [(1, 1, 8, 8), (70, 5, 22, 44), (130, 3, 64, 130), (16, 2, 512, 128)])
def test_head_linear(gpu, dtype, sizes):
    t, h, k, n = sizes
    g = torch.Generator().manual_seed(k)
    x, w = rnd(g, t, h, k + 6, dtype=dtype), rnd(g, h, n, k, dtype=dtype, std=k ** -0.5)
    got = op("head_linear")(x.to(gpu)[..., :k], w.to(gpu))
    close(got, torch.einsum("thk,hnk->thn", x[..., :k].double(), w.double()), dtype, "head linear", 2)
