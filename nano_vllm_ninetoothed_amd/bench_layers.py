"""Measurements behind `bench.py --op nepulix`, `--op sozarax`, `--op lulizen` and `--op fedovik`: prefill and decode throughput of models with layers
of real sizes beside models of equal width, depth, feed-forward and vocabulary (Qwen3 and the designs that came before), and every
kernel of the design beside the like kernel of those.  Random weights and inputs."""
from __future__ import annotations

import torch

HBM = 8000.0       # GB/s
MFMA = 2500.0      # TFLOP/s, dense bf16


def nepulix_dict(width, layers, ff, vocab, ret, mam, lat):
    kinds = ["retention", "mamba2", "latent_attention"]
    sizes = {"retention": ret, "mamba2": mam, "latent_attention": lat}
    return {"architecture": "Nepulix", "width": width, "vocab": vocab, "norm": {"eps": 1e-6},
            "layers": [{"type": kinds[i % 3], "mixer": sizes[kinds[i % 3]], "mlp": {"kind": "dense", "ff": ff, "limit": 7.0}} for i in range(layers)]}


def _retention(heads, dim, vdim):
    return {"heads": heads, "dim": dim, "vdim": vdim, "decay": [1 - 2.0 ** (-5 - i % 8) for i in range(heads)], "rot": {"base": 1e4, "dims": dim}}


def _latent(heads, q_rank):
    return {"heads": heads, "dim": 128, "rot_dim": 64, "vdim": 128, "q_rank": q_rank, "kv_rank": 512, "scale": 192 ** -0.5, "rot": {"base": 1e4, "dims": 64}}


def sizes():
    """name -> (Nepulix config.json dict, Qwen3Shape of equal size)"""
    from .models.qwen3 import Qwen3Shape
    return {
        "w1024": (nepulix_dict(1024, 12, 3072, 32768, _retention(8, 128, 128),
                               {"heads": 32, "vdim": 64, "state": 128, "groups": 1, "conv": 4, "norm_groups": 1}, _latent(16, 768)),
                  Qwen3Shape(num_layers=12, hidden=1024, intermediate=3072, vocab=32768)),
        "w2048": (nepulix_dict(2048, 6, 6144, 32768, _retention(16, 128, 128),
                               {"heads": 64, "vdim": 64, "state": 128, "groups": 8, "conv": 4, "norm_groups": 8}, _latent(16, 1536)),
                  Qwen3Shape(num_layers=6, hidden=2048, intermediate=6144, vocab=32768)),
    }


def sozarax_dict(width, layers, ff, vocab, wkv, att, experts, top):
    """Two time-mixing layers, one attention layer and so on; dense and routed feed-forwards in turn, a token's experts together as
    wide as the dense one."""
    mlps = [{"kind": "dense", "ff": ff}, {"kind": "moe", "expert": {"ff": ff // top}, "router": {"experts": experts, "top": top}}]
    out = [{"type": "attention" if i % 3 == 2 else "wkv", "mixer": att if i % 3 == 2 else wkv, "mlp": mlps[i % 2]} for i in range(layers)]
    return {"architecture": "Sozarax", "width": width, "vocab": vocab, "norm": {"eps": 1e-6}, "embedding": {"scale": width ** 0.5}, "layers": out,
            "loop": {"start": 0, "stop": layers, "times": 1}}


def sozarax_sizes():
    """name -> (Sozarax config.json dict, Nepulix dict and Qwen3Shape of equal size)"""
    att = {"heads": 16, "kv_heads": 8, "dim": 128, "vdim": 128, "scale": 128 ** -0.5, "q_temp": {"coef": 0.1, "every": 1024}}
    near = sizes()
    return {"w1024": (sozarax_dict(1024, 12, 3072, 32768, {"heads": 16, "dim": 64}, att, 16, 2), *near["w1024"]),
            "w2048": (sozarax_dict(2048, 6, 6144, 32768, {"heads": 16, "dim": 128}, att, 32, 4), *near["w2048"])}


def lulizen_dict(width, layers, ff, vocab, heads, experts, top):
    """Layers over chunks and over windows in turn; of three layers one is dense, and a token's experts and the shared one are together
    as wide as the dense one."""
    att = {"heads": heads, "kv_heads": heads // 2, "dim": 128, "vdim": 128, "scale": 128 ** -0.5, "softcap": 30.0, "rot": {"base": 5e5, "dims": 128}}
    kinds = [("attention", dict(att, mask={"size": 8192})), ("attention_2", dict(att, mask={"size": 512, "keep_first": 16}, rot={"base": 1e4, "dims": 64}))]
    unit = ff // 3 if top == 2 else ff // 6
    moe = {"kind": "moe", "expert": {"ff": unit, "limit": 7.0}, "shared": {"ff": ff - top * unit, "limit": 7.0},
           "router": {"experts": experts, "top": top, "scale": 2.5, "groups": {"count": 4, "keep": 2}}}
    out = [{"type": kinds[i % 2][0], "mixer": kinds[i % 2][1], "mlp": {"kind": "dense", "ff": ff} if i % 3 == 0 else moe} for i in range(layers)]
    return {"architecture": "Lulizen", "width": width, "vocab": vocab, "norm": {"eps": 1e-6}, "layers": out,
            "embedding": {"bigram": {"buckets": vocab - 1, "mul_prev": 37, "mul_cur": 17}}}


def lulizen_sizes():
    """name -> (Lulizen config.json dict, Sozarax dict and Qwen3Shape of equal size)"""
    near = {n: (c[0], c[-1]) for n, c in sozarax_sizes().items()}
    return {"w1024": (lulizen_dict(1024, 12, 3072, 32768, 16, 16, 2), *near["w1024"]),
            "w2048": (lulizen_dict(2048, 6, 6144, 32768, 16, 32, 4), *near["w2048"])}


def fedovik_dict(width, layers, ff, vocab, memory, att, left, right):
    """A matrix memory, attention with sigmoid weights, and attention over a window beside a delta rule in turn; one pass of the loop, so
    that a token runs through as many layers as in the other models."""
    kinds = [("mlstm", memory), ("attention", att), ("parallel", {"left": left, "right": right, "left_scale": 0.7, "right_scale": 0.7})]
    out = [{"type": kinds[i % 3][0], "mixer": kinds[i % 3][1], "mlp": {"kind": "dense", "ff": ff}} for i in range(layers)]
    return {"architecture": "Fedovik", "width": width, "vocab": vocab, "norm": {"eps": 1e-6}, "embedding": {"scale": width ** 0.5}, "layers": out,
            "loop": {"start": 0, "stop": layers, "times": 1}}


def fedovik_sizes():
    """name -> (Fedovik config.json dict, Sozarax dict and Qwen3Shape of equal size)"""
    att = {"heads": 16, "kv_heads": 8, "dim": 128, "vdim": 128, "scale": 128 ** -0.5}
    left = lambda heads: dict(att, heads=heads, kv_heads=heads // 2, mask={"size": 512})      # noqa: E731
    near = {n: (c[0], c[-1]) for n, c in sozarax_sizes().items()}
    rot = {"rot": {"base": 5e5, "dims": 128}}
    return {"w1024": (fedovik_dict(1024, 12, 3072, 32768, {"heads": 8, "dim": 128, "vdim": 128, "gate_cap": 15.0}, {**att, **rot}, left(8),
                                   {"heads": 8, "kv_heads": 8, "dim": 128, "vdim": 128, "conv": 4}), *near["w1024"]),
            "w2048": (fedovik_dict(2048, 6, 6144, 32768, {"heads": 16, "dim": 128, "vdim": 128, "gate_cap": 15.0}, {**att, **rot}, left(16),
                                   {"heads": 16, "kv_heads": 16, "dim": 128, "vdim": 128, "conv": 4}), *near["w2048"])}


DESIGNS = {"nepulix": (sizes, "Qwen3"), "sozarax": (sozarax_sizes, "Nepulix and Qwen3"), "lulizen": (lulizen_sizes, "Sozarax and Qwen3"),
           "fedovik": (fedovik_sizes, "Sozarax and Qwen3")}


def _events(fn, warmup, steps):
    for _ in range(warmup):
        fn()
    torch.cuda.synchronize()
    a, b = torch.cuda.Event(enable_timing=True), torch.cuda.Event(enable_timing=True)
    a.record()
    for _ in range(steps):
        fn()
    b.record()
    torch.cuda.synchronize()
    return a.elapsed_time(b) / steps * 1e-3


def model_throughput(config, seed=0, prompts=16, prompt_len=1024, decode=((64, 1024), (256, 1024)), steps=20, warmup=5):
    """Tokens per second of one prefill step (prompts x prompt_len tokens) and of decode steps (batch, context) replayed from
    HIP graphs."""
    from .engine import Engine
    max_bs = max(b for b, _ in decode)
    max_ctx = max(c for _, c in decode) + 64
    blocks = max(prompts * -(-prompt_len // 256), max(b * -(-(c + 64) // 256) for b, c in decode))
    eng = Engine(config, num_blocks=blocks, max_num_seqs=max_bs, seed=seed, max_num_batched_tokens=prompts * prompt_len, max_model_len=8192)
    g = torch.Generator().manual_seed(seed)
    for _ in range(prompts):
        eng.add_request(torch.randint(0, eng.model.vocab, (prompt_len,), generator=g).tolist(), 4)
    seqs, is_prefill = eng._schedule()
    assert is_prefill and len(seqs) == prompts
    ids, pos, ctx = eng._prepare_prefill(seqs)
    out = {"prefill": {"prompts": prompts, "prompt_len": prompt_len}, "decode": []}
    dt = _events(lambda: eng.forward(ids, pos, dict(ctx)), warmup, steps)      # a fresh ctx: per-step plans are made anew
    out["prefill"].update(ms=round(dt * 1e3, 3), tok_per_s=round(prompts * prompt_len / dt))
    for q in list(eng.running):
        eng.running.remove(q)
        eng.cache.release(q)
    eng.capture_decode_graphs(max_bs=max_bs, max_model_len=max_ctx)
    for bs, context in decode:
        live = []
        for _ in range(bs):
            q = eng.open_sequence()
            q.token_ids = [1] * (context - 1) + [int(torch.randint(0, eng.model.vocab, (), generator=g))]
            eng.cache.hold(q, context)
            live.append(q)
        ids, pos, dctx = eng._prepare_decode(live)
        dt = _events(lambda: eng._decode_replay(ids, pos, dctx), warmup, steps)
        out["decode"].append({"batch": bs, "context": context, "ms": round(dt * 1e3, 3), "tok_per_s": round(bs / dt)})
        for q in live:
            eng.cache.release(q)
    del eng
    torch.cuda.empty_cache()
    return out


def graph_time(fn, calls=10, replays=10):
    """Seconds per call of fn(i), `calls` of them captured into a graph and replayed back to back."""
    for i in range(3):
        fn(i)
    torch.cuda.synchronize()
    graph = torch.cuda.CUDAGraph()
    with torch.cuda.graph(graph):
        for i in range(calls):
            fn(i)
    return _events(graph.replay, 3, replays) / calls


class KernelTable:
    """Rows {kernel, shape, us, bound, achieved, unit, frac, like, like_frac, times_further}: algorithmic work over time, as a fraction of
    the roof, beside the fraction of a like kernel timed before."""

    def __init__(self, dev, seed=0, only=""):
        self.dev, self.seed, self.only = dev, seed, tuple(x for x in only.split(",") if x)
        self.g = torch.Generator(device=dev).manual_seed(seed)
        self.rows, self.likes = [], {}

    def rnd(self, *shape):
        return torch.randn(shape, generator=self.g, device=self.dev, dtype=torch.float32).bfloat16()

    def f32(self, *shape):
        return torch.randn(shape, generator=self.g, device=self.dev)

    def i32(self, x):
        return torch.tensor(x, dtype=torch.int32, device=self.dev)

    def add(self, name, shape, timed, nbytes=0.0, flops=0.0, like=None):
        if self.only and not name.startswith(self.only):
            return
        seconds = timed()
        t_mem, t_math = nbytes / (HBM * 1e9), flops / (MFMA * 1e12)
        bound = "hbm" if t_mem >= t_math else "mfma"
        value, unit = (nbytes / seconds / 1e9, "GB/s") if bound == "hbm" else (flops / seconds / 1e12, "TFLOP/s")
        r = {"kernel": name, "shape": shape, "us": round(seconds * 1e6, 2), "bound": bound, "achieved": round(value, 1), "unit": unit,
             "frac": round(max(t_mem, t_math) / seconds, 4)}
        if like is None:
            self.likes[name] = r["frac"]
        else:
            known = self.likes.get(like)
            r.update(like=like, like_frac=known, times_further=None if known is None else round(known / r["frac"], 2))
            self.likes.setdefault(f"{name} {shape}", r["frac"])
        self.rows.append(r)


PROMPTS = [1024] * 16
T = sum(PROMPTS)      # tokens of a prefill step


def op(name):
    from . import mops
    return mops.get_op(name, "hip")


def decode_contexts(t):
    """Context lengths of a decode step, blocks of the pool, block table of shuffled blocks, lengths on the device."""
    from . import workloads as W
    ctx = W.random_seq_lens(256, 512, 4096, seed=t.seed)
    nb = [(c + 255) // 256 for c in ctx]
    perm = torch.randperm(sum(nb), generator=torch.Generator().manual_seed(t.seed)).to(torch.int32)
    table, at = torch.full((256, max(nb)), -1, dtype=torch.int32), 0
    for b, n in enumerate(nb):
        table[b, :n] = perm[at:at + n]
        at += n
    return ctx, sum(nb), table.to(t.dev), t.i32(ctx)


def _handles(t):
    return t.add, t.rnd, t.i32, t.dev


def qwen3_kernels(t):
    """The Qwen3 path's kernels, the yardstick."""
    from . import workloads as W
    add, rnd, i32, dev = _handles(t)
    ctx, blocks, table, lens_g = decode_contexts(t)
    kc, vc, q = rnd(blocks, 256, 8, 128), rnd(blocks, 256, 8, 128), rnd(256, 1, 16, 128)
    add("paged_decode", "256 x uniform[512,4096], 16/8 heads", lambda: graph_time(lambda i: op("flash_attn_with_kvcache")(
        q, kc, vc, cache_seqlens=lens_g, block_table=table, softmax_scale=0.088, causal=True), 4), nbytes=W.decode_bytes(ctx, 16, 8, table.shape[1]))
    del kc, vc
    d = W.to_device(W.prefill_inputs(PROMPTS, seed=t.seed), dev)
    add("varlen_prefill", "16 x 1024, 16/8 heads of 128", lambda: _events(lambda: op("flash_attn_varlen_func")(
        d["q"], d["k"], d["v"], max_seqlen_q=1024, cu_seqlens_q=d["cu_seqlens"], max_seqlen_k=1024, cu_seqlens_k=d["cu_seqlens"], softmax_scale=d["scale"],
        causal=True, block_table=None), 300, 200), flops=W.prefill_flops(PROMPTS, 16))
    bufs = [rnd(T, 6144) for _ in range(4)]
    halves = [b.chunk(2, dim=-1) for b in bufs]
    add("siluAndMul", f"{T} x 3072", lambda: graph_time(lambda i: op("siluAndMul")(*halves[i % 4]), 8), nbytes=T * 3072 * 6)
    x4, r4, w4 = [rnd(512, 4096) for _ in range(24)], [rnd(512, 4096) for _ in range(24)], rnd(4096)
    add("add_rms", "512 x 4096", lambda: graph_time(lambda i: op("add_rms_forward")(x4[i % 24], r4[i % 24], w4, 1e-6), 24), nbytes=512 * 4096 * 8)
    xt, rt, w1 = [rnd(T, 1024) for _ in range(4)], [rnd(T, 1024) for _ in range(4)], rnd(1024)
    add("add_rms prefill", f"{T} x 1024", lambda: graph_time(lambda i: op("add_rms_forward")(xt[i % 4], rt[i % 4], w1, 1e-6), 8), nbytes=T * 1024 * 8)
    qkv, kc2 = [rnd(T, 4096) for _ in range(2)], torch.zeros((T // 256, 256, 8, 128), dtype=torch.bfloat16, device=dev)
    vc2, ang, slots = torch.zeros_like(kc2), torch.rand((T, 1, 64), device=dev), torch.randperm(T, device=dev).to(torch.int32)
    nw = rnd(128)
    cs, sn = ang.cos(), ang.sin()
    add("qk_norm_rope_store", f"{T} tokens, 16/8 heads", lambda: graph_time(lambda i: op("qk_norm_rope_store")(
        qkv[i % 2], nw, nw, 1e-6, cs, sn, kc2, vc2, slots, 16, 8, need_k=False), 8), nbytes=T * (4096 * 2 + 512 + 4 + 2048 * 2 + 2 * 1024 * 2))
    wl = rnd(1024, 1024)
    xl = [rnd(T, 1024) for _ in range(4)]
    add("linear", f"{T} x 1024 x 1024 (library)", lambda: graph_time(lambda i: op("linear")(xl[i % 4], wl), 8), flops=2.0 * T * 1024 * 1024, nbytes=T * 1024 * 4)
    wls = [rnd(1024, 1024) for _ in range(64)]
    xs = rnd(256, 1024)
    add("linear decode", "256 x 1024 x 1024 (library)", lambda: graph_time(lambda i: op("linear")(xs, wls[i % 64]), 64), nbytes=1024 * 1024 * 2 + 256 * 1024 * 4)


def latent_kernels(t):
    from .layers import Rotary
    from .mops.hip import recurrent_ops as R
    add, rnd, i32, dev = _handles(t)
    ctx, blocks, table, lens_g = decode_contexts(t)
    slots = torch.randperm(T, device=dev).to(torch.int32)
    H, kr, rot, dim, vdim = 16, 512, 64, 128, 128
    cache, ql, qn = rnd(blocks, 256, kr + rot), rnd(256, H, kr), rnd(256, H, dim + rot)
    trig = Rotary(8192, dev).table(1e4, rot)
    add("latent_decode", "256 x uniform[512,4096], 16 heads, 512+64", lambda: graph_time(lambda i: op("latent_decode")(
        ql, qn[..., dim:], cache, trig, lens_g, table, 0.07), 4), nbytes=sum(ctx) * (kr + rot) * 2 + 256 * H * (2 * kr + rot) * 2,
        flops=2.0 * sum(ctx) * H * (2 * kr + rot), like="paged_decode")
    wabs, wv = rnd(H, kr, dim), rnd(H, vdim, kr)
    add("head_linear", "256 rows, 16 x 128 -> 512", lambda: graph_time(lambda i: op("head_linear")(qn[..., :dim], wabs), 16),
        nbytes=H * kr * dim * 2 + 256 * H * (dim + kr) * 2, flops=2.0 * 256 * H * dim * kr, like="linear decode")
    add("head_linear", "256 rows, 16 x 512 -> 128", lambda: graph_time(lambda i: op("head_linear")(ql, wv), 16),
        nbytes=H * kr * vdim * 2 + 256 * H * (vdim + kr) * 2, flops=2.0 * 256 * H * vdim * kr, like="linear decode")
    del cache
    p32 = (torch.arange(T, device=dev) % 1024).to(torch.int32)
    row_seq, row_pos, tiles = R.latent_prefill_plan(PROMPTS, [0] * 16, 0, 0)
    row_seq, row_pos, tiles = i32(row_seq), i32(row_pos), i32(tiles)
    qp, kp, krp, vt = rnd(T, H, dim + rot), rnd(T, H * dim), rnd(T, rot), rnd(H * vdim, T)
    op_out = torch.empty((T, H, vdim), dtype=torch.bfloat16, device=dev)
    add("latent_prefill", "16 x 1024, 16 heads, 192/128", lambda: _events(lambda: op("latent_prefill")(qp, kp, krp, vt, tiles, 0.07, op_out), 300, 200),
        flops=sum(2.0 * H * (dim + rot + vdim) * n * (n + 1) / 2 for n in PROMPTS), like="varlen_prefill")
    add("rotate_pairs", f"{T} x 16 heads x 64", lambda: graph_time(lambda i: op("rotate_pairs")(qp[..., dim:], p32, trig), 8), nbytes=T * H * rot * 4.0, like="qk_norm_rope_store")
    pages = rnd(T // 256, 256, kr + rot)
    ptab = torch.arange(T // 256, dtype=torch.int32, device=dev).view(16, -1)
    add("latent_gather", f"{T} rows", lambda: graph_time(lambda i: op("latent_gather")(pages, ptab, row_seq, row_pos, kr, rot), 8), nbytes=T * (kr + rot) * 4, like="siluAndMul")
    down, wq, wk = [rnd(T, 768 + kr + rot) for _ in range(4)], rnd(768), rnd(kr)
    add("latent_prepare", f"{T} tokens, 768 / 512+64", lambda: graph_time(lambda i: op("latent_prepare")(down[i % 4], wq, wk, 1e-6, trig, p32, slots, pages, 768, kr, rot), 8),
        nbytes=T * (768 + kr + rot) * 4, like="qk_norm_rope_store")


def decayed_kernels(t, tag, heads, groups, dd, vd, const):
    from .layers import Rotary
    from .mops.hip import recurrent_ops as R
    add, rnd, i32, dev = _handles(t)
    bs = 256
    pitch = R.recurrence_state_pitch(dd)
    state = torch.randn((bs, heads, vd, pitch), generator=t.g, device=dev)
    gn, inner = groups * dd, heads * vd
    opts, conv = {"k_scale": dd ** -0.5}, None
    if const:
        dec = torch.tensor([1 - 2.0 ** (-5 - i % 8) for i in range(heads)], dtype=torch.float64)
        opts.update(decay=dec.float().to(dev), log_decay=dec.log().float().to(dev), cos_sin=Rotary(8192, dev).table(1e4, dd))
    else:
        f = t.f32
        ch = inner + 2 * gn
        opts.update(dt_bias=f(heads) - 2, neg_a=-torch.exp(f(heads)), skip=f(heads))
        conv = (f(4, ch), f(ch), torch.zeros((bs, 4, ch), dtype=torch.bfloat16, device=dev), (inner + gn, inner, 0))
    width = 2 * gn + inner
    x, dt, o = rnd(bs, width), rnd(bs, heads), torch.empty((bs, inner), dtype=torch.bfloat16, device=dev)
    sl, st = torch.arange(bs, dtype=torch.int32, device=dev), torch.full((bs,), 1000, dtype=torch.int32, device=dev)
    more = {} if const else {"dt": dt, "conv": conv}
    add("decayed_recurrence " + tag, f"{bs} sequences, {heads} x {dd} x {vd}", lambda: graph_time(lambda i: op("decayed_recurrence")(
        x[:, inner + gn:], x[:, inner:inner + gn], x[:, :inner], o, state, sl, st, heads, groups, dd, vd, **opts, **more), 6),
        nbytes=2.0 * bs * heads * dd * vd * 4 + bs * (width + inner) * 2, like="paged_decode")
    xs = [rnd(T, width) for _ in range(2)]
    dts, oT = rnd(T, heads), torch.empty((T, inner), dtype=torch.bfloat16, device=dev)
    for nseq in (16, 1):
        cu = list(range(0, T + 1, T // nseq))
        segs, bounds = R.recurrence_segments([T // nseq] * nseq, heads, groups, vd)
        segs, bounds, cu = i32(segs), i32(bounds), i32(cu)
        more = {} if const else {"dt": dts}
        # least arithmetic at 64 tokens a chunk: scores and their product below the diagonal, state in and out
        add("decayed_chunks " + tag, f"{nseq} x {T // nseq}, {heads} x {dd} x {vd}", lambda: _events(lambda: op("decayed_chunks")(
            xs[0][:, inner + gn:], xs[0][:, inner:inner + gn], xs[0][:, :inner], oT, state, sl[:nseq], torch.zeros_like(st[:nseq]), heads, groups, dd, vd, segs,
            bounds, cu_seqlens=cu, **opts, **more), 20, 50), flops=T * heads * (65.0 * (dd + vd) + 4.0 * dd * vd), nbytes=T * (width + inner) * 2.0,
            like="varlen_prefill")
    if not const:
        tok_seq, sl16 = torch.arange(T, device=dev).div(1024, rounding_mode="floor").to(torch.int32), sl[:16]
        cu16, z16 = i32(list(range(0, T + 1, 1024))), torch.zeros(16, dtype=torch.int32, device=dev)
        big = [rnd(T, width + inner + heads) for _ in range(2)]
        add("short_conv", f"{T} x {width}, 4 taps", lambda: graph_time(lambda i: op("short_conv")(
            big[i % 2][:, inner:inner + width], conv[0], conv[1], conv[2], tok_seq, cu16, z16, sl16), 4), nbytes=T * width * 4.0, like="siluAndMul")


def nepulix_kernels(t):
    add, rnd, i32, dev = _handles(t)
    latent_kernels(t)
    decayed_kernels(t, "retention", 16, 16, 128, 128, True)
    decayed_kernels(t, "mamba2", 64, 8, 128, 64, False)
    bufs = [rnd(T, 6144) for _ in range(4)]
    halves = [b.chunk(2, dim=-1) for b in bufs]
    x4, r4, w4 = [rnd(512, 4096) for _ in range(24)], [rnd(512, 4096) for _ in range(24)], rnd(4096)
    xt, rt, w1 = [rnd(T, 1024) for _ in range(4)], [rnd(T, 1024) for _ in range(4)], rnd(1024)
    lim = lambda i: op("clamped_glu")(*halves[i % 4], 7.0)      # noqa: E731
    add("clamped_glu", f"{T} x 3072", lambda: graph_time(lim, 8), nbytes=T * 3072 * 6, like="siluAndMul")
    add("gated_group_norm", f"{T} x 3072, 24 groups", lambda: graph_time(lambda i: op("gated_group_norm")(*halves[i % 4], 24, 1e-6), 8), nbytes=T * 3072 * 6, like="siluAndMul")
    add("gated_group_norm", f"{T} x 3072, 1 group", lambda: graph_time(lambda i: op("gated_group_norm")(*halves[i % 4], 1, 1e-6, gate_first=True), 8), nbytes=T * 3072 * 6,
        like="siluAndMul")
    f4 = [x.float() for x in r4]
    add("norm_residual_add", "512 x 4096", lambda: graph_time(lambda i: op("norm_residual_add")(f4[i % 24], x4[i % 24], w4, 1e-6, 1.0), 24), nbytes=512 * 4096 * 12, like="add_rms")
    ft = [x.float() for x in rt]
    add("norm_residual_add", f"{T} x 1024", lambda: graph_time(lambda i: op("norm_residual_add")(ft[i % 4], xt[i % 4], w1, 1e-6, 1.0), 8), nbytes=T * 1024 * 12, like="add_rms prefill")
    add("rms_norm_f32", "512 x 4096", lambda: graph_time(lambda i: op("rms_norm_f32")(f4[i % 24], w4, 1e-6, 1.0), 24), nbytes=512 * 4096 * 6, like="add_rms")
    emb, ids = rnd(32768, 1024), [torch.randint(0, 32768, (T,), device=dev) for _ in range(4)]
    add("embed_residual", f"{T} x 1024", lambda: graph_time(lambda i: op("embed_residual")(ids[i % 4], emb), 8), nbytes=T * 1024 * 8.0, like="add_rms prefill")


def sozarax_attention(t):
    from .mops.hip.attention_ops import biased_prefill_tiles
    from .layers.biased_attention import distance_slopes
    add, rnd, i32, dev = _handles(t)
    ctx, blocks, table, lens_g = decode_contexts(t)
    H, G, d = 16, 8, 128
    slopes = distance_slopes(H).to(dev)
    kp, vp, q = rnd(blocks, 256, G, d), rnd(blocks, 256, G, d), rnd(256, H, d)
    add("biased_decode", "256 x uniform[512,4096], 16/8 heads of 128", lambda: graph_time(lambda i: op("biased_decode")(q, kp, vp, d, d, lens_g, table, 0.088, slopes=slopes), 4),
        nbytes=sum(ctx) * G * 2 * d * 2.0 + 256 * H * 2 * d * 2, like="paged_decode")
    del kp, vp
    kp, vp, q = rnd(T // 256, 256, G, d), rnd(T // 256, 256, G, d), rnd(T, H, d)
    tiles, ptab = i32(biased_prefill_tiles(PROMPTS, [0] * 16, 0, 0)), torch.arange(T // 256, dtype=torch.int32, device=dev).view(16, -1)
    out, lens = torch.empty((T, H, d), dtype=torch.bfloat16, device=dev), i32([0] * T)
    add("biased_prefill", "16 x 1024, 16/8 heads of 128", lambda: _events(lambda: op("biased_prefill")(q, kp, vp, d, d, tiles, ptab, 0.088, lens, slopes=slopes, out=out), 300, 200),
        flops=sum(2.0 * H * 2 * d * n * (n + 1) / 2 for n in PROMPTS), like="varlen_prefill")
    qkv, wq, wk = [rnd(T, (H + 2 * G) * d) for _ in range(2)], rnd(H * d), rnd(G * d)
    pos, slots = (torch.arange(T, device=dev) % 1024).to(torch.int32), torch.randperm(T, device=dev).to(torch.int32)
    add("attention_prepare", f"{T} tokens, 16/8 heads of 128", lambda: graph_time(lambda i: op("attention_prepare")(qkv[i % 2], wq, wk, 1e-6, pos, slots, kp, vp, H, G, d, d), 8),
        nbytes=T * (H + 2 * G) * d * 4.0, like="qk_norm_rope_store")


def time_mixing_kernels(t):
    from .mops.hip import recurrent_ops as R
    add, rnd, i32, dev = _handles(t)
    for heads, dd in ((16, 64), (16, 128)):
        n = heads * dd
        bs, pitch = 256, R.recurrence_state_pitch(dd)
        state, sl = torch.randn((bs, heads, dd, pitch), generator=t.g, device=dev), torch.arange(bs, dtype=torch.int32, device=dev)
        st, u = torch.full((bs,), 1000, dtype=torch.int32, device=dev), t.f32(n)
        x, ld, o = rnd(3, bs, n), -torch.exp(t.f32(bs, n) - 3), torch.empty((bs, n), dtype=torch.bfloat16, device=dev)
        add("decayed_recurrence channels", f"{bs} sequences, {heads} x {dd} x {dd}", lambda: graph_time(lambda i: op("decayed_recurrence")(
            x[0], x[1], x[2], o, state, sl, st, heads, heads, dd, dd, channel_decay=ld, bonus=u), 6), nbytes=2.0 * bs * n * dd * 4 + bs * n * 12, like="decayed_recurrence retention 256 sequences, 16 x 128 x 128")
        xs, ldT, oT = rnd(3, T, n), -torch.exp(t.f32(T, n) - 3), torch.empty((T, n), dtype=torch.bfloat16, device=dev)
        for nseq in (16, 1):
            segs, ends = (i32(v) for v in R.channel_segments([T // nseq] * nseq, heads, dd))
            cu, zero = i32(list(range(0, T + 1, T // nseq))), torch.zeros(nseq, dtype=torch.int32, device=dev)
            add("channel_chunks", f"{nseq} x {T // nseq}, {heads} x {dd} x {dd}", lambda: _events(lambda: op("channel_chunks")(
                xs[0], xs[1], xs[2], oT, state, sl[:nseq], zero, heads, heads, dd, dd, segs, ends, cu_seqlens=cu, channel_decay=ldT, bonus=u), 20, 50),
                flops=T * heads * (17.0 * 2 * dd + 4.0 * dd * dd), nbytes=T * n * 12.0, like=f"decayed_chunks retention {nseq} x {T // nseq}, 16 x 128 x 128")
    width, rank = 1024, 32
    xw, mu, before = [rnd(T, width) for _ in range(4)], t.f32(5, width), torch.zeros((16, width), dtype=torch.bfloat16, device=dev)
    cu16, z16, sl16 = i32(list(range(0, T + 1, 1024))), torch.zeros(16, dtype=torch.int32, device=dev), torch.arange(16, dtype=torch.int32, device=dev)
    seq = torch.arange(T, device=dev).div(1024, rounding_mode="floor").to(torch.int32)
    add("token_mix", f"{T} x {width}, 5 blends", lambda: graph_time(lambda i: op("token_mix")(xw[i % 4], mu, before, z16, sl16, seq, cu16), 4), nbytes=T * width * 12.0, like="siluAndMul")
    z, w2, w0 = [rnd(T, rank) for _ in range(4)], rnd(1024, rank), t.f32(1024)
    add("low_rank_decay", f"{T} x {rank} -> 1024", lambda: graph_time(lambda i: op("low_rank_decay")(z[i % 4], w2, w0), 4), nbytes=T * (rank * 2 + 1024 * 4.0), like="siluAndMul")
    y, gate, wn = [rnd(T, 1024) for _ in range(4)], [rnd(T, 1024) for _ in range(4)], rnd(1024)
    add("gated_group_norm", f"{T} x 1024, 16 groups", lambda: graph_time(lambda i: op("gated_group_norm")(y[i % 4], gate[i % 4], 16, 1e-6, weight=wn), 8), nbytes=T * 1024 * 6.0, like="siluAndMul")
    mixes, wr, w1 = rnd(5, 256, width), [rnd(4, 1024, width) for _ in range(16)], rnd(rank, width)
    add("grouped_linear", f"256 rows, 4 x 1024 -> 1024 and {rank}", lambda: graph_time(lambda i: op("grouped_linear")(mixes, wr[i % 16], w1), 16),
        nbytes=4 * 1024 * 1024 * 2 + 256 * 9 * 1024 * 2, flops=2.0 * 256 * 4 * 1024 * 1024, like="linear decode")


EXPERTS = ((T, 1024, 1536, 16, 2), (256, 1024, 1536, 16, 2), (T, 2048, 1536, 32, 4), (256, 2048, 1536, 32, 4))      # tokens, width, ff, experts, top


def sozarax_experts(t):
    add, rnd, i32, dev = _handles(t)
    for tokens, w, ff, experts, top in EXPERTS:
        tag, n = f"{tokens} x {w}, top {top} of {experts} x {ff}", tokens * top
        sets = 2 if tokens == T else 4
        h, router = [rnd(tokens, w) for _ in range(sets)], rnd(experts, w)
        gu, down = [rnd(experts, 2, ff, w) for _ in range(sets)], [rnd(experts, w, ff) for _ in range(sets)]
        routing = [op("moe_route")(x, router, top) for x in h]
        ys = [op("moe_gate_up")(h[i], gu[i], routing[i]) for i in range(sets)]
        like = "linear" if tokens == T else "linear decode"
        add("moe_route", tag, lambda: graph_time(lambda i: op("moe_route")(h[i % sets], router, top), 8), nbytes=tokens * w * 2.0 + n * 24, like="add_rms prefill" if tokens == T else "linear decode")
        add("moe_gate_up", tag, lambda: graph_time(lambda i: op("moe_gate_up")(h[i % sets], gu[i % sets], routing[i % sets]), 8),
            nbytes=experts * 2.0 * ff * w * 2 + tokens * w * 2.0 + n * ff * 2.0, flops=4.0 * n * ff * w, like=like)
        add("moe_down", tag, lambda: graph_time(lambda i: op("moe_down")(ys[i % sets], down[i % sets], routing[i % sets]), 8),
            nbytes=experts * float(ff) * w * 2 + n * ff * 2.0 + n * w * 2.0, flops=2.0 * n * ff * w, like=like)


def sozarax_residual(t):
    add, rnd, i32, dev = _handles(t)
    sq = [rnd(T, 3072) for _ in range(4)]
    add("squared_relu", f"{T} x 3072", lambda: graph_time(lambda i: op("squared_relu")(sq[i % 4]), 8), nbytes=T * 3072 * 4.0, like="siluAndMul")
    for rows, n, parts, like in ((512, 4096, 1, "add_rms"), (T, 1024, 1, "add_rms prefill"), (T, 1024, 2, "add_rms prefill")):
        sets = 24 if rows == 512 else 4
        res, yy, wa, wb = [t.f32(rows, n) for _ in range(sets)], [rnd(rows * parts, n) for _ in range(sets)], rnd(n), rnd(n)
        add("add_norm_norm", f"{rows} x {n}, {parts} part{'s' if parts > 1 else ''}", lambda: graph_time(lambda i: op("add_norm_norm")(res[i % sets], yy[i % sets], wa, wb, 1e-6), 24 if rows == 512 else 8),
            nbytes=rows * n * (10.0 + 2 * parts), like=like)


def sozarax_kernels(t):
    sozarax_attention(t)
    time_mixing_kernels(t)
    sozarax_experts(t)
    sozarax_residual(t)


def lulizen_kernels(t):
    from .layers import Rotary
    from .mops.hip.attention_ops import Scores, biased_prefill_tiles
    from .mops.hip.mixture_ops import CommonUnit, Weighted
    add, rnd, i32, dev = _handles(t)
    # ---- attention
    ctx, blocks, table, lens_g = decode_contexts(t)
    H, G, d, cap = 16, 8, 128, 30.0
    sinks = t.f32(H)
    kp, vp, q, gate = rnd(blocks, 256, G, d), rnd(blocks, 256, G, d), rnd(256, H, d), rnd(256, H)
    like = "biased_decode 256 x uniform[512,4096], 16/8 heads of 128"
    for label, scores, g, seen in (
            ("chunks of 8192, sinks", Scores(softcap=cap, chunk=8192, sinks=sinks), None, lambda n: n),
            ("chunks of 1024, sinks", Scores(softcap=cap, chunk=1024, sinks=sinks), None, lambda n: (n - 1) % 1024 + 1),
            ("window of 1024 and 64, gate", Scores(softcap=cap, window=1024, keep_first=64), gate, lambda n: min(n, 1024 + 64)),
            ("chunks of 8192, cap 100", Scores(softcap=100.0, chunk=8192), None, lambda n: n)):
        add("biased_decode", f"256 x uniform[512,4096], {label}", lambda: graph_time(lambda i: op("biased_decode")(q, kp, vp, d, d, lens_g, table, 0.088, scores=scores, gate=g), 4),
            nbytes=sum(map(seen, ctx)) * G * 2 * d * 2.0 + 256 * H * 2 * d * 2, like=like)
    del kp, vp
    kp, vp, q, gate = rnd(T // 256, 256, G, d), rnd(T // 256, 256, G, d), rnd(T, H, d), rnd(T, H)
    out, lens = torch.empty((T, H, d), dtype=torch.bfloat16, device=dev), i32([0] * T)
    for n, label, scores, g, seen in (
            (1024, "chunks of 8192, sinks", Scores(softcap=cap, chunk=8192, sinks=sinks), None, lambda i: i + 1),
            (1024, "cap 100", Scores(softcap=100.0, chunk=8192), None, lambda i: i + 1),
            (4096, "chunks of 1024, sinks", Scores(softcap=cap, chunk=1024, sinks=sinks), None, lambda i: i % 1024 + 1),
            (4096, "window of 1024 and 64, gate", Scores(softcap=cap, window=1024, keep_first=64), gate, lambda i: min(i + 1, 1024 + 64)),
            (4096, "window of 512 and 16, gate", Scores(softcap=cap, window=512, keep_first=16), gate, lambda i: min(i + 1, 512 + 16))):
        b = T // n
        tiles, ptab = i32(biased_prefill_tiles([n] * b, [0] * b, 0, 0)), torch.arange(T // 256, dtype=torch.int32, device=dev).view(b, -1)
        add("biased_prefill", f"{b} x {n}, {label}", lambda: _events(lambda: op("biased_prefill")(
            q, kp, vp, d, d, tiles, ptab, 0.088, lens, out=out, scores=scores, gate=g), 300, 200), flops=2.0 * H * 2 * d * b * sum(map(seen, range(n))),
            like="biased_prefill 16 x 1024, 16/8 heads of 128")
    qkv, w = [rnd(T, (H + 2 * G) * d + 16) for _ in range(2)], rnd(d)
    pos, slots = (torch.arange(T, device=dev) % 1024).to(torch.int32), torch.randperm(T, device=dev).to(torch.int32)
    for label, rot, norm in (("norms, 128 rotated", 128, w), ("64 rotated", 64, None)):
        trig = Rotary(8192, dev).table(1e4, rot)
        add("rotary_prepare", f"{T} tokens, 16/8 heads of 128, {label}", lambda: graph_time(lambda i: op("rotary_prepare")(
            qkv[i % 2], pos, slots, kp, vp, H, G, d, d, cos_sin=trig, q_weight=norm, k_weight=norm, eps=1e-6), 8), nbytes=T * (H + 2 * G) * d * 4.0,
            like=f"attention_prepare {T} tokens, 16/8 heads of 128")
    # ---- experts
    for tokens, wd, ff, experts, top in EXPERTS:
        tag, n = f"{tokens} x {wd}, top {top} of {experts} x {ff}", tokens * top
        sets = 2 if tokens == T else 4
        h, router, form = [rnd(tokens, wd) for _ in range(sets)], rnd(experts, wd), Weighted(0.1 * t.f32(experts), 4, 2, 2.5)
        gu, down = [rnd(experts, 2, ff, wd) for _ in range(sets)], [rnd(experts, wd, ff) for _ in range(sets)]
        routing = [op("moe_route")(x, router, top, weighted=form) for x in h]
        ys = [op("moe_gate_up")(h[i], gu[i], routing[i], 7.0) for i in range(sets)]
        if tokens != T:
            fs = ff * top // 2
            cu = [CommonUnit(rnd(2 * fs, wd), rnd(wd, fs), fs, fs, 7.0) for _ in range(sets)]
            yc = rnd(tokens, fs)
            add("moe_gate_up", f"{tag}, and a shared unit of {fs}", lambda: graph_time(lambda i: op("moe_gate_up")(h[i % sets], gu[i % sets], routing[i % sets], 7.0, common=cu[i % sets]), 8),
                nbytes=(experts * ff + fs) * 2.0 * wd * 2 + tokens * wd * 2.0 + (n * ff + tokens * fs) * 2.0, flops=4.0 * (n * ff + tokens * fs) * wd, like=f"moe_gate_up {tag}")
            add("moe_down", f"{tag}, and a shared unit of {fs}", lambda: graph_time(lambda i: op("moe_down")(ys[i % sets], down[i % sets], routing[i % sets], cu[i % sets], yc), 8),
                nbytes=(experts * ff + fs) * wd * 2.0 + (n * ff + tokens * fs) * 2.0 + (n + tokens) * wd * 2.0, flops=2.0 * (n * ff + tokens * fs) * wd, like=f"moe_down {tag}")
        add("moe_route", f"{tag}, 2 of 4 groups", lambda: graph_time(lambda i: op("moe_route")(h[i % sets], router, top, weighted=form), 8), nbytes=tokens * wd * 2.0 + n * 24,
            like=f"moe_route {tag}")
        add("moe_gate_up", f"{tag}, clamped", lambda: graph_time(lambda i: op("moe_gate_up")(h[i % sets], gu[i % sets], routing[i % sets], 7.0), 8),
            nbytes=experts * 2.0 * ff * wd * 2 + tokens * wd * 2.0 + n * ff * 2.0, flops=4.0 * n * ff * wd, like=f"moe_gate_up {tag}")
        add("moe_down", f"{tag}, weighted", lambda: graph_time(lambda i: op("moe_down")(ys[i % sets], down[i % sets], routing[i % sets]), 8),
            nbytes=experts * float(ff) * wd * 2 + n * ff * 2.0 + n * wd * 2.0, flops=2.0 * n * ff * wd, like=f"moe_down {tag}")
    # ---- around the sublayers
    halves = [rnd(T, 6144).chunk(2, dim=-1) for _ in range(4)]
    add("gelu_glu", f"{T} x 3072", lambda: graph_time(lambda i: op("gelu_glu")(*halves[i % 4]), 8), nbytes=T * 3072 * 6.0, like="siluAndMul")
    add("clamped_glu", f"{T} x 3072", lambda: graph_time(lambda i: op("clamped_glu")(*halves[i % 4], 7.0), 8), nbytes=T * 3072 * 6.0, like="siluAndMul")
    for rows, n, parts, more, like in ((512, 4096, 1, False, "512 x 4096, 1 part"), (T, 1024, 1, False, f"{T} x 1024, 1 part"), (T, 1024, 2, True, f"{T} x 1024, 2 parts")):
        sets = 24 if rows == 512 else 4
        res, yy, wa, wb = [t.f32(rows, n) for _ in range(sets)], [rnd(rows * parts, n) for _ in range(sets)], rnd(n), rnd(n)
        extra = [rnd(rows, n) if more else None for _ in range(sets)]
        add("add_norm_norm", f"{rows} x {n}, layer norms, {parts}{' + 1 parts' if more else ' part'}", lambda: graph_time(lambda i: op("add_norm_norm")(
            res[i % sets], yy[i % sets], wa, wb, 1e-6, center=True, extra=extra[i % sets]), 24 if rows == 512 else 8),
            nbytes=rows * n * (10.0 + 2 * (parts + more)), like=f"add_norm_norm {like}")
    res, w1 = [t.f32(T, 1024) for _ in range(4)], rnd(1024)
    add("layer_norm_f32", f"{T} x 1024", lambda: graph_time(lambda i: op("layer_norm_f32")(res[i % 4], w1, 1e-6), 8), nbytes=T * 1024 * 6.0, like="add_rms prefill")
    emb, pairs, ids = rnd(32768, 1024), rnd(32768, 1024), [torch.randint(0, 32768, (T,), device=dev) for _ in range(4)]
    before, cu16, z16, sl16 = torch.zeros(16, dtype=torch.int32, device=dev), i32(list(range(0, T + 1, 1024))), i32([0] * 16), torch.arange(16, dtype=torch.int32, device=dev)
    seq = torch.arange(T, device=dev).div(1024, rounding_mode="floor").to(torch.int32)
    add("embed_pairs", f"{T} x 1024", lambda: graph_time(lambda i: op("embed_pairs")(ids[i % 4], emb, pairs, 37, 17, before, z16, sl16, seq, cu16), 8), nbytes=T * 1024 * 8.0,
        like="add_rms prefill")


def fedovik_attention(t):
    from .layers import Rotary
    from .mops.hip.attention_ops import Scores, biased_prefill_tiles
    add, rnd, i32, dev = _handles(t)
    ctx, blocks, table, lens_g = decode_contexts(t)
    H, G, d = 16, 8, 128
    far = (t.f32(H).abs(), t.f32(H).abs())
    kp, vp, q, gate = rnd(blocks, 256, G, d), rnd(blocks, 256, G, d), rnd(256, H, d), rnd(256, H * d)
    like = "biased_decode 256 x uniform[512,4096], 16/8 heads of 128"
    for label, scores, g, seen in (
            ("sigmoid weights, gates", Scores(weight_bias=t.f32(H)), gate, lambda n: n),
            ("log distance", Scores(log_distance=far), None, lambda n: n),
            ("log distance, window of 512", Scores(log_distance=far, window=512), None, lambda n: min(n, 512))):
        add("biased_decode", f"256 x uniform[512,4096], {label}", lambda: graph_time(lambda i: op("biased_decode")(q, kp, vp, d, d, lens_g, table, 0.088, scores=scores, gate=g), 4),
            nbytes=sum(map(seen, ctx)) * G * 2 * d * 2.0 + 256 * H * (2 if g is None else 3) * d * 2, like=like)
    del kp, vp
    kp, vp, q, gate = rnd(T // 256, 256, G, d), rnd(T // 256, 256, G, d), rnd(T, H, d), rnd(T, H * d)
    out, lens = torch.empty((T, H * d), dtype=torch.bfloat16, device=dev), i32([0] * T)
    for n, label, scores, g, seen in (
            (1024, "sigmoid weights, gates", Scores(weight_bias=t.f32(H)), gate, lambda i: i + 1),
            (1024, "log distance", Scores(log_distance=far), None, lambda i: i + 1),
            (4096, "log distance, window of 512", Scores(log_distance=far, window=512), None, lambda i: min(i + 1, 512))):
        b = T // n
        tiles, ptab = i32(biased_prefill_tiles([n] * b, [0] * b, 0, 0)), torch.arange(T // 256, dtype=torch.int32, device=dev).view(b, -1)
        add("biased_prefill", f"{b} x {n}, {label}", lambda: _events(lambda: op("biased_prefill")(
            q, kp, vp, d, d, tiles, ptab, 0.088, lens, out=out, scores=scores, gate=g), 300, 200), flops=2.0 * H * 2 * d * b * sum(map(seen, range(n))),
            like="biased_prefill 16 x 1024, 16/8 heads of 128")
    qkv, w, bias = [rnd(T, (H + 2 * G) * d) for _ in range(2)], rnd(d), rnd((H + 2 * G) * d)
    pos, slots = (torch.arange(T, device=dev) % 1024).to(torch.int32), torch.randperm(T, device=dev).to(torch.int32)
    trig = Rotary(8192, dev).table(1e4, 128)
    for label, more in (("biases, neighbours turned", {"cos_sin": trig}), ("biases, norms", {"q_weight": w, "k_weight": w})):
        add("rotary_prepare", f"{T} tokens, 16/8 heads of 128, {label}", lambda: graph_time(lambda i: op("rotary_prepare")(
            qkv[i % 2], pos, slots, kp, vp, H, G, d, d, eps=1e-6, bias=bias, neighbours=True, **more), 8), nbytes=T * (H + 2 * G) * d * 4.0,
            like=f"attention_prepare {T} tokens, 16/8 heads of 128")


def fedovik_recurrences(t):
    from .mops.hip import recurrent_ops as R
    add, rnd, i32, dev = _handles(t)
    bs, heads = 256, 16
    sl, st = torch.arange(bs, dtype=torch.int32, device=dev), torch.full((bs,), 1000, dtype=torch.int32, device=dev)
    for dd in (64, 128):
        n, pitch = heads * dd, R.recurrence_state_pitch(dd)
        shape = f"{heads} x {dd} x {dd}"
        state = torch.randn((bs, heads, dd, pitch), generator=t.g, device=dev) / 16
        x, ld, o, beta = rnd(bs, 3 * n), -torch.exp(t.f32(bs, n) - 3), torch.empty((bs, n), dtype=torch.bfloat16, device=dev), rnd(bs, heads)
        conv = (t.f32(4, 3 * n), torch.zeros((bs, 4, 3 * n), dtype=torch.bfloat16, device=dev), (0, n, 2 * n))
        opts = dict(q_scale=dd ** -0.5, unit_eps=1e-6)
        like = f"decayed_recurrence channels {bs} sequences, {shape}"
        add("delta_rule", f"{bs} sequences, {shape}", lambda: graph_time(lambda i: op("delta_rule")(
            x[:, :n], x[:, n:2 * n], x[:, 2 * n:], o, state, sl, st, heads, heads, dd, dd, log_decay=ld, beta=beta, **opts), 6),
            nbytes=2.0 * bs * n * dd * 4 + bs * n * 12, like=like)
        add("delta_rule", f"{bs} sequences, {shape}, convolutions of 4", lambda: graph_time(lambda i: op("delta_rule")(
            x[:, :n], x[:, n:2 * n], x[:, 2 * n:], o, state, sl, st, heads, heads, dd, dd, log_decay=ld, beta=beta, conv=conv, **opts), 6),
            nbytes=2.0 * bs * n * dd * 4 + bs * n * (12 + 24), like=like)
        xs, ldT, oT, betas = rnd(T, 3 * n), -torch.exp(t.f32(T, n) - 3), torch.empty((T, n), dtype=torch.bfloat16, device=dev), rnd(T, heads)
        for nseq in (16, 1):
            cuts = [i32(v) for v in R.delta_cuts([T // nseq] * nseq, heads, dd)]
            cu, zero = i32(list(range(0, T + 1, T // nseq))), torch.zeros(nseq, dtype=torch.int32, device=dev)
            # least arithmetic at 16 tokens a chunk: the products inside it, the triangular system, state in and out and what a key finds there
            add("delta_chunks", f"{nseq} x {T // nseq}, {shape}", lambda: _events(lambda: op("delta_chunks")(
                xs[:, :n], xs[:, n:2 * n], xs[:, 2 * n:], oT, state, sl[:nseq], zero, heads, heads, dd, dd, *cuts, cu_seqlens=cu, log_decay=ldT, beta=betas, **opts), 20, 50),
                flops=T * heads * (17.0 * 4 * dd + 6.0 * dd * dd), nbytes=T * n * 12.0, like=f"channel_chunks {nseq} x {T // nseq}, {shape}")
        del xs, ldT, oT
        copies = R.matrix_memory_copies(dd)
        state, top = torch.randn((bs, heads, dd + copies, pitch), generator=t.g, device=dev), torch.zeros((bs, heads, copies), device=dev)
        bi, bf = t.f32(heads), t.f32(heads) + 3
        x, both = rnd(bs, 3 * n), rnd(bs, 2 * heads)
        memory = lambda g: R.MemoryGates(g[:, :heads], g[:, heads:], bi, bf, 15.0, top, dd ** -0.5)      # noqa: E731
        add("decayed_recurrence memory", f"{bs} sequences, {shape}", lambda: graph_time(lambda i: op("decayed_recurrence")(
            x[:, :n], x[:, n:2 * n], x[:, 2 * n:], o, state, sl, st, heads, heads, dd, dd, gates=memory(both)), 6),
            nbytes=2.0 * bs * n * dd * 4 + bs * n * 8, like="decayed_recurrence retention 256 sequences, 16 x 128 x 128")
        xs, boths, oT = rnd(T, 3 * n), rnd(T, 2 * heads), torch.empty((T, n), dtype=torch.bfloat16, device=dev)
        for nseq in (16, 1):
            segs, ends = (i32(v) for v in R.recurrence_segments([T // nseq] * nseq, heads, heads, dd))
            cu, zero = i32(list(range(0, T + 1, T // nseq))), torch.zeros(nseq, dtype=torch.int32, device=dev)
            add("decayed_chunks memory", f"{nseq} x {T // nseq}, {shape}", lambda: _events(lambda: op("decayed_chunks")(
                xs[:, :n], xs[:, n:2 * n], xs[:, 2 * n:], oT, state, sl[:nseq], zero, heads, heads, dd, dd, segs, ends, cu_seqlens=cu, gates=memory(boths)), 20, 50),
                flops=T * heads * (65.0 * 2 * dd + 4.0 * dd * dd), nbytes=T * n * 8.0, like=f"decayed_chunks retention {nseq} x {T // nseq}, 16 x 128 x 128")
        del xs, oT
    rank = 32
    z, w2, w0, rate = [rnd(T, rank) for _ in range(4)], rnd(1024, rank), t.f32(1024), -torch.exp(t.f32(16))
    add("low_rank_decay", f"{T} x {rank} -> 1024, rates", lambda: graph_time(lambda i: op("low_rank_decay")(z[i % 4], w2, w0, rate=rate), 4), nbytes=T * (rank * 2 + 1024 * 4.0),
        like=f"low_rank_decay {T} x {rank} -> 1024")
    y, gate, wn = [rnd(T, 1024) for _ in range(4)], [rnd(T, 1024) for _ in range(4)], rnd(64)
    add("gated_group_norm", f"{T} x 1024, 16 groups, sigmoid", lambda: graph_time(lambda i: op("gated_group_norm")(y[i % 4], gate[i % 4], 16, 1e-6, weight=wn, activation="sigmoid", scale=0.7), 8),
        nbytes=T * 1024 * 6.0, like=f"gated_group_norm {T} x 1024, 16 groups")


def fedovik_rows(t):
    add, rnd, i32, dev = _handles(t)
    halves = [rnd(T, 6144).chunk(2, dim=-1) for _ in range(4)]
    add("relu_glu", f"{T} x 3072", lambda: graph_time(lambda i: op("relu_glu")(*halves[i % 4]), 8), nbytes=T * 3072 * 6.0, like="siluAndMul")
    for rows, n in ((512, 4096), (T, 1024)):
        sets = 24 if rows == 512 else 4
        res, yy, w, b, shift = [t.f32(rows, n) for _ in range(sets)], [rnd(rows, n) for _ in range(sets)], rnd(n), rnd(n), t.f32(n)
        add("add_norm", f"{rows} x {n}, layer norms", lambda: graph_time(lambda i: op("add_norm")(res[i % sets], yy[i % sets], shift, False, w, b, 1e-6, center=True), 24 if rows == 512 else 8),
            nbytes=rows * n * 12.0, like=f"add_norm_norm {rows} x {n}, 1 part")


def fedovik_kernels(t):
    fedovik_attention(t)
    fedovik_recurrences(t)
    fedovik_rows(t)


def kernel_table(dev, seed=0, only="", design="nepulix"):
    """The rows of a design's kernels behind those of the models it is measured against."""
    t = KernelTable(dev, seed, only)
    qwen3_kernels(t)
    if design == "sozarax":
        decayed_kernels(t, "retention", 16, 16, 128, 128, True)
        sozarax_kernels(t)
    elif design == "lulizen":
        sozarax_attention(t)
        sozarax_experts(t)
        sozarax_residual(t)
        lulizen_kernels(t)
    elif design == "fedovik":
        decayed_kernels(t, "retention", 16, 16, 128, 128, True)
        sozarax_attention(t)
        time_mixing_kernels(t)
        sozarax_residual(t)
        fedovik_kernels(t)
    else:
        nepulix_kernels(t)
    return t.rows
