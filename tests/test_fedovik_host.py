"""No GPU: the oracle of the Fedovik design against closed forms, mistakes planted in it that must show, and the host side of what
runs the design - configuration, registry, passes, plans, argument checks."""
import json
import math

import pytest
import torch

from fedovik_cases import CONFIGS, attention, config, memory, parallel, random_tokens, random_weights, tensor_shapes
from nepulix_cases import logit_error, write_checkpoint
from oracle import fedovik as O

D = torch.float64


# ------------------------------------------------------------------------------------------------ the oracle itself
def test_delta_rule_writes_what_is_missing():
    """Without decay and with full strength a key reads back the value last written under it, and orthogonal keys do not touch it."""
    eye = torch.eye(4, dtype=D)
    k = torch.stack([eye[0], eye[1], eye[0], eye[2]])[:, None]
    v = torch.randn((4, 1, 3), generator=torch.Generator().manual_seed(0), dtype=D)
    ones = torch.ones((4, 1, 4), dtype=D)
    q = torch.stack([eye[0], eye[0], eye[0], eye[1]])[:, None]
    o, S = O.delta_rule(q, k, v, ones, torch.ones((4, 1), dtype=D))
    assert torch.allclose(o[:, 0], torch.stack([v[0, 0], v[0, 0], v[2, 0], v[1, 0]])) and torch.allclose(S[0, 2], v[3, 0])
    half, _ = O.delta_rule(q, k, v, ones, torch.full((4, 1), 0.5, dtype=D))
    assert torch.allclose(half[2, 0], 0.25 * v[0, 0] + 0.5 * v[2, 0])


def test_delta_rule_equals_its_matrix_form_and_can_be_cut():
    g = torch.Generator().manual_seed(1)
    T, H, G, N, V = 9, 4, 2, 3, 5
    q, k = (O.unit(torch.randn((T, G, N), generator=g, dtype=D)) for _ in range(2))
    v, a, b = torch.randn((T, H, V), generator=g, dtype=D), torch.rand((T, H, N), generator=g, dtype=D), torch.rand((T, H), generator=g, dtype=D)
    o, S = O.delta_rule(q, k, v, a, b)
    for h in range(H):
        M = torch.zeros((N, V), dtype=D)
        for t in range(T):
            kk = k[t, h // 2][:, None]
            M = (torch.eye(N, dtype=D) - b[t, h] * kk @ kk.T) @ torch.diag(a[t, h]) @ M + b[t, h] * kk @ v[t, h][None]
            assert torch.allclose(o[t, h], M.T @ q[t, h // 2])
    o1, S1 = O.delta_rule(q[:4], k[:4], v[:4], a[:4], b[:4])
    o2, S2 = O.delta_rule(q[4:], k[4:], v[4:], a[4:], b[4:], S1)
    assert torch.allclose(torch.cat((o1, o2)), o) and torch.allclose(S2, S)


def test_matrix_memory_equals_its_form_without_a_running_maximum():
    g = torch.Generator().manual_seed(2)
    T, H, N, V = 12, 2, 3, 4
    q, k, v = (torch.randn((T, H, n), generator=g, dtype=D) for n in (N, N, V))
    i, f = O.log_gates(4 * torch.randn((T, H), generator=g, dtype=D), 4 * torch.randn((T, H), generator=g, dtype=D), 3.0)
    assert i.abs().max() < 3 and f.max() < 0 and f.min() > -3.1
    o, (S, n, m) = O.matrix_memory(q, k, v, i, f)
    plain, norm, top = torch.zeros((H, N, V), dtype=D), torch.zeros((H, N), dtype=D), torch.zeros(H, dtype=D)
    for t in range(T):
        plain = f[t].exp()[:, None, None] * plain + i[t].exp()[:, None, None] * k[t][:, :, None] * v[t][:, None]
        norm = f[t].exp()[:, None] * norm + i[t].exp()[:, None] * k[t]
        top = torch.maximum(top + f[t], i[t])
        den = torch.maximum((norm * q[t]).sum(-1).abs(), torch.ones(H, dtype=D)) + 1e-6 * top.exp()
        assert torch.allclose(o[t], torch.einsum("hdv,hd->hv", plain, q[t]) / den[:, None])
    assert torch.allclose(S, plain * (-top).exp()[:, None, None]) and torch.allclose(n, norm * (-top).exp()[:, None]) and torch.allclose(m, top)
    o1, s1 = O.matrix_memory(q[:5], k[:5], v[:5], i[:5], f[:5])
    o2, _ = O.matrix_memory(q[5:], k[5:], v[5:], i[5:], f[5:], s1)
    assert torch.allclose(torch.cat((o1, o2)), o)


def test_attention_weights_by_hand():
    s = torch.tensor([[[0.3, 9.0, 9.0], [0.1, -0.4, 9.0], [2.0, 0.0, 1.0]]], dtype=D)
    sig = lambda x: 1 / (1 + math.exp(-x))      # noqa: E731
    w = O.sigmoid_weights(s, torch.tensor([0.5], dtype=D))[0]
    assert torch.allclose(w, torch.tensor([[sig(0.8), 0, 0], [sig(0.6), sig(0.1), 0], [sig(2.5), sig(0.5), sig(1.5)]], dtype=D))
    for window in (2, 3):
        w = O.log_distance_weights(s, torch.tensor([0.7], dtype=D), torch.tensor([2.0], dtype=D), window)[0]
        e = [math.exp(2.0 - 0.7 * math.log(5)) if window == 3 else 0.0, math.exp(-0.7 * math.log(3)), math.exp(1.0)]
        assert torch.allclose(w[2], torch.tensor([x / sum(e) for x in e], dtype=D)) and w[0].tolist() == [1, 0, 0]


def test_rotation_of_neighbours_is_a_complex_product():
    x = torch.randn((5, 2, 9), generator=torch.Generator().manual_seed(3), dtype=D)
    y = O.rotate_neighbours(x, torch.tensor([0, 1, 7, 100, 5000]), 1e3, 6)
    for t, p in enumerate((0, 1, 7, 100, 5000)):
        for i in range(3):
            z = torch.complex(x[t, :, 2 * i], x[t, :, 2 * i + 1]) * torch.exp(torch.tensor(1j * p * 1e3 ** (-2 * i / 6), dtype=torch.complex128))
            assert torch.allclose(y[t, :, 2 * i], z.real) and torch.allclose(y[t, :, 2 * i + 1], z.imag)
    assert torch.equal(y[..., 6:], x[..., 6:])


def test_short_convolution_and_decays():
    x, w = torch.arange(1.0, 7.0, dtype=D)[:, None], torch.tensor([[100.0, 10.0, 1.0]], dtype=D)
    assert torch.allclose(O.short_convolution(x, w)[:, 0], O.silu(torch.tensor([1.0, 12.0, 123.0, 234.0, 345.0, 456.0], dtype=D)))
    d = O.channel_decays(torch.tensor([[0.3, -2.0]], dtype=D), torch.tensor([0.5], dtype=D), torch.tensor([0.1, 0.2], dtype=D), 1)
    assert torch.allclose(d[0, 0], torch.tensor([math.exp(-math.exp(0.5) * math.log1p(math.exp(x))) for x in (0.4, -1.8)], dtype=D))


@pytest.mark.parametrize("name", ["odd", "plain"])
def test_logits_depend_on_earlier_tokens_only(name):
    cfg, w = CONFIGS[name], random_weights(CONFIGS[name], 1)
    s = random_tokens(cfg, 40, 2)
    other = s[:25] + [(t + 1) % cfg["vocab"] for t in s[25:]]
    a, b = O.forward(cfg, w, s), O.forward(cfg, w, other)
    assert torch.equal(a[:25], b[:25]) and (a[25:] - b[25:]).abs().max() > 0.1


def test_passes_of_a_loop():
    assert O.passes(CONFIGS["odd"]) == [(0, None), (1, 0), (2, None), (1, 1), (2, None), (1, 2), (2, None), (3, None)]
    cfg, w = CONFIGS["odd"], random_weights(CONFIGS["odd"], 1)
    layers = []
    O.forward(cfg, w, [1, 2, 3], layers_out=layers)
    assert len(layers) == 8
    # one pass by hand: the entry, then the layers as in a model without a loop
    once = dict(cfg, loop={"start": 0, "stop": 4, "times": 1})
    x0 = w["embed"].double()[[1, 2, 3]] * cfg["embedding"]["scale"]
    entered = torch.cat((x0, x0), -1) @ w["loop.in"].double().T + w["loop.step"].double()[0]
    h = O.layer_norm(entered, w["l0.norm1"].double(), w["l0.norm1.b"].double(), cfg["norm"]["eps"])
    first = entered + O.sigmoid_attention(h, O._under(w, "l0.mix.", D), cfg["layers"][0]["mixer"], 1e-5) + O.dense(h, O._under(w, "l0.mlp.", D))
    layers = []
    O.forward(once, w, [1, 2, 3], layers_out=layers)
    assert torch.allclose(layers[0], first)


# --------------------------------------------------------------------------------------------- planted mistakes that must show
def planted(monkeypatch, name):
    """One mistake in the oracle."""
    def wrap(function, make):
        monkeypatch.setattr(O, function, make(getattr(O, function)))
    {"a window one token too wide": lambda: wrap("log_distance_weights", lambda f: lambda s, a, b, n: f(s, a, b, n + 1)),
     "a window one token too narrow": lambda: wrap("log_distance_weights", lambda f: lambda s, a, b, n: f(s, a, b, max(1, n - 1))),
     "no distance bias": lambda: wrap("log_distance_weights", lambda f: lambda s, a, b, n: f(s, 0 * a, b, n)),
     "a distance counted from one": lambda: wrap("distances", lambda f: lambda n: f(n) + (f(n) >= 0)),
     "no number per head": lambda: wrap("sigmoid_weights", lambda f: lambda s, b: f(s, 0 * b)),
     "normalised weights": lambda: wrap("sigmoid_weights", lambda f: lambda s, b: f(s, b) / f(s, b).sum(-1, keepdim=True)),
     "pairs half a rotation apart": lambda: monkeypatch.setattr(O, "rotate_neighbours", rotate_halves),
     "no projection biases": lambda: monkeypatch.setattr(O, "biased_product", lambda h, w, n: O.product(h, w[n])),
     "a read in front of the write": lambda: wrap("delta_rule", early_read),
     "a decay behind the write": lambda: wrap("delta_rule", lambda f: lambda q, k, v, g, b: f(q, k, v, torch.cat((torch.ones_like(g[:1]), g[:-1])), b)),
     "queries and keys as they come": lambda: monkeypatch.setattr(O, "unit", lambda x: x),
     "taps in the other order": lambda: wrap("short_convolution", lambda f: lambda x, w: f(x, w.flip(1))),
     "a state lost after 30 tokens": lambda: (wrap("delta_rule", lost), wrap("matrix_memory", lost)),
     "gates without a cap": lambda: monkeypatch.setattr(O, "capped", lambda x, cap: x),
     "one layer norm too plain": lambda: monkeypatch.setattr(O, "layer_norm", lambda x, w, b, eps: O.over_rms(x, eps) * w + b),
     "a linear feed-forward gate": lambda: monkeypatch.setattr(O, "dense", lambda h, w: O.product(O.product(h, w["gate"]) * O.product(h, w["up"]), w["down"]))}[name]()


def rotate_halves(x, positions, base, dims):
    order = [i // 2 + dims // 2 * (i % 2) for i in range(dims)]
    back = [order.index(i) for i in range(dims)]
    y = ROTATE(torch.cat((x[..., order], x[..., dims:]), -1), positions, base, dims)
    return torch.cat((y[..., back], y[..., dims:]), -1)


ROTATE = O.rotate_neighbours


def early_read(f):
    def rule(q, k, v, g, beta):
        o, S = f(q, k, v, g, beta)
        own = beta[..., None] * (v - f(k, k, v, g, beta)[0])       # close to what the current token adds
        return o - (q * k).sum(-1).repeat_interleave(v.shape[1] // q.shape[1], dim=1)[..., None] * own, S
    return rule


def lost(f):
    def rule(*args):
        n = 30
        parts = [f(*(a[i:i + n] for a in args)) for i in range(0, args[0].shape[0], n)]
        return torch.cat([p[0] for p in parts]), parts[-1][1]
    return rule


MISTAKES = {"odd": ["a window one token too wide", "a window one token too narrow", "no distance bias", "a distance counted from one", "no number per head",
                    "normalised weights", "pairs half a rotation apart", "no projection biases", "a read in front of the write", "a decay behind the write",
                    "queries and keys as they come", "taps in the other order", "a state lost after 30 tokens", "gates without a cap", "one layer norm too plain",
                    "a linear feed-forward gate"],
            "plain": ["a window one token too wide", "a state lost after 30 tokens", "a read in front of the write"]}


@pytest.mark.parametrize("name,mistake", [(n, m) for n, ms in MISTAKES.items() for m in ms])
def test_a_planted_mistake_shows_in_the_logits(monkeypatch, name, mistake):
    """It moves some positions by far more than what rounding alone does, and nearly every mistake most of them."""
    cfg = CONFIGS[name]
    w = random_weights(cfg, 11)
    s = random_tokens(cfg, 97, 101)
    want = O.forward(cfg, w, s)
    with O.sixteen_bit_products(1):
        noise = logit_error(O.forward(cfg, w, s), want)
    planted(monkeypatch, mistake)
    moved = logit_error(O.forward(cfg, w, s), want)
    assert moved.max() > 3 * noise.quantile(0.95), (moved.max(), noise.max())


@pytest.mark.parametrize("name,change", [("odd", "loop.step"), ("odd", "l0.mix.o.b"), ("odd", "l2.mix.left.r2"), ("odd", "final.norm.b"), ("odd", "l1.norm1.b"),
                                         ("plain", "l1.mix.right.dt_bias"), ("plain", "l2.mix.f.b"), ("plain", "l2.mix.i"), ("odd", "l3.mix.i"), ("plain", "l0.mix.pb")])
def test_every_small_tensor_matters(name, change):
    cfg = CONFIGS[name]
    w = random_weights(cfg, 11)
    s = random_tokens(cfg, 60, 101)
    want = O.forward(cfg, w, s)
    assert logit_error(O.forward(cfg, dict(w, **{change: w[change] * 0}), s), want).median() > 0.01


# --------------------------------------------------------------------------------------------------- configuration and weights
def made(cfg):
    from nano_vllm_ninetoothed_amd.models import parse_config
    return parse_config(cfg)


def test_configuration_and_registry(tmp_path):
    from nano_vllm_ninetoothed_amd.models import architectures, load_config, model_class
    assert "Fedovik" in architectures()
    write_checkpoint(tmp_path, CONFIGS["odd"], random_weights(CONFIGS["odd"]))
    c = load_config(tmp_path)
    assert type(c).__name__ == "FedovikConfig" and c.width == 76 and c.embedding_scale == 1.5 and c.loop == (1, 3, 3)
    assert c.order() == [0, 1, 2, 1, 2, 1, 2, 3] and c.passes() == {1: 0, 3: 1, 5: 2}
    cls = model_class(c)
    assert cls.dtypes == (torch.bfloat16, torch.float32) and cls.needs(c) == (True, True)
    assert cls.needs(made(config(64, 64, [(memory(1, 8, 8), None)]))) == (False, True)
    assert cls.needs(made(config(64, 64, [(attention(1, 1, 8, 8, 8, 1.0), 8)]))) == (True, False)
    for name, cfg in CONFIGS.items():
        c = made(json.loads(json.dumps(cfg)))
        assert c.order() == [i for i, _ in O.passes(cfg)], name
        assert c.passes() == {at: t for at, (_, t) in enumerate(O.passes(cfg)) if t is not None}, name
    assert made(CONFIGS["plain"]).passes() == {}


def test_unusable_configurations_are_refused():
    def broken(change, name="odd"):
        cfg = json.loads(json.dumps(CONFIGS[name]))
        change(cfg)
        return cfg

    def put(*path, to):
        def change(cfg):
            for p in path[:-1]:
                cfg = cfg[p]
            cfg[path[-1]] = to
        return change

    mixer = lambda i, *path, to: put("layers", i, "mixer", *path, to=to)      # noqa: E731
    for change in (put("layers", 0, "type", to="retention"), put("layers", 0, "mlp", "kind", to="moe"), put("layers", 0, "mlp", "ff", to=0), mixer(0, "kv_heads", to=4),
                   mixer(0, "rot", "dims", to=15), mixer(0, "rot", "dims", to=24), mixer(1, "gate_cap", to=0.0), mixer(1, "heads", to=True), mixer(2, "left", "mask", "size", to=0),
                   mixer(2, "right", "kv_heads", to=4), mixer(2, "right", "conv", to=0), put("loop", "stop", to=5), put("loop", "times", to=0), put("loop", "start", to=4)):
        with pytest.raises(ValueError):
            made(broken(change))


def test_plans():
    from nano_vllm_ninetoothed_amd.mops.hip.recurrent_ops import delta_cuts
    chunks, segments, ends = delta_cuts([5, 16, 33, 1], 4, 64)
    assert chunks == [(0, 5), (5, 16), (21, 16), (37, 16), (53, 1), (54, 1)] and ends == [0, 1, 2, 3, 4]
    assert segments == [(0, 0, 5, 0), (1, 5, 21, 1), (2, 21, 54, 2), (3, 54, 55, 5)]
    for counts in ([5, 2000, 40], [10], [700] * 300, [1111, 2]):
        chunks, segments, ends = delta_cuts(counts, 4, 64)
        at = 0
        for i, n in enumerate(counts):      # the segments of a portion follow each other, begin with a chunk and cover it
            mine = segments[ends[i]:ends[i + 1]]
            assert all(s[0] == i and chunks[s[3]][0] == s[1] for s in mine) and mine[0][1] == at and mine[-1][2] == at + n
            assert all(a[2] == b[1] for a, b in zip(mine, mine[1:]))
            at += n
        assert sum(n for _, n in chunks) == sum(counts)
    assert len(delta_cuts([2000], 4, 64)[1]) > 1 and len(delta_cuts([700] * 300, 4, 64)[1]) == 300


class Numbers:
    """Stands for the device operators of sublayers on the CPU."""

    @staticmethod
    def linear(x, w, bias=None):
        return torch.nn.functional.linear(x, w, bias)


def test_joined_sublayers_equal_their_sum(monkeypatch):
    """Paddings, factors, biases, parts inside parts; a part again keeps the weights."""
    from nano_vllm_ninetoothed_amd.layers import Mixer, joined
    monkeypatch.setattr(joined, "hip_op", lambda name: getattr(Numbers, name))
    g = torch.Generator().manual_seed(0)
    rnd = lambda *s: torch.randn(s, generator=g, dtype=D)      # noqa: E731

    class Part(joined.TwoProducts, Mixer):
        def __init__(self, n, inner, bias):
            self.into, self.out_of = [rnd(n, 12), rnd(inner, 12)], rnd(12, inner)
            self.products(self.into, self.out_of, rnd(12) if bias else None)
            self.bias_kept = self.bias
            self.allocate(None)

        def allocate(self, cache):
            self.calls = []

        def mix(self, p, ctx, out, scale=1.0):
            self.calls.append(ctx)
            a, b = self.parts_of(p)
            out.copy_(scale * (b + a.sum(-1, keepdim=True)))

        def plain(self, x):
            a, b = (x @ w.T for w in self.into)
            y = (b + a.sum(-1, keepdim=True)) @ self.out_of.T
            return y if self.bias_kept is None else y + self.bias_kept

    x = rnd(5, 12)
    single = Part(3, 9, True)
    assert torch.allclose(single(x), single.plain(x))
    parts = [Part(3, 9, True), Part(8, 16, False), Part(5, 1, True)]
    inner = joined.Joined(parts[:2], (0.5, -2.0))
    outer = joined.Joined([inner, parts[2]])
    want = 0.5 * parts[0].plain(x) - 2.0 * parts[1].plain(x) + parts[2].plain(x)
    assert outer.padded and torch.allclose(outer(x), want) and outer.bias.dtype == torch.float32
    again = outer.again(None)
    assert torch.allclose(again(x), want) and again.w_in is outer.w_in and again.w_out is outer.w_out
    assert again.parts[1] is not outer.parts[1] and again.parts[0].parts[0] is not inner.parts[0]
    assert not joined.Joined([Part(8, 16, False)]).padded


def test_argument_validation_on_the_host():
    """The C ABI refuses what the kernels do not cover before any launch."""
    from ctypes import byref
    from nano_vllm_ninetoothed_amd import _capi
    if not _capi.LIB_PATH.exists():
        from nano_vllm_ninetoothed_amd import build
        build.build(force=False)
    lib, A = _capi.load(), 0x1000
    d = _capi.Delta()
    assert lib.mops_hip_delta_rule(None, None) == -1 and lib.mops_hip_delta_rule(byref(d), None) == 0      # no sequences: nothing to do
    for n in ("q", "k", "v", "out", "state", "state_slots", "starts", "log_decay", "beta"):
        setattr(d, n, A)
    d.batch, d.heads, d.groups, d.d, d.vd, d.num_slots, d.dtype = 2, 4, 2, 32, 16, 4, 0
    d.q_stride = d.k_stride = 64
    d.v_stride = d.out_stride = 64
    d.log_decay_stride, d.beta_stride = 128, 4
    assert lib.mops_hip_delta_chunks(byref(d), A, 3, A, 2, A, A, 1 << 30, None) == -1              # no cu_seqlens
    d.cu_seqlens = A
    assert lib.mops_hip_delta_chunks(byref(d), A, 3, A, 2, A, A, 100, None) == -4 and lib.mops_hip_delta_chunks(byref(d), A, 0, A, 0, A, None, 0, None) == 0
    d.beta_stride = 3
    assert lib.mops_hip_delta_rule(byref(d), None) == -1
    d.beta_stride, d.groups = 4, 3
    assert lib.mops_hip_delta_rule(byref(d), None) == -1
    d.groups, d.d, d.q_stride, d.k_stride, d.log_decay_stride = 2, 600, 1200, 1200, 2400
    assert lib.mops_hip_delta_rule(byref(d), None) == -2
    d.d, d.dtype = 300, 0
    assert lib.mops_hip_delta_chunks(byref(d), A, 3, A, 2, A, A, 1 << 30, None) == -2
    assert lib.mops_hip_delta_chunks_workspace_bytes(0, 1, 1, 4, 64, 48) == 0
    assert lib.mops_hip_delta_chunks_workspace_bytes(2, 1, 1, 4, 64, 48) == 8 * (14 * 1024 + 256)
    assert lib.mops_hip_delta_chunks_workspace_bytes(2, 2, 1, 4, 64, 48) == 8 * (14 * 1024 + 256 + 16 * 1024 + 48 * 64 * 4)
    assert lib.mops_hip_matrix_memory_copies(64) == 1 and lib.mops_hip_matrix_memory_copies(65) == 2
    r = _capi.Recurrence()
    for n in ("q", "k", "v", "out", "state", "state_slots", "starts", "input_gate"):
        setattr(r, n, A)
    r.batch, r.heads, r.groups, r.d, r.vd, r.num_slots, r.dtype = 1, 2, 2, 16, 16, 2, 0
    r.q_stride = r.k_stride = r.v_stride = r.out_stride = 32
    assert lib.mops_hip_decayed_recurrence(byref(r), None) == -1                                  # gates without biases and a maximum
    assert lib.mops_hip_matrix_memory_gates(byref(r), A, A, A, None) == -1
    n = _capi.AddNorm()
    n.residual, n.rows, n.n, n.replace = A, 2, 64, 1
    assert lib.mops_hip_add_norm(byref(n), None) == -1                                            # nothing to replace the residual with
    n.replace, n.b = 0, A
    assert lib.mops_hip_add_norm(byref(n), None) == -1                                            # a bias without a weight
    b = _capi.BiasedAttention()
    b.q = b.k_pages = b.v_pages = b.context_lens = b.block_table = b.out = A
    b.block_table_stride, b.block_size, b.num_blocks, b.max_blocks = 4, 32, 8, 4
    b.rows, b.heads, b.kv_heads, b.dim, b.vdim, b.scale, b.dtype = 2, 4, 2, 64, 64, 1.0, 0
    b.log_rate = A
    assert lib.mops_hip_biased_attention_rows(byref(b), None) == -1                               # a rate without a step
    b.log_step, b.weight_bias = A, A
    assert lib.mops_hip_biased_attention_rows(byref(b), None) == -1                               # two kinds of scores
    b.log_rate = b.log_step = None
    b.sinks = A
    assert lib.mops_hip_biased_decode(byref(b), None, 0, None) == -1                              # a sink without a softmax
    b.sinks, b.gate, b.gate_each, b.gate_stride = None, A, 1, 255
    assert lib.mops_hip_biased_decode(byref(b), None, 0, None) == -1
    b.gate_stride, b.out_stride = 256, 255
    assert lib.mops_hip_biased_decode(byref(b), None, 0, None) == -1
    assert lib.mops_hip_relu_glu(A, 32, A, 64, A, 64, 0, 4, 64, None) == -1
    assert lib.mops_hip_gated_group_norm(A, 64, A, 64, A, 0, 1e-5, 0, 1, 1.0, A + 64, 63, 0, 4, 2, 32, None) == -1


def test_tensor_names_of_a_configuration():
    """The model asks for exactly the tensors of a checkpoint."""
    names = set(tensor_shapes(CONFIGS["odd"]))
    assert {"l2.mix.left.r1", "l2.mix.right.g2", "l1.mix.i.b", "l0.mix.pb", "loop.step", "final.norm.b", "l3.norm1.b"} <= names
    assert "l1.mlp.gate" not in names and "loop.in" not in tensor_shapes(CONFIGS["plain"])
    assert parallel((1, 1, 8, 8, 3, 1.0), (1, 1, 8, 8, 4), 1.0, 2.0)["mixer"]["left"]["mask"]["size"] == 3
