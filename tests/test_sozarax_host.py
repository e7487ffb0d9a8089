"""No GPU: the oracle of the Sozarax design against closed forms, and the host side of what runs it - configuration, registry,
layer order, weights whose sizes only the tensors tell, batch plans."""
import json
import math

import pytest
import torch

from nepulix_cases import write_checkpoint
from oracle import sozarax as O
from sozarax_cases import CONFIGS, attention, config, dense, moe, random_tokens, random_weights, tensor_shapes, wkv

D = torch.float64


# ------------------------------------------------------------------------------------------------ the oracle itself
def test_recurrence_equals_its_closed_form():
    g = torch.Generator().manual_seed(1)
    T, H, N, V = 9, 2, 3, 4
    r, k, v = (torch.randn((T, H, n), generator=g, dtype=D) for n in (N, N, V))
    w, u = torch.rand((T, H, N), generator=g, dtype=D), torch.randn((H, N), generator=g, dtype=D)
    o, S = O.channel_recurrence(r, k, v, w, u)
    for h in range(H):
        for t in range(T):
            # token s reaches token t through the decays strictly between them; t reaches itself through the bonus
            want = sum((r[t, h] * k[s, h] * w[s + 1:t, h].prod(0)).sum() * v[s, h] for s in range(t)) + (r[t, h] * u[h] * k[t, h]).sum() * v[t, h]
            assert torch.allclose(o[t, h], want)
    o1, S1 = O.channel_recurrence(r[:4], k[:4], v[:4], w[:4], u)
    o2, S2 = O.channel_recurrence(r[4:], k[4:], v[4:], w[4:], u, S1)
    assert torch.allclose(torch.cat((o1, o2)), o) and torch.allclose(S2, S)


def test_token_mix_and_decay():
    x = torch.tensor([[1.0, 10.0], [3.0, 30.0], [5.0, 50.0]], dtype=D)
    mu = torch.tensor([0.5, 1.0], dtype=D)
    assert torch.equal(O.token_mix(x, mu), torch.tensor([[0.5, 0.0], [2.0, 10.0], [4.0, 30.0]], dtype=D))
    assert torch.equal(O.token_mix(x[1:], mu, x[0]), O.token_mix(x, mu)[1:])
    w = O.channel_decay(torch.tensor([[0.3]], dtype=D), torch.eye(1, dtype=D), torch.tensor([[2.0]], dtype=D), torch.tensor([-1.0], dtype=D))
    assert math.isclose(w.item(), math.exp(-math.exp(2 * math.tanh(0.3) - 1)))


def test_attention_equals_a_plain_loop():
    g = torch.Generator().manual_seed(2)
    T, H, G, d, v = 7, 4, 2, 3, 5
    q, k, val = (torch.randn((T, n, s), generator=g, dtype=D) for n, s in ((H, d), (G, d), (G, v)))
    slopes = O.distance_slopes(H)
    assert slopes.tolist() == [2 ** -2.0, 2 ** -4.0, 2 ** -6.0, 2 ** -8.0]
    o = O.biased_attention(q, k, val, 0.7, slopes)
    for i in range(T):
        for h in range(H):
            s = [0.7 * float(q[i, h] @ k[j, h // 2]) - float(slopes[h]) * (i - j) for j in range(i + 1)]
            p = [math.exp(x) for x in s]
            want = sum(x * val[j, h // 2] for j, x in enumerate(p)) / sum(p)
            assert torch.allclose(o[i, h], want)
    t = O.query_temperature(torch.tensor([0, 2, 3, 6, 7]), 0.5, 4)      # steps where (p + 1) reaches a multiple of 4
    assert torch.allclose(t, 1 + 0.5 * torch.log(torch.tensor([1.0, 1, 2, 2, 3], dtype=D)))


def test_mixture_scales_the_input():
    g = torch.Generator().manual_seed(3)
    w = {"router": torch.tensor([[4.0, 0], [0, 4.0], [-1, -1]], dtype=D)}
    for e in range(3):
        w.update({f"e{e}.gate": torch.randn((3, 2), generator=g, dtype=D), f"e{e}.up": torch.randn((3, 2), generator=g, dtype=D), f"e{e}.down": torch.randn((2, 3), generator=g, dtype=D)})
    h = torch.tensor([[1.0, 0.5]], dtype=D)
    s = [1 / (1 + math.exp(-z)) for z in (4.0, 2.0)]
    run = lambda e, x: (O.silu(x @ w[f"e{e}.gate"].T) * (x @ w[f"e{e}.up"].T)) @ w[f"e{e}.down"].T      # noqa: E731
    for top, want in ((1, run(0, s[0] * h)), (2, run(0, s[0] * h) + run(1, s[1] * h))):
        assert torch.allclose(O.mixture(h, w, {"router": {"experts": 3, "top": top}}), want)
    assert torch.equal(O.squared_relu(torch.tensor([-2.0, 3.0])), torch.tensor([0.0, 9.0]))
    y = torch.tensor([[3.0, 4.0]], dtype=D)
    assert torch.allclose(O.unit_rms(y, 0.0), y / math.sqrt(12.5)) and torch.equal(O.unit_rms(y * 0, 1e-6), y * 0)


@pytest.mark.parametrize("name", ["odd", "ones"])
def test_oracle_is_causal_and_reads_every_tensor(name):
    cfg, w = CONFIGS[name], random_weights(name, 4)
    s = random_tokens(cfg, 24, 1)
    a = O.forward(cfg, w, s)
    b = O.forward(cfg, w, s[:10] + random_tokens(cfg, 14, 2))
    assert torch.allclose(a[:10], b[:10]) and not torch.allclose(a[10:], b[10:])
    assert a.shape == (24, cfg["vocab"])
    assert (O.forward(cfg, w, [(s[0] + 1) % cfg["vocab"]] + s[1:])[-1] - a[-1]).abs().max() > 1e-4      # the first token is not forgotten
    for n in w:
        if ".e" in n or n.endswith("router"):
            continue      # an expert may have no token
        changed = dict(w)
        changed[n] = (w[n].float() * 1.5 + 0.1).to(w[n].dtype)
        assert (O.forward(cfg, changed, s) - a).abs().max() > 1e-4, n


def test_a_loop_repeats_layers_with_a_state_of_its_own():
    cfg, w = CONFIGS["states"], random_weights("states", 1)
    assert O.layer_order(cfg) == [0, 1, 0, 1, 0, 1]
    unrolled = dict(cfg, layers=cfg["layers"] * 3, loop=None)
    w3 = {n: t for n, t in w.items() if n[0] != "l"}
    for i in range(6):
        w3.update({f"l{i}." + n.split(".", 1)[1]: t for n, t in w.items() if n.startswith(f"l{i % 2}.")})
    s = random_tokens(cfg, 12, 0)
    assert torch.equal(O.forward(cfg, w, s), O.forward(unrolled, w3, s))


# ------------------------------------------------------------------------------------------------ host side of the product
def test_registry_and_configuration(tmp_path, capsys):
    from nano_vllm_ninetoothed_amd.__main__ import main
    from nano_vllm_ninetoothed_amd.models import architectures, load_config, model_class
    from nano_vllm_ninetoothed_amd.models.sozarax import SozaraxConfig, SozaraxModel
    assert "Sozarax" in architectures()
    (tmp_path / "config.json").write_text(json.dumps(CONFIGS["odd"]))
    c = load_config(tmp_path)
    assert isinstance(c, SozaraxConfig) and (c.width, c.vocab, c.eps, c.embedding_scale, len(c.layers)) == (72, 101, 1e-5, 3.7, 4)
    assert model_class(c) is SozaraxModel and SozaraxModel.needs(c) == (True, True)
    for name, cfg in CONFIGS.items():
        c = SozaraxConfig.from_dict(cfg)
        assert c.order() == O.layer_order(cfg)
        assert SozaraxModel.needs(c) == (name != "states", name != "pages")
    without = {k: v for k, v in CONFIGS["odd"].items() if k != "loop"}
    assert SozaraxConfig.from_dict(without).order() == [0, 1, 2, 3] == SozaraxConfig.from_dict(dict(without, loop=None)).order()
    assert main(["models"]) == 0 and "Sozarax" in capsys.readouterr().out


@pytest.mark.parametrize("layer,mlp,change", [
    (wkv(2, 8, 4), None, {"heads": 0}), (wkv(2, 8, 4), None, {"dim": "8"}), (attention(4, 2, 8, 8, 0.1, 4), None, {"kv_heads": 3}),
    (attention(4, 2, 8, 8, 0.1, 4), None, {"vdim": -1}), (attention(4, 2, 8, 8, 0.1, 4), None, {"q_temp": {"coef": 0.1, "every": 0}}),
    (wkv(2, 8, 4), moe(8, 2, 3), None), (wkv(2, 8, 4), moe(0, 2, 1), None), (wkv(2, 8, 4), dense(0), None), (wkv(2, 8, 4), {"kind": "other", "ff": 8}, None)])
def test_configurations_that_make_no_sense_are_refused(layer, mlp, change):
    from nano_vllm_ninetoothed_amd.models.sozarax import SozaraxConfig
    SozaraxConfig.from_dict(config(16, 16, [layer], [None], (0, 0, 1), 1.0)[0])
    bad = dict(layer, mixer={**layer["mixer"], **(change or {})})
    with pytest.raises(ValueError):
        SozaraxConfig.from_dict(config(16, 16, [bad], [mlp], (0, 0, 1), 1.0)[0])


@pytest.mark.parametrize("loop", [(0, 2, 1), (1, 0, 1), (0, 1, 0), (-1, 1, 2)])
def test_loops_that_make_no_sense_are_refused(loop):
    from nano_vllm_ninetoothed_amd.models.sozarax import SozaraxConfig
    with pytest.raises(ValueError):
        SozaraxConfig.from_dict(config(16, 16, [wkv(2, 8, 4)], [None], loop, 1.0)[0])


def test_shapes_that_only_the_tensors_tell(tmp_path):
    from nano_vllm_ninetoothed_amd.weights import CheckpointWeights, RandomWeights, TensorWeights
    w = random_weights("odd", 0)
    assert {n: tuple(t.shape) for n, t in w.items()} == tensor_shapes("odd")
    write_checkpoint(tmp_path / "m", CONFIGS["odd"], w)
    for source in (CheckpointWeights(tmp_path / "m", torch.float32, "cpu"), TensorWeights(w, torch.float32, "cpu")):
        assert source.shape_of("l1.mix.w1") == (5, 72)
        assert torch.equal(source.take("l1.mix.w1", (5, 72)), w["l1.mix.w1"].float())
        with pytest.raises(KeyError):
            source.shape_of("l0.mix.w1")
    assert RandomWeights(0, torch.float32, "cpu").shape_of("l1.mix.w1") is None


def test_position_steps_and_slopes():
    from nano_vllm_ninetoothed_amd.layers import Rotary
    from nano_vllm_ninetoothed_amd.layers.biased_attention import distance_slopes
    r = Rotary(1000, "cpu")
    assert r.steps(0.3, 7) is r.steps(0.3, 7) and r.steps(0.3, 7) is not r.steps(0.3, 8)
    assert torch.equal(r.steps(0.3, 7), O.query_temperature(torch.arange(1000), 0.3, 7).float())
    for h in (1, 3, 12, 32):
        assert torch.equal(distance_slopes(h), O.distance_slopes(h).float())


def test_plans():
    from nano_vllm_ninetoothed_amd.layers.biased_attention import LONG_PORTION, BiasedAttention
    from nano_vllm_ninetoothed_amd.mops.hip.attention_ops import biased_prefill_tiles
    from nano_vllm_ninetoothed_amd.mops.hip.recurrent_ops import channel_segments
    tiles = biased_prefill_tiles([130, 64], [0, 100], 5, 2)
    assert sorted(tiles) == [(5, 128, 0, 2, 130), (133, 2, 128, 2, 130), (135, 64, 100, 3, 164)] and tiles[0] == (135, 64, 100, 3, 164)
    ctx = {"is_prefill": True, "seq_counts": [1, 1, LONG_PORTION - 1, LONG_PORTION, 300], "seq_starts": [9, 4, 0, 3, 0]}
    first, t = BiasedAttention._plan(ctx, "cpu")
    assert first == LONG_PORTION + 1 and t.shape == (4, 5) and BiasedAttention._plan(ctx, "cpu")[1] is t
    assert BiasedAttention._plan({"is_prefill": True, "seq_counts": [1, 5], "seq_starts": [3, 0]}, "cpu") is None
    assert BiasedAttention._plan({"is_prefill": False}, "cpu") is None
    for counts in ([5, 2000, 40], [10], [700] * 300):
        segments, ends = channel_segments(counts, 4, 64)
        at = 0
        for i, n in enumerate(counts):      # the segments of a portion follow each other and cover it
            mine = segments[ends[i]:ends[i + 1]]
            assert all(s[0] == i for s in mine) and mine[0][1] == at and mine[-1][2] == at + n and all(a[2] == b[1] for a, b in zip(mine, mine[1:]))
            at += n
    assert len(channel_segments([2000], 4, 64)[0]) > 1 and len(channel_segments([700] * 300, 4, 64)[0]) == 300


def test_a_mixer_again_shares_weights_but_not_state():
    from nano_vllm_ninetoothed_amd.layers import Mixer

    class Counter(Mixer):
        def __init__(self, cache):
            self.weight = object()
            self.allocate(cache)

        def allocate(self, cache):
            self.state = cache.per_slot(3)

    from nano_vllm_ninetoothed_amd.cache import CacheManager
    c = CacheManager(1, 32, 2, "cpu", pages=False, slots=True)
    a = Counter(c)
    b = a.again(c)
    assert a.weight is b.weight and a.state.data_ptr() != b.state.data_ptr() and b.state.shape == (2, 3)


def test_argument_validation_on_the_host():
    """The C ABI refuses what the kernels do not cover before any launch."""
    from ctypes import byref
    from nano_vllm_ninetoothed_amd import _capi
    if not _capi.LIB_PATH.exists():
        from nano_vllm_ninetoothed_amd import build
        build.build(force=False)
    lib, A = _capi.load(), 0x1000
    assert lib.mops_hip_token_mix(A, 64, A, 5, A, 4, A, None, A, A, A, 0, 3, 64, None) == -1      # token_seq without cu_seqlens
    assert lib.mops_hip_token_mix(A, 32, A, 5, A, 4, None, None, A, A, A, 0, 3, 64, None) == -1   # rows overlap
    assert lib.mops_hip_token_mix(None, 64, None, 5, None, 4, None, None, None, None, None, 0, 0, 64, None) == 0
    assert lib.mops_hip_low_rank_decay(A, 8, A, A, None, 0, A, 0, 3, 64, 16, None) == -1
    assert lib.mops_hip_low_rank_decay(A, 5000, A, A, None, 0, A, 0, 3, 64, 5000, None) == -2
    assert lib.mops_hip_add_norm_norm(A, A, 64, 1, None, A, A, 1e-5, 0, A, 0, 4, 64, None) == -1           # out aliases y
    assert lib.mops_hip_squared_relu(A, 8, A, 0, 4, 64, None) == -1
    m = _capi.Moe()
    m.rows = m.tiles = m.score = A
    m.tokens, m.experts, m.top, m.width, m.ff, m.block_rows, m.dtype = 4, 8, 2, 64, 32, 32, 0
    assert lib.mops_hip_moe_down(A, 32, A, 16, A, 64, byref(m), None) == -1                       # depth below ff
    m.top = 9
    assert lib.mops_hip_moe_gate_up(A, 64, A, 32, A, 32, byref(m), None) == -1
    m.top, m.experts = 2, 2000
    assert lib.mops_hip_moe_gate_up(A, 64, A, 32, A, 32, byref(m), None) == -2
    m.experts, m.block_rows, m.dtype = 8, 128, 1
    assert lib.mops_hip_moe_gate_up(A, 64, A, 32, A, 32, byref(m), None) == -1                    # large blocks are bf16
    assert lib.mops_hip_moe_max_tiles(100, 8, 2, 32) == 6 + 8 and lib.mops_hip_moe_max_tiles(1, 8, 2, 32) == 2
    assert lib.mops_hip_grouped_linear(A, A, A, A, None, 8, 4, 3, 64, 64, None) == -1
    b = _capi.BiasedAttention()
    b.q = b.k_pages = b.v_pages = b.context_lens = b.block_table = b.out = A
    b.block_table_stride, b.block_size, b.num_blocks, b.max_blocks = 4, 32, 8, 4
    b.rows, b.heads, b.kv_heads, b.dim, b.vdim, b.scale, b.dtype = 2, 4, 2, 64, 64, 1.0, 0
    assert lib.mops_hip_biased_decode(byref(b), None, 0, None) == -4
    b.dim = 300
    assert lib.mops_hip_biased_decode(byref(b), A, 1 << 30, None) == -2
    b.dim, b.block_size = 64, 24
    assert lib.mops_hip_biased_decode(byref(b), A, 1 << 30, None) == -2
    b.kv_heads = 3
    assert lib.mops_hip_biased_attention_rows(byref(b), None) == -1
