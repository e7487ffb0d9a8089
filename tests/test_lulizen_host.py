"""No GPU: the oracle of the Lulizen design against closed forms, and the host side of what runs it - configuration, registry,
layer order, weights, argument checks."""
import json
import math

import pytest
import torch

from lulizen_cases import CONFIGS, chunked, config, dense, moe, random_tokens, random_weights, settled_tokens, tensor_shapes, windowed
from nepulix_cases import write_checkpoint
from oracle import lulizen as O

D = torch.float64


# ------------------------------------------------------------------------------------------------ the oracle itself
def test_norms():
    x, w = torch.tensor([[1.0, 2.0, 6.0]], dtype=D), torch.tensor([1.0, 2.0, -1.0], dtype=D)
    assert torch.allclose(O.layer_norm(x, w, 0.0), torch.tensor([[-2.0, -1.0, 3.0]], dtype=D) / math.sqrt(14 / 3) * w)
    assert torch.allclose(O.rms_norm(x, w, 0.0), x / math.sqrt(41 / 3) * w)
    same = torch.full((1, 4), 7.0, dtype=D)
    assert torch.equal(O.layer_norm(same, torch.ones(4, dtype=D), 1e-6), torch.zeros((1, 4), dtype=D))
    assert torch.allclose(O.rms_norm(torch.zeros((1, 3), dtype=D) + 1e-3, torch.ones(3, dtype=D), 1e-6), torch.full((1, 3), 1 / math.sqrt(2), dtype=D))      # eps inside the root


def test_rows_of_pairs():
    assert O.bigram_rows([5, 3, 3, 9], 10, 7, 2) == [10, (35 + 6) % 10, (21 + 6) % 10, (21 + 18) % 10]
    assert O.bigram_rows([4], 3, 1, 1) == [3] and O.bigram_rows([1, 2], 5, -3, 0) == [5, 2]


def test_rotation_turns_pairs_half_a_head_apart():
    x = torch.arange(1.0, 7.0, dtype=D).view(1, 1, 6)
    y = O.rotate(x, torch.tensor([3]), 100.0, 4)      # pairs (0, 2) and (1, 3); 4 and 5 stay
    for i, f in ((0, 1.0), (1, 0.1)):
        u, v, a = float(x[0, 0, i]), float(x[0, 0, i + 2]), 3 * f
        assert math.isclose(float(y[0, 0, i]), u * math.cos(a) - v * math.sin(a)) and math.isclose(float(y[0, 0, i + 2]), v * math.cos(a) + u * math.sin(a))
    assert torch.equal(y[..., 4:], x[..., 4:]) and torch.equal(O.rotate(x, torch.tensor([0]), 100.0, 6), x)


def test_masks_pair_by_pair():
    c, w = O.chunk_mask(9, 4), O.window_mask(9, 3, 2)
    for i in range(9):
        assert c[i].nonzero().flatten().tolist() == [j for j in range(i + 1) if j // 4 == i // 4]
        assert w[i].nonzero().flatten().tolist() == [j for j in range(i + 1) if i - j < 3 or j < 2]
    assert torch.equal(O.window_mask(9, 9, 0), torch.ones(9, 9, dtype=torch.bool).tril()) and torch.equal(O.chunk_mask(9, 1), torch.eye(9, dtype=torch.bool))


def test_attention_pair_by_pair():
    g = torch.Generator().manual_seed(2)
    T, H, G = 7, 4, 2
    q, k, val = (torch.randn((T, n, d), generator=g, dtype=D) for n, d in ((H, 3), (G, 3), (G, 2)))
    sink, mask = torch.randn(H, generator=g, dtype=D), O.window_mask(T, 3, 1)
    for s in (None, sink):
        o = O.masked_attention(q, k, val, 2.0, 1.5, mask, s)
        for i in range(T):
            for h in range(H):
                p = {j: math.exp(1.5 * math.tanh(2.0 * float(q[i, h] @ k[j, h // 2]) / 1.5)) for j in range(T) if mask[i, j]}
                total = sum(p.values()) + (math.exp(float(s[h])) if s is not None else 0)
                assert torch.allclose(o[i, h], sum(x * val[j, h // 2] for j, x in p.items()) / total)


def test_choices_by_hand():
    s = torch.tensor([[0.9, 0.1, 0.6, 0.5, 0.2, 0.3]], dtype=D)
    zero = torch.zeros(6, dtype=D)
    pick = lambda c, top, count, keep: sorted(O.choose(s, c, top, {"count": count, "keep": keep})[0].tolist())      # noqa: E731
    assert pick(zero, 2, 1, 1) == [0, 2] and pick(zero, 2, 3, 1) == [2, 3] and pick(zero, 3, 3, 2) == [0, 2, 3]
    assert pick(zero, 2, 2, 1) == [0, 2] and pick(zero, 1, 6, 1) == [0]      # groups of three: 1.5 against 0.8; groups of one
    push = zero.clone()
    push[4:] = 0.7
    assert pick(push, 2, 3, 1) == [4, 5]
    assert pick(zero - 5, 3, 3, 2) == [0, 2, 3]      # negative choice scores lose to nothing that was dropped
    router = torch.log(s / (1 - s)).T
    chosen, weight = O.route(torch.ones((1, 1), dtype=D), router, push, {"top": 2, "groups": {"count": 3, "keep": 1}, "scale": 2.0})
    want = {4: 0.2, 5: 0.3}
    assert all(math.isclose(float(weight[0, i]), want[int(chosen[0, i])] / 0.5 * 2.0) for i in range(2))      # without the correction


def test_units():
    z = torch.linspace(-6, 6, 50, dtype=D)
    assert torch.allclose(O.gelu_tanh(z), torch.nn.functional.gelu(z, approximate="tanh"))
    w = {"gate": torch.tensor([[3.0]], dtype=D), "up": torch.tensor([[-4.0]], dtype=D), "down": torch.tensor([[1.0]], dtype=D)}
    for x, g, u in ((1.0, 2.0, -2.0), (-1.0, -3.0, 2.0), (0.1, 0.3, -0.4)):      # the gate has no lower limit
        assert math.isclose(float(O.clamped_unit(torch.tensor([[x]], dtype=D), w, 2.0)), g / (1 + math.exp(-1.702 * g)) * (u + 1))


@pytest.mark.parametrize("name", list(CONFIGS))
def test_oracle_is_causal_and_reads_every_tensor(name):
    cfg, w = CONFIGS[name], random_weights(CONFIGS[name], 4)
    assert {n: tuple(t.shape) for n, t in w.items()} == tensor_shapes(cfg)
    s = random_tokens(cfg, 24, 1)
    a = O.forward(cfg, w, s)
    b = O.forward(cfg, w, s[:10] + random_tokens(cfg, 14, 2))
    assert torch.allclose(a[:10], b[:10]) and not torch.allclose(a[10:], b[10:])
    for n in w:
        if ".e" in n or n.endswith(("router", "correction")):
            continue      # an expert may have no token
        changed = dict(w)
        changed[n] = (w[n].float() * torch.linspace(0.5, 2, w[n].shape[-1]) + 0.1).to(w[n].dtype)
        assert (O.forward(cfg, changed, s) - a).abs().max() > 1e-6, n


def test_a_layer_with_the_weights_of_another():
    cfg, w = CONFIGS["odd"], random_weights(CONFIGS["odd"], 1)
    unrolled = dict(cfg, layers=[{k: v for k, v in layer.items() if k != "weights_of"} for layer in cfg["layers"]])
    w6 = dict(w)
    for i, layer in enumerate(cfg["layers"]):
        if "weights_of" in layer:
            w6.update({f"l{i}." + n.split(".", 1)[1]: t for n, t in w.items() if n.startswith(f"l{layer['weights_of']}.")})
    s = random_tokens(cfg, 12, 0)
    assert torch.equal(O.forward(cfg, w, s), O.forward(unrolled, w6, s))


def test_settled_tokens_have_no_close_choice():
    cfg, w = CONFIGS["odd"], random_weights(CONFIGS["odd"], 1)
    s = settled_tokens(cfg, w, 60, 3)
    with O.watching_choices() as margins:
        O.forward(cfg, w, s)
    assert len(margins) == 4 and all((m >= 4e-3).all() for m in margins)


# ------------------------------------------------------------------------------------------------ host side of the product
def test_registry_and_configuration(tmp_path, capsys):
    from nano_vllm_ninetoothed_amd.__main__ import main
    from nano_vllm_ninetoothed_amd.models import architectures, load_config, model_class
    from nano_vllm_ninetoothed_amd.models.lulizen import LulizenConfig, LulizenModel
    assert "Lulizen" in architectures()
    (tmp_path / "config.json").write_text(json.dumps(CONFIGS["odd"]))
    c = load_config(tmp_path)
    assert isinstance(c, LulizenConfig) and (c.width, c.vocab, c.eps, c.bigram, len(c.layers)) == (76, 101, 1e-5, (67, 13, 5), 6)
    assert model_class(c) is LulizenModel and LulizenModel.needs(c) == (True, True) and LulizenModel.dtypes == (torch.bfloat16, torch.float32)
    assert c.order() == [0, 1, 2, 0, 1, 0]
    for cfg in CONFIGS.values():
        LulizenConfig.from_dict(cfg)
    assert main(["models"]) == 0 and "Lulizen" in capsys.readouterr().out


A, B = chunked(4, 2, 16, 8, 8, 5, 0.1, 3.0), windowed(4, 2, 16, 8, 8, 5, 0, 0.1, 3.0)


@pytest.mark.parametrize("layer,mlp,change", [
    (A, None, {"heads": 0}), (A, None, {"dim": "8"}), (A, None, {"kv_heads": 3}), (A, None, {"vdim": -1}), (A, None, {"softcap": 0}), (A, None, {"rot": {"base": 10.0, "dims": 18}}),
    (A, None, {"rot": {"base": 10.0, "dims": 7}}), (A, None, {"rot": {"base": -1.0, "dims": 8}}), (A, None, {"mask": {"size": 0}}), (B, None, {"mask": {"size": 4, "keep_first": -1}}),
    (B, None, {"mask": {"size": 1.5, "keep_first": 1}}), (A, moe(8, 6, 3, 3, 1, 8), None), (A, moe(8, 6, 2, 4, 1, 8), None), (A, moe(8, 6, 2, 3, 4, 8), None), (A, moe(0, 6, 2, 3, 1, 8), None),
    (A, moe(8, 6, 2, 3, 1, 0), None), (A, moe(8, 2, 3, 1, 1, 8), None), (A, dense(0), None), (A, {"kind": "other", "ff": 8}, None)])
def test_configurations_that_make_no_sense_are_refused(layer, mlp, change):
    from nano_vllm_ninetoothed_amd.models.lulizen import LulizenConfig
    LulizenConfig.from_dict(config(16, 16, [(layer, None)], (3, 1, 1)))
    with pytest.raises(ValueError):
        LulizenConfig.from_dict(config(16, 16, [(dict(layer, mixer={**layer["mixer"], **(change or {})}), mlp)], (3, 1, 1)))


def test_borrowed_weights():
    from nano_vllm_ninetoothed_amd.models.lulizen import LulizenConfig
    good = config(16, 16, [(A, dense(8)), (B, None), 0, 2], (3, 1, 1))
    assert LulizenConfig.from_dict(good).order() == [0, 1, 0, 0]
    later = dict(good, layers=[dict(good["layers"][1], weights_of=1), good["layers"][1]])
    assert LulizenConfig.from_dict(later).order() == [1, 1]
    for i, j in ((0, 0), (0, 4), (0, -1), (0, 2), (2, 1), (1, "0")):      # itself, no layer, in a circle, another kind
        layers = [dict(x) for x in good["layers"]]
        layers[i]["weights_of"] = j
        with pytest.raises(ValueError):
            LulizenConfig.from_dict(dict(good, layers=layers))
    with pytest.raises(ValueError):
        LulizenConfig.from_dict(config(16, 16, [(A, None)], (0, 1, 1)))
    with pytest.raises(ValueError):
        LulizenConfig.from_dict(dict(good, layers=[dict(A, type="attention_3", mlp=None)]))


def test_checkpoint_names(tmp_path):
    from nano_vllm_ninetoothed_amd.weights import CheckpointWeights
    w = random_weights(CONFIGS["ones"], 0)
    write_checkpoint(tmp_path / "m", CONFIGS["ones"], w)
    source = CheckpointWeights(tmp_path / "m", torch.float32, "cpu")
    assert torch.equal(source.take("l0.mlp.shared.gate", (24, 64)), w["l0.mlp.shared.gate"].float())
    with pytest.raises(ValueError):
        source.take("bigram", (1, 64))


def test_the_last_token_is_a_slot_of_one_integer():
    from nano_vllm_ninetoothed_amd.cache import CacheManager
    t = CacheManager(1, 32, 3, "cpu", slots=True).per_slot(dtype=torch.int32)
    assert t.shape == (3,) and t.dtype == torch.int32


def test_argument_validation_on_the_host():
    """The C ABI refuses what the kernels do not cover before any launch."""
    from ctypes import byref
    from nano_vllm_ninetoothed_amd import _capi
    if not _capi.LIB_PATH.exists():
        from nano_vllm_ninetoothed_amd import build
        build.build(force=False)
    lib, A = _capi.load(), 0x1000
    assert lib.mops_hip_layer_norm_f32(A, A, 1e-5, A, 0, 4, 64, None) == -1                       # out aliases x
    assert lib.mops_hip_layer_norm_f32(None, None, 1e-5, None, 0, 0, 64, None) == 0
    assert lib.mops_hip_add_norm_norm(A, 2 * A, 64, 1, A, A, A, 1e-5, 1, A, 0, 4, 64, None) == -1  # out aliases extra
    assert lib.mops_hip_gelu_glu(A, 32, A, 64, A, 64, 0, 4, 64, None) == -1
    e = _capi.EmbedPairs()
    e.ids = e.table = e.pairs = e.residual = e.before = e.starts = e.state_slots = A
    e.table_stride = e.pairs_stride = e.width = 64
    e.buckets, e.mul_prev, e.mul_cur, e.num_slots, e.tokens, e.vocab = 5, 1, 1, 2, 3, 10
    e.token_seq = A
    assert lib.mops_hip_embed_pairs(byref(e), None) == -1                                         # token_seq without cu_seqlens
    e.token_seq, e.mul_prev = None, 1 << 40
    assert lib.mops_hip_embed_pairs(byref(e), None) == -2
    e.buckets = 0
    assert lib.mops_hip_embed_pairs(byref(e), None) == -1
    p = _capi.RotaryPrepare()
    p.qkv = p.positions = p.slot_mapping = p.q = p.k_pages = p.v_pages = p.cos_sin = A
    p.num_slots, p.tokens, p.heads, p.kv_heads, p.dim, p.vdim, p.max_positions, p.qkv_stride = 64, 2, 4, 2, 16, 8, 10, 200
    for rot, stride in ((18, 200), (7, 200), (-2, 200), (8, 100)):
        p.rot, p.qkv_stride = rot, stride
        assert lib.mops_hip_rotary_prepare(byref(p), None) == -1
    m = _capi.Moe()
    m.rows = m.tiles = m.score = A
    m.tokens, m.experts, m.top, m.width, m.ff, m.block_rows = 4, 8, 3, 64, 32, 32
    for groups, keep, unit in ((3, 1, 1), (4, 5, 1), (4, 1, 1), (4, 0, 1), (2, 1, 2), (-1, 1, 0)):
        m.groups, m.keep, m.unit = groups, keep, unit
        assert lib.mops_hip_moe_gate_up(A, 64, A, 32, A, 32, byref(m), None) == -1
    m.groups, m.keep, m.unit = 4, 2, 1
    assert lib.mops_hip_moe_route(A, 64, A, A, A, A, byref(m), None) == -1                        # no correction
    b = _capi.BiasedAttention()
    b.q = b.k_pages = b.v_pages = b.context_lens = b.block_table = b.out = A
    b.block_table_stride, b.block_size, b.num_blocks, b.max_blocks = 4, 32, 8, 4
    b.rows, b.heads, b.kv_heads, b.dim, b.vdim, b.scale = 2, 4, 2, 64, 64, 1.0
    for bad in (dict(window=4, chunk=4), dict(window=-1), dict(keep_first=-1), dict(softcap=-1.0), dict(softcap=float("nan")), dict(softcap=1.0, slopes=A), dict(gate=A, gate_stride=3)):
        for n, v in bad.items():
            setattr(b, n, v)
        assert lib.mops_hip_biased_attention_rows(byref(b), None) == -1, bad
        assert lib.mops_hip_biased_decode(byref(b), A, 1 << 30, None) == -1 and lib.mops_hip_biased_prefill(byref(b), A, 1, None) == -1, bad
        for n in bad:
            setattr(b, n, None if n in ("slopes", "gate") else 0)
    b.chunk = 1 << 31
    assert lib.mops_hip_biased_attention_rows(byref(b), None) == -2
