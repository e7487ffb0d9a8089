"""No GPU: the oracle of the Nepulix design against itself and against closed forms, and the host side of what runs it -
configuration, registry, checkpoint reader, cache manager, batch plans."""
import json
import math

import pytest
import torch

from nepulix_cases import CONFIGS, config, latent, mamba2, random_tokens, random_weights, retention, tensor_shapes, write_checkpoint
from oracle import nepulix as O

D = torch.float64


# ------------------------------------------------------------------------------------------------ the oracle itself
def test_rotations():
    g = torch.Generator().manual_seed(0)
    x = torch.randn((4, 2, 12), generator=g, dtype=D)
    pos = torch.tensor([0, 1, 5, 900])
    for rotate, pair in ((O.rotate_half, lambda i, n: (i, i + n // 2)), (O.rotate_interleaved, lambda i, n: (2 * i, 2 * i + 1))):
        y = rotate(x, pos, 100.0, 8)
        assert torch.equal(y[0], x[0]) and torch.equal(y[..., 8:], x[..., 8:])
        for i in range(4):
            a, b = pair(i, 8)
            z = torch.complex(x[..., a], x[..., b]) * torch.exp(1j * pos.to(D)[:, None] * 100.0 ** (-2 * i / 8))
            assert torch.allclose(y[..., a], z.real) and torch.allclose(y[..., b], z.imag)
    # scores depend on distances only
    q, k = x[:1].expand(2, -1, -1), x[1:2].expand(2, -1, -1)
    qa, ka = O.rotate_half(q, torch.tensor([7, 107]), 50.0, 8), O.rotate_half(k, torch.tensor([3, 103]), 50.0, 8)
    s = (qa * ka).sum(-1)
    assert torch.allclose(s[0], s[1])


def test_recurrence_equals_its_closed_form():
    g = torch.Generator().manual_seed(1)
    T, H, N, V = 9, 2, 3, 4
    q, k, v = (torch.randn((T, H, n), generator=g, dtype=D) for n in (N, N, V))
    a = torch.rand((T, H), generator=g, dtype=D)
    o, S = O.decayed_recurrence(q, k, v, a)
    for h in range(H):
        for t in range(T):
            want = sum(a[s + 1:t + 1, h].prod() * (q[t, h] @ k[s, h]) * v[s, h] for s in range(t + 1))
            assert torch.allclose(o[t, h], want)
    o1, S1 = O.decayed_recurrence(q[:4], k[:4], v[:4], a[:4])
    o2, S2 = O.decayed_recurrence(q[4:], k[4:], v[4:], a[4:], S1)
    assert torch.allclose(torch.cat((o1, o2)), o) and torch.allclose(S2, S)


def test_causal_conv_equals_conv1d():
    g = torch.Generator().manual_seed(2)
    x, w, b = torch.randn((11, 5), generator=g, dtype=D), torch.randn((5, 4), generator=g, dtype=D), torch.randn(5, generator=g, dtype=D)
    want = torch.nn.functional.conv1d(torch.nn.functional.pad(x.T[None], (3, 0)), w[:, None], b, groups=5)[0].T
    assert torch.allclose(O.causal_conv(x, w, b), want)
    assert torch.allclose(O.causal_conv(x[5:], w, b, before=x[2:5]), want[5:])


def test_small_functions():
    x = torch.linspace(-40, 40, 81, dtype=D)
    assert torch.allclose(O.silu(x), torch.nn.functional.silu(x)) and torch.allclose(O.softplus(x), torch.nn.functional.softplus(x))
    y = torch.tensor([[3.0, 4.0]], dtype=D)
    assert torch.allclose(O.rms(y, 0.0), y / math.sqrt(12.5)) and torch.allclose(O.rms(y * 0, 1e-6), y * 0)
    assert torch.allclose(O.group_rms(torch.tensor([[3.0, 4.0, 0.0, 2.0]], dtype=D), 2, 0.0), torch.tensor([[3 / 12.5 ** .5, 4 / 12.5 ** .5, 0, 2 ** .5]], dtype=D))
    w = {"gate": torch.eye(3, dtype=D), "up": torch.tensor([[1., 0, 0]] * 3, dtype=D), "down": torch.eye(3, dtype=D)}
    got = O.dense_ff(torch.tensor([[9.0, -9.0, 0.5]], dtype=D), w, {"limit": 2.0})[0]
    want = [g / (1 + math.exp(-1.702 * g)) * 3.0 for g in (2.0, -9.0, 0.5)]      # the gate is bounded from above only
    assert torch.allclose(got, torch.tensor(want, dtype=D))


def test_latent_attention_in_the_latent_space():
    """The absorbed form - keys and values never expanded - is the same function."""
    cfg = CONFIGS["odd"]
    m = cfg["layers"][2]["mixer"]
    w = {k[len("l2.mix."):]: v.to(D) for k, v in random_weights(cfg, 1).items() if k.startswith("l2.mix.")}
    h = torch.randn((7, cfg["width"]), dtype=D, generator=torch.Generator().manual_seed(3))
    pos = torch.arange(7)
    want, _ = O.latent_attention(h, w, m, 1e-5, pos)
    H, dim, R, V, K = (m[k] for k in ("heads", "dim", "rot_dim", "vdim", "kv_rank"))
    q = ((O.rms(h @ w["dq"].T, 1e-5) * w["dq.norm"]) @ w["uq"].T).view(7, H, dim + R)
    down = h @ w["dkv"].T
    c = O.rms(down[:, :K], 1e-5) * w["dkv.norm"]
    ql = torch.einsum("thd,hdk->thk", q[..., :dim], w["uk"].view(H, dim, K))
    qr = O.rotate_interleaved(q[..., dim:], pos, m["rot"]["base"], R)
    kr = O.rotate_interleaved(down[:, None, K:], pos, m["rot"]["base"], R)[:, 0]
    s = (torch.einsum("ihk,jk->hij", ql, c) + torch.einsum("ihr,jr->hij", qr, kr)) * m["scale"]
    p = torch.softmax(s.masked_fill(torch.ones(7, 7).triu(1).bool(), -math.inf), -1)
    o = torch.einsum("hik,hvk->ihv", p @ c, w["uv"].view(H, V, K)).reshape(7, -1) @ w["o"].T
    assert torch.allclose(o, want)


@pytest.mark.parametrize("name", ["odd", "ones"])
def test_oracle_is_causal(name):
    cfg = CONFIGS[name]
    w = random_weights(cfg, 4)
    s = random_tokens(cfg, 24, 1)
    a = O.forward(cfg, w, s)
    b = O.forward(cfg, w, s[:10] + random_tokens(cfg, 14, 2))
    assert torch.allclose(a[:10], b[:10]) and not torch.allclose(a[10:], b[10:])
    assert a.shape == (24, cfg["vocab"])


def test_mixers_depend_on_what_they_keep():
    """Every mechanism matters in the logits: the first token through state and cache, the decay, the skip, the conv's taps."""
    cfg = CONFIGS["odd"]
    w = random_weights(cfg, 4)
    s = random_tokens(cfg, 30, 1)
    base = O.forward(cfg, w, s)[-1]
    assert (O.forward(cfg, w, [(s[0] + 1) % cfg["vocab"]] + s[1:])[-1] - base).abs().max() > 1e-3
    for name in ("l0.mix.D", "l0.mix.dt_bias", "l0.mix.A_log", "l0.mix.conv", "l0.mix.conv.b", "l1.mix.g", "l2.mix.dkv.norm", "l0.norm1", "l0.norm2", "final.norm"):
        changed = dict(w)
        changed[name] = w[name] + 0.5
        assert (O.forward(cfg, changed, s)[-1] - base).abs().max() > 1e-3, name


# ------------------------------------------------------------------------------------------------ host side of the product
def test_registry_and_configuration(tmp_path):
    from nano_vllm_ninetoothed_amd.models import architectures, load_config, model_class
    from nano_vllm_ninetoothed_amd.models.nepulix import NepulixConfig, NepulixModel
    from nano_vllm_ninetoothed_amd.models.qwen3 import Qwen3Model, Qwen3Shape
    assert {"Nepulix", "Qwen3ForCausalLM"} <= set(architectures())
    (tmp_path / "config.json").write_text(json.dumps(CONFIGS["odd"]))
    c = load_config(tmp_path)
    assert isinstance(c, NepulixConfig) and (c.width, c.vocab, c.eps, len(c.layers)) == (72, 101, 1e-5, 4)
    assert model_class(c) is NepulixModel and NepulixModel.needs(c) == (True, True)
    assert NepulixModel.needs(NepulixConfig.from_dict(config(8, 8, [latent(1, 8, 2, 8, 8, 8)]))) == (True, False)
    assert NepulixModel.needs(NepulixConfig.from_dict(config(8, 8, [retention(1, 8, 8, 8)]))) == (False, True)
    assert model_class(Qwen3Shape()) is Qwen3Model
    (tmp_path / "config.json").write_text(json.dumps({"architecture": "Other"}))
    with pytest.raises(ValueError):
        load_config(tmp_path)
    with pytest.raises(ValueError):
        model_class(object())


@pytest.mark.parametrize("layer,change", [
    (retention(2, 8, 8, 8), {"decay": [0.5]}), (retention(2, 8, 8, 8), {"decay": [0.5, 1.5]}), (retention(2, 8, 8, 8), {"rot": {"base": 1e4, "dims": 10}}),
    (mamba2(4, 8, 8, 2, 3, 2), {"groups": 3}), (mamba2(4, 8, 8, 2, 3, 2), {"norm_groups": 5}), (mamba2(4, 8, 8, 2, 3, 2), {"conv": 0}),
    (latent(2, 8, 4, 8, 8, 8), {"rot": {"base": 1e4, "dims": 2}}), (latent(2, 8, 4, 8, 8, 8), {"kv_rank": "8"})])
def test_configurations_that_make_no_sense_are_refused(layer, change):
    from nano_vllm_ninetoothed_amd.models.nepulix import NepulixConfig
    NepulixConfig.from_dict(config(16, 16, [layer]))
    bad = dict(layer, mixer={**layer["mixer"], **change})
    with pytest.raises(ValueError):
        NepulixConfig.from_dict(config(16, 16, [bad]))
    with pytest.raises(ValueError):
        NepulixConfig.from_dict(config(16, 16, [dict(layer, type="other")]))


def test_checkpoint_reader(tmp_path, capsys):
    from safetensors.torch import load_file
    from nano_vllm_ninetoothed_amd.weights import CheckpointWeights, read_safetensors
    cfg = CONFIGS["ones"]
    w = random_weights(cfg, 0)
    w["table"] = torch.arange(5, dtype=torch.int32)
    w["single"] = torch.tensor([1.5], dtype=torch.bfloat16)
    write_checkpoint(tmp_path / "m", cfg, w)
    mine, theirs = read_safetensors(tmp_path / "m" / "model.safetensors"), load_file(tmp_path / "m" / "model.safetensors")
    assert mine.keys() == theirs.keys() and all(torch.equal(mine[k], theirs[k]) and mine[k].dtype == theirs[k].dtype for k in mine)
    src = CheckpointWeights(tmp_path / "m", torch.float32, "cpu")
    for name, shape in tensor_shapes(cfg).items():
        assert torch.equal(src.take(name, shape), w[name].float())
    assert src.take("table", (5,)).dtype == torch.int32
    src.finish()
    assert "single" in capsys.readouterr().err
    with pytest.raises(ValueError):
        src.take("single", (2,))
    with pytest.raises(KeyError):
        src.take("embed", (1, 1))
    (tmp_path / "empty").mkdir()
    with pytest.raises(FileNotFoundError):
        CheckpointWeights(tmp_path / "empty")
    bad = bytearray((tmp_path / "m" / "model.safetensors").read_bytes())
    (tmp_path / "short.safetensors").write_bytes(bad[:-64])
    with pytest.raises(ValueError):
        read_safetensors(tmp_path / "short.safetensors")


def test_cache_manager_hands_out_and_takes_back():
    from nano_vllm_ninetoothed_amd.cache import CacheManager
    from nano_vllm_ninetoothed_amd.engine import Sequence
    c = CacheManager(4, 32, 2, "cpu", pages=True, slots=True)
    a, b, d = Sequence([1], 1, 1.0), Sequence([1], 1, 1.0), Sequence([1], 1, 1.0)
    c.hold(a, 33)
    c.hold(b, 32)
    assert len(a.block_table) == 2 and len(b.block_table) == 1 and a.state_slot != b.state_slot
    assert not c.can_hold(d, 1)                      # no slot left
    c.hold(a, 64)
    assert len(a.block_table) == 2
    assert c.can_hold(b, 64) and not c.can_hold(b, 65)
    with pytest.raises(RuntimeError):
        c.hold(b, 65)
    freed = a.block_table
    c.release(a)
    assert a.state_slot == -1 and a.block_table == []
    c.hold(d, 96)
    assert set(freed) <= set(d.block_table) and d.state_slot == 0
    c.release(b)
    c.release(d)
    assert sorted(c.free_blocks) == [0, 1, 2, 3] and sorted(c.free_slots) == [0, 1]
    assert c.paged(8).shape == (4, 32, 8) and c.per_slot(3, 5).shape == (2, 3, 5)
    # a model without pages needs none, however long the sequence
    s = CacheManager(1, 32, 1, "cpu", pages=False, slots=True)
    s.hold(a, 10 ** 6)
    assert a.block_table == [] and a.state_slot == 0


def test_rotary_tables_are_shared_and_exact():
    from nano_vllm_ninetoothed_amd.layers import Rotary
    r = Rotary(3000, "cpu")
    t = r.table(1e4, 16)
    assert r.table(1e4, 16) is t and r.table(1e4, 8) is not t
    want = O.angles(torch.arange(3000), 1e4, 16)
    assert torch.equal(t, torch.cat((want.cos(), want.sin()), 1).float())


def test_prefill_plan():
    from nano_vllm_ninetoothed_amd.mops.hip.recurrent_ops import latent_prefill_plan
    row_seq, row_pos, tiles = latent_prefill_plan([130, 64], [0, 100], 5, 2)
    assert len(row_pos) == 192 + 192 and row_pos[:130] == list(range(130)) and set(row_pos[130:192]) == {-1}
    assert row_seq == [2] * 192 + [3] * 192 and row_pos[192:192 + 164] == list(range(164))
    assert sorted(tiles) == [(5, 128, 0, 0, 130), (133, 2, 128, 0, 130), (135, 64, 100, 192, 164)]
    assert tiles[0] == (135, 64, 100, 192, 164)


def test_command_line_lists_the_models(capsys):
    from nano_vllm_ninetoothed_amd.__main__ import main
    assert main(["models"]) == 0
    assert "Nepulix" in capsys.readouterr().out
    with pytest.raises(SystemExit):
        main(["trace"])
