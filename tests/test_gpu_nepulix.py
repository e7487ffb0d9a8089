"""GPU: Nepulix models of several shapes through the engine - its batches, cache manager, scheduler, sampler, command line -
against the plain float64 restatement in oracle/nepulix.py."""
import json
import subprocess
import sys
from pathlib import Path

import numpy as np
import pytest
import torch

import model_harness as H
from nepulix_cases import CONFIGS, logit_error, random_tokens, random_weights, write_checkpoint
from oracle import nepulix as O

pytestmark = pytest.mark.gpu
ROOT = Path(__file__).resolve().parent.parent
DTYPES = [torch.float32, torch.bfloat16]
check, feed = H.check, H.feed


def Wanted(cfg, w, tokens):
    return H.Wanted(O, cfg, w, tokens)


def engine(gpu, cfg, *args, **kw):
    from nano_vllm_ninetoothed_amd.models.nepulix import NepulixConfig
    return H.engine(gpu, NepulixConfig.from_dict(cfg), *args, **kw)


@pytest.fixture(scope="module")
def case():
    """(config, weights, tokens by name, oracle logits by name), computed once per configuration."""
    made = {}

    def get(name, lengths=(300, 97, 65, 1)):
        if name not in made:
            cfg = CONFIGS[name]
            w = random_weights(cfg, 11)
            seqs = [random_tokens(cfg, n, 100 + i) for i, n in enumerate(lengths)]
            # far keys: a rare token early on, asked for again and again later
            seqs[0][5:8] = seqs[0][150:153] = seqs[0][290:293]
            made[name] = (cfg, w, seqs, [Wanted(cfg, w, s) for s in seqs])
        return made[name]
    return get


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", list(CONFIGS))
def test_whole_prompts_and_every_layer(gpu, case, name, dtype):
    cfg, w, seqs, wants = case(name)
    eng = engine(gpu, cfg, w, dtype)
    for s, want in zip(seqs, wants):
        q = eng.open_sequence()
        check(feed(eng, s, q, [len(s)]), want, dtype, f"{len(s)} tokens")
        eng.close_sequence(q)
    layers = []
    O.forward(cfg, w, seqs[2], layers_out=layers)
    seen = []
    eng.model.layer_hook = lambda i, x: seen.append(x.clone())
    feed(eng, seqs[2], eng.open_sequence(), [len(seqs[2])])
    for i, (a, b) in enumerate(zip(seen, layers)):
        err = ((a.double().cpu() - b).norm() / b.norm()).item()
        assert err <= (2e-6 if dtype == torch.float32 else 2e-2), f"layer {i}: {err:.3g}"


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", list(CONFIGS))
def test_portions_and_token_by_token(gpu, case, name, dtype):
    """Prompts cut anywhere, down to two tokens and to single ones; the same slots and pages serve one run after another."""
    cfg, w, seqs, wants = case(name)
    eng = engine(gpu, cfg, w, dtype, tokens=320, slots=1)          # just enough for one sequence: everything is used again
    n = len(seqs[0])
    plans = {"two by two": list(range(2, n, 2)) + [n], "one by one": list(range(1, 101)) + [n], "prefill, then decode": [200] + list(range(201, n + 1)),
             "borders": [31, 32, 33, 63, 65, 96, 98, 127, 128, 129, 191, 255, 257, n], "large after small": [3, 67, 70, 198, n]}
    for what, cuts in plans.items():
        q = eng.open_sequence()
        check(feed(eng, seqs[0], q, cuts), wants[0], dtype, what)
        eng.close_sequence(q)
        assert len(eng.cache.free_slots) == 1 and len(eng.free_blocks) == eng.num_blocks


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", list(CONFIGS))
def test_mixed_batches(gpu, case, name, dtype):
    """Unequal requests side by side, portions beside single tokens, some left out of a step, each against itself alone;
    requests come and go, so that pages and slots change hands."""
    cfg, w, seqs, wants = case(name)
    eng = engine(gpu, cfg, w, dtype, tokens=32 * 24, slots=4)
    got = H.mixed_batches(eng, seqs, [0, 1, 2, 3, 1, 2, 1, 3, 2, 1])
    assert len(got) == 10
    for i, pos, logits in got:
        check(logits, wants[i][pos], dtype, f"request {i}")


def test_nothing_wanted_and_order_of_rows(gpu, case):
    cfg, w, seqs, wants = case("odd")
    eng = engine(gpu, cfg, w, torch.float32)
    a, b = eng.open_sequence(), eng.open_sequence()
    assert eng.run_portions([(a, seqs[0][:70], []), (b, seqs[1][:1], [])]) is None
    out = eng.run_portions([(a, seqs[0][70:200], [129, 3]), (b, seqs[1][1:2], [0])])
    check(out[:2], wants[0][[199, 73]], torch.float32, "first")
    check(out[2:], wants[1][[1]], torch.float32, "second")


@pytest.mark.parametrize("dtype", DTYPES)
def test_long_decoding(gpu, dtype):
    """Hundreds of decoded tokens behind a short prompt, across many pages; the first tokens stay reachable."""
    cfg = CONFIGS["odd"]
    w = random_weights(cfg, 3)
    s = random_tokens(cfg, 420, 5)
    want = Wanted(cfg, w, s)
    eng = engine(gpu, cfg, w, dtype, tokens=448, block_size=64)
    check(feed(eng, s, eng.open_sequence(), [7] + list(range(8, 421))), want, dtype, "long decoding")


@pytest.mark.parametrize("mode", ["stepwise", "chunked", "graphs", "pipelined"])
def test_greedy_generation(gpu, mode):
    """generate() in every mode of the scheduler against greedy decoding by the oracle (float32, so that rounding does not
    pick another token); twice on one engine."""
    cfg = CONFIGS["odd"]
    w = random_weights(cfg, 21)
    prompts = [random_tokens(cfg, n, 50 + n) for n in (1, 40, 9, 70, 3, 2)]
    n_out = [9, 4, 12, 6, 1, 8]
    want = [O.greedy(cfg, w, p, n) for p, n in zip(prompts, n_out)]
    eng = engine(gpu, cfg, w, torch.float32, tokens=32 * 12, chunked_prefill=mode == "chunked", max_num_batched_tokens=16 if mode == "chunked" else 80)
    if mode in ("graphs", "pipelined"):
        eng.capture_decode_graphs(max_bs=4, max_model_len=128)
        eng.pipelined = mode == "pipelined"
    for _ in range(2):
        outs, stats = eng.generate(prompts, n_out)
        assert outs == want
        assert len(eng.free_blocks) == 12 and len(eng.cache.free_slots) == 4 and not eng.running and not eng.waiting
        if mode == "chunked":
            assert stats["prefill_tokens"] >= sum(len(p) for p in prompts)


def test_graph_replay_equals_eager_decode(gpu):
    """The captured decode step in bf16, replayed with eager work in between, against the eager step on the same padded batch."""
    cfg = CONFIGS["wide"]
    w = random_weights(cfg, 2)
    outs = []
    for graphs in (True, False):
        eng = engine(gpu, cfg, w, torch.bfloat16, tokens=32 * 40, slots=8)
        if graphs:
            eng.capture_decode_graphs(max_bs=8, max_model_len=256)
        for i, n in enumerate((33, 5, 64)):
            eng.add_request(random_tokens(cfg, n, i), 32)
        eng.step()
        rows = []
        for it in range(6):
            seqs, is_prefill = eng._schedule()
            assert not is_prefill
            ids, pos, ctx = eng._prepare_decode(seqs)
            rows.append((eng._decode_replay(ids, pos, ctx) if graphs else eng.forward(ids, pos, ctx)).float().cpu())
            torch.cuda.synchronize()
            for j, q in enumerate(seqs):
                q.num_cached = len(q)
                q.token_ids.append((17 * it + j) % cfg["vocab"])
        outs.append(torch.stack(rows))
    assert logit_error(outs[0].flatten(0, 1), outs[1].flatten(0, 1)).max() < 2e-2


def test_checkpoint_folder_command_line_and_trace(gpu, case, tmp_path):
    """A folder with config.json and safetensors through Engine.from_pretrained, the generate command and a replayed trace."""
    cfg, w, seqs, wants = case("odd")
    write_checkpoint(tmp_path / "model", cfg, w)
    from nano_vllm_ninetoothed_amd.engine import Engine
    eng = Engine.from_pretrained(tmp_path / "model", dtype=torch.float32, num_blocks=8, block_size=64, max_num_seqs=2, max_model_len=512)
    check(feed(eng, seqs[1], eng.open_sequence(), [len(seqs[1])]), wants[1], torch.float32, "from_pretrained")
    prompts, want = [seqs[2][:20], seqs[1][:3]], []
    for p in prompts:
        want.append(O.greedy(cfg, w, p, 5))
    cmd = [sys.executable, "-m", "nano_vllm_ninetoothed_amd", "generate", "--model", str(tmp_path / "model"), "--dtype", "float32", "--max-tokens", "5",
           "--block-size", "64", "--chunked-prefill", "--max-num-batched-tokens", "7"]
    for p in prompts:
        cmd += ["--prompt", ",".join(map(str, p))]
    r = subprocess.run(cmd, cwd=ROOT, capture_output=True, text=True, timeout=110)
    assert r.returncode == 0, r.stderr
    assert [json.loads(x) for x in r.stdout.strip().splitlines()] == want
    out = tmp_path / "out"
    out.mkdir()
    a, b = seqs[0], seqs[1]
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": a[:40], "want": [39, 2]}], "end": []},
             {"step": 1, "entries": [{"id": "b", "tokens": b[:1], "want": []}, {"id": "a", "tokens": a[40:42], "want": []}], "end": []},
             {"step": 2, "entries": [{"id": "a", "tokens": a[42:130], "want": [87]}, {"id": "b", "tokens": b[1:2], "want": [0]}], "end": ["a"]},
             {"step": 3, "entries": [{"id": "b", "tokens": b[2:97], "want": [94]}], "end": ["b"]},
             {"step": 4, "entries": [{"id": "c", "tokens": a[:150], "want": [149]}], "end": ["c"]}]
    r = subprocess.run([str(ROOT / "bin" / "trace_run"), "--model", str(tmp_path / "model"), "--dtype", "float32", "--out", str(out), "--max-tokens", "256"],
                       input="\n".join(map(json.dumps, steps)) + "\n", cwd=ROOT, capture_output=True, text=True, timeout=110)
    assert r.returncode == 0, r.stderr
    assert [x for x in r.stdout.splitlines() if x.startswith("done ")] == [f"done {i}" for i in range(5)]
    read = lambda i: torch.from_numpy(np.fromfile(out / f"{i}.f32", dtype="<f4").reshape(-1, cfg["vocab"]))   # noqa: E731
    check(read(0), wants[0][[39, 2]], torch.float32, "step 0")
    assert not (out / "1.f32").exists()
    got = read(2)
    check(got[:1], wants[0][[129]], torch.float32, "step 2 a")
    check(got[1:], wants[1][[1]], torch.float32, "step 2 b")
    check(read(3), wants[1][[96]], torch.float32, "step 3")
    check(read(4), wants[0][[149]], torch.float32, "step 4")


def test_qwen3_takes_portions_and_checkpoints_too(gpu, tmp_path):
    """The Qwen3 model through the same machinery: a checkpoint folder, portions behind cached tokens, mixed batches and the
    chunked scheduler give the logits and tokens of whole prompts."""
    from safetensors.torch import save_file
    from nano_vllm_ninetoothed_amd.engine import Engine
    g = torch.Generator().manual_seed(0)
    hid, ff, vocab, layers, hq, hkv, d = 256, 512, 512, 2, 4, 2, 128
    t = {"model.embed_tokens.weight": (vocab, hid), "model.norm.weight": (hid,)}
    for i in range(layers):
        p = f"model.layers.{i}."
        t.update({p + "input_layernorm.weight": (hid,), p + "post_attention_layernorm.weight": (hid,), p + "self_attn.q_norm.weight": (d,),
                  p + "self_attn.k_norm.weight": (d,), p + "self_attn.q_proj.weight": (hq * d, hid), p + "self_attn.k_proj.weight": (hkv * d, hid),
                  p + "self_attn.v_proj.weight": (hkv * d, hid), p + "self_attn.o_proj.weight": (hid, hq * d), p + "mlp.gate_proj.weight": (ff, hid),
                  p + "mlp.up_proj.weight": (ff, hid), p + "mlp.down_proj.weight": (hid, ff)})
    w = {k: ((torch.randn(s, generator=g) * s[-1] ** -0.5) if len(s) == 2 else 1 + 0.1 * torch.randn(s, generator=g)).bfloat16() for k, s in t.items()}
    folder = tmp_path / "qwen"
    folder.mkdir()
    save_file(w, str(folder / "model.safetensors"))
    (folder / "config.json").write_text(json.dumps(dict(architectures=["Qwen3ForCausalLM"], num_hidden_layers=layers, hidden_size=hid, num_attention_heads=hq,
                                                        num_key_value_heads=hkv, head_dim=d, intermediate_size=ff, vocab_size=vocab, rms_norm_eps=1e-6,
                                                        rope_theta=1e6, tie_word_embeddings=True, max_position_embeddings=2048)))
    eng = Engine.from_pretrained(folder, num_blocks=12)
    s = torch.randint(0, vocab, (300,), generator=g).tolist()
    whole = feed(eng, s, eng.open_sequence(), [300]).float().cpu()
    for cuts in ([299, 300], [2, 130, 256, 258, 300]):
        assert logit_error(feed(eng, s, eng.open_sequence(), cuts), whole).max() < 4e-2
    prompts = [s[:40], s[100:101], s[30:90]]
    outs = []
    for chunked in (False, True):
        e = Engine.from_pretrained(folder, num_blocks=12, chunked_prefill=chunked, max_num_batched_tokens=128)
        outs.append(e.generate(prompts, 6)[0])
    same = sum(a == b for x, y in zip(*outs) for a, b in zip(x, y))
    assert same >= 12 and [len(x) for x in outs[1]] == [6, 6, 6]
    with pytest.raises(ValueError):
        Engine.from_pretrained(folder, dtype=torch.float32)
