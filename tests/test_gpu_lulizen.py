"""GPU: Lulizen models of several shapes through the engine - its batches, cache manager, scheduler, sampler, command line -
against the plain float64 restatement in oracle/lulizen.py."""
import json
import subprocess
import sys
from pathlib import Path

import numpy as np
import pytest
import torch

import model_harness as H
from lulizen_cases import CONFIGS, chunked, config, dense, moe, random_tokens, random_weights, settled_tokens, windowed
from nepulix_cases import logit_error, write_checkpoint
from oracle import lulizen as O

pytestmark = pytest.mark.gpu
ROOT = Path(__file__).resolve().parent.parent
DTYPES = [torch.float32, torch.bfloat16]
NAMES = list(CONFIGS)
LENGTHS = (300, 97, 65, 1)


def made(cfg):
    from nano_vllm_ninetoothed_amd.models import parse_config
    return parse_config(cfg)


def engine(gpu, cfg, *args, **kw):
    return H.engine(gpu, made(cfg), *args, **kw)


@pytest.fixture(scope="module")
def case():
    """(config, weights, tokens by number, oracle logits by number), computed once per configuration."""
    done = {}

    def get(name):
        if name not in done:
            cfg, w = CONFIGS[name], random_weights(CONFIGS[name], 11)
            seqs = [settled_tokens(cfg, w, n, 100 + i) for i, n in enumerate(LENGTHS)]
            done[name] = (cfg, w, seqs, [H.Wanted(O, cfg, w, s) for s in seqs])
        return done[name]
    return get


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", NAMES)
def test_whole_prompts_and_every_layer(gpu, case, name, dtype):
    cfg, w, seqs, wants = case(name)
    eng = engine(gpu, cfg, w, dtype)
    for s, want in zip(seqs, wants):
        q = eng.open_sequence()
        H.check(H.feed(eng, s, q, [len(s)]), want, dtype, f"{len(s)} tokens")
        eng.close_sequence(q)
    layers, seen = [], []
    O.forward(cfg, w, seqs[2], layers_out=layers)
    eng.model.layer_hook = lambda i, x: seen.append((i, x.clone()))
    H.feed(eng, seqs[2], eng.open_sequence(), [len(seqs[2])])
    assert [i for i, _ in seen] == list(range(len(layers))) and len(layers) == len(cfg["layers"])
    for (i, a), b in zip(seen, layers):
        err = ((a.double().cpu() - b).norm(dim=1) / b.norm(dim=1)).max().item()
        assert err <= (1e-5 if dtype == torch.float32 else 6e-2), f"layer run {i}: {err:.3g}"


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", NAMES)
def test_portions_and_token_by_token(gpu, case, name, dtype):
    """Prompts cut anywhere, down to two tokens and to single ones; the same slot and pages serve one run after another."""
    cfg, w, seqs, wants = case(name)
    eng = engine(gpu, cfg, w, dtype, tokens=320, slots=1)          # just enough for one sequence: everything is used again
    n = len(seqs[0])
    plans = {"two by two": list(range(2, n, 2)) + [n], "one by one": list(range(1, 101)) + [n], "prefill, then decode": [200] + list(range(201, n + 1)),
             "borders": [15, 16, 17, 31, 32, 33, 63, 65, 96, 98, 127, 128, 129, 191, 255, 257, n], "large after small": [3, 67, 70, 198, n],
             "chunks and windows": [24, 25, 26, 36, 37, 38, 49, 50, 73, 75, 90, 111, 180, 200, n]}
    for what, cuts in plans.items():
        q = eng.open_sequence()
        H.check(H.feed(eng, seqs[0], q, cuts), wants[0], dtype, what)
        eng.close_sequence(q)
        assert len(eng.free_blocks) == eng.num_blocks and len(eng.cache.free_slots) == eng.cache.num_slots


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", NAMES)
def test_mixed_batches(gpu, case, name, dtype):
    """Unequal requests side by side, each against itself alone."""
    cfg, w, seqs, wants = case(name)
    eng = engine(gpu, cfg, w, dtype, tokens=32 * 24, slots=4)
    got = H.mixed_batches(eng, seqs, [0, 1, 2, 3, 1, 2, 1, 3, 2, 1])
    assert len(got) == 10
    for i, pos, logits in got:
        H.check(logits, wants[i][pos], dtype, f"request {i}")


@pytest.mark.parametrize("name", ["odd", "large"])
def test_what_pages_and_slots_held_before_does_not_matter(gpu, case, name):
    """Garbage in every page and slot in front of a run, whose bits are those of a run on zeros."""
    cfg, w, seqs, wants = case(name)
    outs = []
    for garbage in (False, True):
        eng = engine(gpu, cfg, w, torch.bfloat16, tokens=320, slots=1)
        if garbage:
            eng.model.before.fill_(7)
            for _, mixer, *_ in eng.model.runs:
                mixer.k_pages.fill_(float("nan"))
                mixer.v_pages.fill_(float("nan"))
        outs.append(H.feed(eng, seqs[0], eng.open_sequence(), [1, 40, 41, 150, 290, 291, 300]))
    assert torch.isfinite(outs[1]).all() and logit_error(outs[1], outs[0].double().cpu()).max() < 1e-6


def test_every_run_of_a_layer_has_its_own_cache(gpu, case):
    cfg, w, _, _ = case("odd")
    eng = engine(gpu, cfg, w, torch.float32)
    mixers = [m for _, m, *_ in eng.model.runs]
    assert len(mixers) == 6 and len({m.k_pages.data_ptr() for m in mixers}) == len({m.v_pages.data_ptr() for m in mixers}) == 6
    assert len({m.qkv.data_ptr() for m in mixers}) == 3


def test_the_token_in_front_survives_between_steps(gpu, case):
    """Two requests whose portions end on different tokens take turns; a slot's next holder starts without one."""
    cfg, w, seqs, wants = case("odd")
    eng = engine(gpu, cfg, w, torch.float32, slots=2)
    a, b = eng.open_sequence(), eng.open_sequence()
    for i in range(30):
        q, s, want = ((a, seqs[0], wants[0]), (b, seqs[1], wants[1]))[i % 2]
        at = i // 2
        H.check(eng.run_portions([(q, s[at:at + 1], [0])]), want[[at]], torch.float32, f"step {i}")
    eng.close_sequence(a)
    c = eng.open_sequence()
    H.check(eng.run_portions([(c, seqs[2][:1], [0])]), wants[2][[0]], torch.float32, "a used slot")


@pytest.mark.parametrize("dtype", DTYPES)
def test_long_decoding(gpu, dtype):
    """Hundreds of decoded tokens behind a short prompt, across many pages, chunks and windows."""
    cfg = CONFIGS["odd"]
    w = random_weights(cfg, 3)
    s = settled_tokens(cfg, w, 420, 5)
    eng = engine(gpu, cfg, w, dtype, tokens=448, block_size=64)
    H.check(H.feed(eng, s, eng.open_sequence(), [7] + list(range(8, 421))), H.Wanted(O, cfg, w, s), dtype, "long decoding")


@pytest.mark.parametrize("dtype", DTYPES)
def test_keys_that_stand_out_at_the_edges(gpu, dtype):
    """Tokens that all others ask for, in front of, at and behind every edge of what a token sees: one wrong key is most of the weight.
    The last token's logits after prompts and after decoding, with everything else of the model small."""
    cfg = config(128, 64, [(chunked(4, 2, 32, 32, 32, 48, 1.0, 30.0), dense(40)), (windowed(4, 2, 32, 32, 16, 40, 10, 1.0, 30.0), moe(16, 8, 2, 2, 1, 24))], (31, 3, 5))
    w = random_weights(cfg, 2)
    loud = 63
    for i in (0, 1):      # the loud token's key channel answers every query's
        for n in ("q", "k"):
            w[f"l{i}.mix.{n}"][:, 20] = 0
            w[f"l{i}.mix.{n}"][31::32, 20] = 1.5 if n == "q" else 0      # dimension 31 turns least, or not at all
    w["embed"][:, 20], w["embed"][loud, 21], w["embed"][:loud, 21] = 2.5, 6.0, 0.0
    for i in (0, 1):
        w[f"l{i}.mix.k"][:, 21] = 0
        w[f"l{i}.mix.k"][31::32, 21] = 1.5
    n = 150
    base = [t % loud for t in settled_tokens(cfg, w, n, 8)]
    for at in ((95,), (96,), (9,), (10,), (n - 41,), (n - 40,), (143, 144), (9, 95, 109)):
        s = list(base)
        for p in at:
            s[p] = loud
        with O.watching_choices() as margins:
            logits = O.forward(cfg, w, s)
        sure = torch.stack(margins).min(0).values > 4e-3
        want = H.Wanted(O, cfg, w, s)
        for cuts in ([n], [30] + list(range(31, n + 1)), [60, 62, 100, 140, n]):
            eng = engine(gpu, cfg, w, dtype, tokens=160, slots=1)
            got = H.feed(eng, s, eng.open_sequence(), cuts)
            H.check(got[sure.to(got.device)], want[sure], dtype, (at, cuts))
        assert (logits - O.forward(cfg, w, base)).abs().max() > 0.05


def test_a_page_size_that_is_no_multiple_of_a_stage(gpu, case):
    """Pages of 24 tokens: single rows take the plain form."""
    cfg, w, seqs, wants = case("large")
    for dtype in DTYPES:
        eng = engine(gpu, cfg, w, dtype, tokens=240, block_size=24)
        H.check(H.feed(eng, seqs[1], eng.open_sequence(), [50, 51, 52, 90, 97]), wants[1], dtype, "pages of 24")


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
        outs, _ = eng.generate(prompts, n_out)
        assert outs == want
        assert len(eng.free_blocks) == 12 and len(eng.cache.free_slots) == 4 and not eng.running and not eng.waiting


@pytest.mark.parametrize("name", ["large", "wide", "odd"])
def test_graph_replay_equals_eager_decode(gpu, name):
    """The captured decode step in bf16, replayed with eager work in between, against the eager step."""
    cfg = CONFIGS[name]
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
            for j, q in enumerate(seqs):      # the same tokens either way
                q.token_ids[-1] = (17 * it + j) % cfg["vocab"]
            ids, pos, ctx = eng._prepare_decode(seqs)
            rows.append((eng._decode_replay(ids, pos, ctx) if graphs else eng.forward(ids, pos, ctx)).float().cpu())
            torch.cuda.synchronize()
            for q in seqs:
                q.num_cached = len(q)
                q.token_ids.append(0)
        outs.append(torch.stack(rows))
    e = logit_error(outs[0].flatten(0, 1), outs[1].flatten(0, 1))
    assert e.median() < 2e-2 and e.max() < 0.3      # another product form may tip a close choice of experts


def test_checkpoint_folder_command_line_and_trace(gpu, case, tmp_path):
    """A folder with config.json and safetensors through Engine.from_pretrained, the generate command and a replayed trace."""
    cfg, w, seqs, wants = case("odd")
    write_checkpoint(tmp_path / "model", cfg, w)
    from nano_vllm_ninetoothed_amd.engine import Engine
    eng = Engine.from_pretrained(tmp_path / "model", dtype=torch.float32, num_blocks=8, block_size=64, max_num_seqs=2, max_model_len=512)
    H.check(H.feed(eng, seqs[1], eng.open_sequence(), [len(seqs[1])]), wants[1], torch.float32, "from_pretrained")
    prompts = [seqs[2][:20], seqs[1][:3]]
    want = [O.greedy(cfg, w, p, 5) for p in prompts]
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
             {"step": 3, "entries": [{"id": "b", "tokens": b[2:97], "want": [94]}], "end": ["b"]}]
    r = subprocess.run([str(ROOT / "bin" / "trace_run"), "--model", str(tmp_path / "model"), "--dtype", "float32", "--out", str(out), "--max-tokens", "256"],
                       input="\n".join(map(json.dumps, steps)) + "\n", cwd=ROOT, capture_output=True, text=True, timeout=110)
    assert r.returncode == 0, r.stderr
    assert [x for x in r.stdout.splitlines() if x.startswith("done ")] == [f"done {i}" for i in range(4)]
    read = lambda i: torch.from_numpy(np.fromfile(out / f"{i}.f32", dtype="<f4").reshape(-1, cfg["vocab"]))   # noqa: E731
    H.check(read(0), wants[0][[39, 2]], torch.float32, "step 0")
    assert not (out / "1.f32").exists()
    got = read(2)
    H.check(got[:1], wants[0][[129]], torch.float32, "step 2 a")
    H.check(got[1:], wants[1][[1]], torch.float32, "step 2 b")
    H.check(read(3), wants[1][[96]], torch.float32, "step 3")


def test_random_weights_run_without_a_checkpoint(gpu):
    from nano_vllm_ninetoothed_amd.engine import Engine
    eng = Engine(made(CONFIGS["large"]), num_blocks=8, block_size=64, max_num_seqs=2, max_model_len=512)
    outs, _ = eng.generate([[1, 2, 3], [4] * 70], 4)
    assert [len(o) for o in outs] == [4, 4]
