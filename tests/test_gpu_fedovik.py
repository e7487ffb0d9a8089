"""GPU: Fedovik models of several shapes through the engine - its batches, cache manager, scheduler, sampler, command line -
against the plain float64 restatement in oracle/fedovik.py."""
import json
import subprocess
import sys
from pathlib import Path

import numpy as np
import pytest
import torch

import model_harness as H
from fedovik_cases import CONFIGS, attention, config, memory, parallel, random_tokens, random_weights
from nepulix_cases import logit_error, write_checkpoint
from oracle import fedovik as O

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


def leaves(mixer):
    """The mixers with a cache or state of their own inside joined ones."""
    parts = getattr(mixer, "parts", None)
    if parts is None:
        return [mixer] if hasattr(mixer, "state") or hasattr(mixer, "k_pages") else []
    return [x for p in parts for x in leaves(p)]


@pytest.fixture(scope="module")
def case():
    """(config, weights, tokens by number, oracle logits by number), computed once per configuration."""
    done = {}

    def get(name):
        if name not in done:
            cfg, w = CONFIGS[name], random_weights(CONFIGS[name], 11)
            seqs = [random_tokens(cfg, n, 100 + i) for i, n in enumerate(LENGTHS)]
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
    assert [i for i, _ in seen] == list(range(len(layers))) and len(layers) == len(O.passes(cfg))
    for (i, a), b in zip(seen, layers):
        err = ((a.double().cpu() - b).norm(dim=1) / b.norm(dim=1)).max().item()
        assert err <= (2e-5 if dtype == torch.float32 else 8e-2), f"layer run {i}: {err:.3g}"


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", NAMES)
def test_portions_and_token_by_token(gpu, case, name, dtype):
    """Prompts cut anywhere, down to two tokens and to single ones; the same slot and pages serve one run after another."""
    cfg, w, seqs, wants = case(name)
    eng = engine(gpu, cfg, w, dtype, tokens=320, slots=1)          # just enough for one sequence: everything is used again
    n = len(seqs[0])
    plans = {"two by two": list(range(2, n, 2)) + [n], "one by one": list(range(1, 101)) + [n], "prefill, then decode": [200] + list(range(201, n + 1)),
             "borders": [15, 16, 17, 31, 32, 33, 63, 65, 96, 98, 127, 128, 129, 191, 255, 257, n], "large after small": [3, 67, 70, 198, n],
             "windows": [24, 25, 26, 33, 49, 50, 64, 65, 70, 72, 90, 111, 180, 200, n]}
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


@pytest.mark.parametrize("name", NAMES)
def test_what_pages_and_slots_held_before_does_not_matter(gpu, case, name):
    """Garbage in every page and slot in front of a run, whose bits are those of a run on zeros."""
    cfg, w, seqs, wants = case(name)
    outs = []
    for garbage in (False, True):
        eng = engine(gpu, cfg, w, torch.bfloat16, tokens=320, slots=1)
        if garbage:
            for _, sublayers, _ in eng.model.runs:
                for mixer in leaves(sublayers):
                    for t in ("k_pages", "v_pages", "state", "ring", "top"):
                        if hasattr(mixer, t):
                            getattr(mixer, t).fill_(float("nan"))
        outs.append(H.feed(eng, seqs[0], eng.open_sequence(), [1, 40, 41, 150, 290, 291, 300]))
    assert torch.isfinite(outs[1]).all() and logit_error(outs[1], outs[0].double().cpu()).max() < 1e-6


def test_every_run_of_a_layer_has_its_own_cache_and_state(gpu, case):
    cfg, w, _, _ = case("odd")
    eng = engine(gpu, cfg, w, torch.float32)
    mixers = [m for _, sublayers, _ in eng.model.runs for m in leaves(sublayers)]
    states = [m.state.data_ptr() for m in mixers if hasattr(m, "state")]
    pages = [m.k_pages.data_ptr() for m in mixers if hasattr(m, "k_pages")]
    assert len(states) == len(set(states)) == 3 + 3 + 1 and len(pages) == len(set(pages)) == 1 + 3
    assert len({sublayers.w_in.data_ptr() for _, sublayers, _ in eng.model.runs}) == 4


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["odd", "plain"])
def test_long_decoding(gpu, name, dtype):
    """Hundreds of decoded tokens behind a short prompt, across many pages, windows and chunks."""
    cfg = CONFIGS[name]
    w = random_weights(cfg, 3)
    s = random_tokens(cfg, 420, 5)
    eng = engine(gpu, cfg, w, dtype, tokens=448, block_size=64)
    H.check(H.feed(eng, s, eng.open_sequence(), [7] + list(range(8, 421))), H.Wanted(O, cfg, w, s), dtype, "long decoding")


def loud_case(layer, window=None):
    """One layer whose queries all ask for the tokens of one kind, by a channel that only these have."""
    cfg = config(64, 64, [(layer, 24)], embedding_scale=1.0)
    w = random_weights(cfg, 2)
    prefix = "l0.mix.left." if layer["type"] == "parallel" else "l0.mix."
    d = (layer["mixer"].get("left") or layer["mixer"])["dim"]
    loud = 63
    for n, channel in (("q", 20), ("k", 21)):
        w[prefix + n][:, 20:22] = 0
        w[prefix + n][d - 1::d, channel] = 3.0      # a dimension that is not turned
    w["l0.norm1"][20:22], w["l0.norm1.b"][20:22] = 1, 0
    w["embed"][:, 20], w["embed"][loud, 21], w["embed"][:loud, 21] = 2.5, 6.0, 0.0
    return cfg, w, loud


@pytest.mark.parametrize("dtype", DTYPES)
def test_keys_that_stand_out_at_the_edges_of_a_window(gpu, dtype):
    """Tokens that all others ask for, just inside and just outside the window of single tokens: one wrong key is most of the weight."""
    n, window = 150, 40
    cfg, w, loud = loud_case(parallel((4, 2, 32, 32, window, 0.5), (2, 2, 16, 16, 4), 2.0, 0.3))
    base = [t % loud for t in random_tokens(cfg, n, 8)]
    for at in ((n - window,), (n - window - 1,), (63, 64), (95, 96), (9, 70, 109)):
        s = list(base)
        for p in at:
            s[p] = loud
        want = H.Wanted(O, cfg, w, s)
        for cuts in ([n], [30] + list(range(31, n + 1)), [60, 62, 100, 140, n]):
            eng = engine(gpu, cfg, w, dtype, tokens=160, slots=1)
            H.check(H.feed(eng, s, eng.open_sequence(), cuts), want, dtype, (at, cuts))
        # the token behind the last one that sees it knows nothing of it through attention
        seen, not_seen = at[-1] + window - 1, at[-1] + window
        moved = logit_error(want.logits, O.forward(cfg, w, base))
        if not_seen < n and len(at) == 1:
            assert moved[seen] > 3 * moved[not_seen]


@pytest.mark.parametrize("dtype", DTYPES)
def test_a_far_token_among_hundreds(gpu, dtype):
    """Attention without a softmax: a key far back whose sigmoid is one among hundreds that are nearly nothing."""
    n = 700
    layer = attention(4, 2, 32, 32, 16, 0.5)
    cfg, w, loud = loud_case(layer)
    w["l0.mix.pb"] = torch.full((4,), -9.0).bfloat16()
    base = [t % loud for t in random_tokens(cfg, n, 8)]
    for p in (0, 1, 63, 64, 300):
        s = list(base)
        s[p] = loud
        want = H.Wanted(O, cfg, w, s)
        moved = logit_error(want.logits, O.forward(cfg, w, base))
        assert moved[p + 1:].median() > 0.01 and moved[p + 1:].min() > 1e-3      # every later token sees it
        for cuts in ([n], [650] + list(range(651, n + 1)), [64, 66, 129, 500, n]):
            eng = engine(gpu, cfg, w, dtype, tokens=704, block_size=64, slots=1)
            H.check(H.feed(eng, s, eng.open_sequence(), cuts), want, dtype, (p, cuts))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("layer", [memory(2, 32, 24, 15.0), parallel((2, 1, 16, 16, 8, 0.5), (2, 1, 32, 24, 4), 0.3, 2.0)], ids=["memory", "delta"])
def test_a_state_that_forgets_little(gpu, layer, dtype):
    """The first tokens still matter hundreds of tokens later, whatever the cuts, and in decoding."""
    n = 500
    cfg = config(64, 64, [(layer, 24), (layer, None)], embedding_scale=1.0)
    w = random_weights(cfg, 4)
    for i in (0, 1):
        if layer["type"] == "mlstm":
            w[f"l{i}.mix.f"] = w[f"l{i}.mix.f"] * 0
            w[f"l{i}.mix.f.b"] = torch.full((2,), 14.0).bfloat16()
        else:
            w[f"l{i}.mix.right.dt_bias"] = torch.full((64,), -14.0).bfloat16()
            w[f"l{i}.mix.right.b"] = w[f"l{i}.mix.right.b"] * 0 - 0.02
    s = random_tokens(cfg, n, 6)
    other = [(t + 7) % 64 for t in s[:6]] + s[6:]
    want = H.Wanted(O, cfg, w, s)
    assert logit_error(want.logits, O.forward(cfg, w, other))[-50:].median() > 5e-3
    for cuts in ([n], [9, 40, 300] + list(range(301, n + 1)), [2, 4, 21, 37, 101, 257, 259, n]):
        eng = engine(gpu, cfg, w, dtype, tokens=512, block_size=64, slots=1)
        H.check(H.feed(eng, s, eng.open_sequence(), cuts), want, dtype, cuts)


def test_a_page_size_that_is_no_multiple_of_a_stage(gpu, case):
    """Pages of 24 tokens: single rows take the plain form."""
    cfg, w, seqs, wants = case("plain")
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


@pytest.mark.parametrize("name", ["large", "wide", "odd", "plain"])
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
    assert e.median() < 2e-2 and e.max() < 0.1


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
    assert "does not use" not in r.stderr
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
