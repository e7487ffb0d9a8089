"""What the GPU tests of models put together layer by layer share: an engine on random weights, limits from what rounding alone
does, portions and mixed batches against the plain restatement of a design."""
import torch

from nepulix_cases import logit_error

LIMIT32 = 2e-5      # float32: per position, of the logits' root mean square


class Wanted:
    """The oracle's logits, and per position what rounding alone does to a 16-bit run (the worst of three realisations, and
    never less than the bulk of the positions shows)."""

    def __init__(self, oracle, cfg, w, tokens, realisations=3):
        self.logits = oracle.forward(cfg, w, tokens)
        errs = []
        for seed in range(realisations):
            with oracle.sixteen_bit_products(seed):
                errs.append(logit_error(oracle.forward(cfg, w, tokens), self.logits))
        e = torch.stack(errs).max(0).values
        self.noise = torch.maximum(e, e.quantile(0.9))

    def __getitem__(self, rows):
        out = object.__new__(Wanted)
        out.logits, out.noise = self.logits[rows], self.noise[rows]
        return out


def engine(gpu, config, w, dtype, tokens=1024, block_size=32, slots=4, **kw):
    """config: a configuration object of a registered model."""
    from nano_vllm_ninetoothed_amd.engine import Engine
    from nano_vllm_ninetoothed_amd.weights import TensorWeights
    return Engine(config, weights=TensorWeights(w, dtype, gpu), num_blocks=-(-tokens // block_size), block_size=block_size,
                  max_num_seqs=slots, max_model_len=tokens, device=str(gpu), **kw)


def check(got, want, dtype, what, limit32=LIMIT32):
    e = logit_error(got, want.logits)
    assert torch.isfinite(e).all(), what
    e = e / (limit32 if dtype == torch.float32 else 3 * want.noise)
    worst, at, over = e.max().item(), int(e.argmax()), int((e > 1).sum())
    assert worst <= 1.5 and over <= max(1, 0.02 * len(e)), f"{what}: {over} of {len(e)} positions over their limit, worst {worst:.3g} at {at}"


def feed(eng, seq, q, cuts):
    """Runs seq in portions that end at cuts, all logits wanted."""
    out, at = [], 0
    for end in cuts:
        out.append(eng.run_portions([(q, seq[at:end], list(range(end - at)))]))
        at = end
    return torch.cat(out)


def mixed_batches(eng, seqs, todo, seed=4):
    """Up to four live requests side by side, portions beside single tokens, some left out of a step; requests come and go, so that
    pages and slots change hands.  Returns (sequence number, positions, their logits) per request of todo."""
    g = torch.Generator().manual_seed(seed)
    todo, live, got = list(todo), [], []
    while todo or live:
        while todo and len(live) < 4 and (len(live) < 2 or torch.rand((), generator=g) < 0.4):
            live.append([todo.pop(0), eng.open_sequence(), 0, []])
        batch = [r for r in live if len(live) == 1 or torch.rand((), generator=g) < 0.8] or live[:1]
        portions = []
        for r in batch:
            left = len(seqs[r[0]]) - r[2]
            n = min(left, [1, 1, 1, 2, 3, 17, 64, 70][int(torch.randint(0, 8, (), generator=g))])
            want = list(range(n)) if n != 17 else [16, 0]
            portions.append((r[1], seqs[r[0]][r[2]:r[2] + n], want))
        logits = eng.run_portions(portions).cpu()
        at = 0
        for r, (_, toks, want) in zip(batch, portions):
            for j in want:
                r[3].append((r[2] + j, logits[at]))
                at += 1
            r[2] += len(toks)
        for r in [r for r in live if r[2] == len(seqs[r[0]])]:
            eng.close_sequence(r[1])
            live.remove(r)
            got.append((r[0], torch.tensor([p for p, _ in r[3]]), torch.stack([x for _, x in r[3]])))
    return got
