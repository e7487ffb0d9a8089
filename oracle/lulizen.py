"""TEST INFRASTRUCTURE ONLY: a plain, slow restatement of the Lulizen design, one function per mechanism, on the CPU and (by
default) in float64.  Nothing here is shared with the product path: no caches, no packed projections; attention is a full score
matrix with a mask of pairs, experts are a loop over experts.

Weights come as a dict of tensors under the checkpoint's names, the configuration as the dict of config.json.
"""
from __future__ import annotations

import contextlib
import math

import torch

_round = None      # see sixteen_bit_products
_margins = None    # see watching_choices


@contextlib.contextmanager
def sixteen_bit_products(seed=0):
    """Inside, every matrix product takes and gives values rounded to bfloat16 (to nearest for seed 0, else stochastically), and so
    are the values marked stored(): what rounding alone does to the result of a 16-bit run.  The router's product is exempt."""
    global _round
    g = torch.Generator().manual_seed(seed)

    def nearest(x):
        return x.to(torch.bfloat16).to(x.dtype)

    def stochastic(x):
        step = torch.exp2(torch.floor(torch.log2(x.abs().clamp(min=1e-30))) - 7)
        return nearest(x + (torch.rand(x.shape, generator=g, dtype=x.dtype) - 0.5) * step)

    _round = stochastic if seed else nearest
    try:
        yield
    finally:
        _round = None


@contextlib.contextmanager
def watching_choices():
    """Inside, every choice of experts appends how far it is from another one: per token the smaller of two gaps, between the last
    expert taken and the first one left, and (halved: two scores add up) between the last group kept and the first one dropped."""
    global _margins
    _margins = []
    try:
        yield _margins
    finally:
        _margins = None


def product(x, w):
    """x W^T"""
    if _round is None:
        return x @ w.T
    return _round(_round(x) @ w.T)


def stored(x):
    """An intermediate that a 16-bit run keeps in 16 bits."""
    return x if _round is None else _round(x)


def sigmoid(x):
    return 1 / (1 + torch.exp(-x))


def layer_norm(x, w, eps):
    d = x - x.mean(dim=-1, keepdim=True)
    return d / torch.sqrt((d * d).mean(dim=-1, keepdim=True) + eps) * w


def rms_norm(x, w, eps):
    return x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps) * w


# ---------------------------------------------------------------------------------------------------- embedding
def bigram_rows(tokens, buckets, mul_prev, mul_cur):
    """Row of the table of pairs per token: a hash of the token and the one in front; a row of its own for the first."""
    rows = [buckets]
    for before, now in zip(tokens[:-1], tokens[1:]):
        rows.append((before * mul_prev + now * mul_cur) % buckets)
    return rows


def embedding(tokens, table, pairs, bigram):
    x = table[torch.as_tensor(tokens)]
    return x + pairs[torch.as_tensor(bigram_rows([int(t) for t in tokens], bigram["buckets"], bigram["mul_prev"], bigram["mul_cur"]))]


# ---------------------------------------------------------------------------------------------------- attention
def rotate(x, positions, base, dims):
    """x [T, heads, D]: the pairs (i, i + dims/2) of the first `dims` elements turn by position * base^(-2i/dims)."""
    half = dims // 2
    f = torch.tensor([float(base) ** (-2.0 * i / dims) for i in range(half)], dtype=torch.float64)
    a = (positions.to(torch.float64)[:, None] * f)[:, None, :]
    c, s = a.cos().to(x.dtype), a.sin().to(x.dtype)
    u, v = x[..., :half], x[..., half:dims]
    return torch.cat((u * c - v * s, v * c + u * s, x[..., dims:]), dim=-1)


def chunk_mask(n, size):
    """[i, j]: i sees j"""
    i, j = torch.arange(n)[:, None], torch.arange(n)[None, :]
    return (j <= i) & (i // size == j // size)


def window_mask(n, size, keep_first):
    i, j = torch.arange(n)[:, None], torch.arange(n)[None, :]
    return (j <= i) & ((i - j < size) | (j < keep_first))


def capped(s, softcap):
    return softcap * torch.tanh(s / softcap)


def masked_attention(q, k, v, scale, softcap, mask, sink=None):
    """q [T, H, D], k [T, G, D], v [T, G, V]; head h reads group h / (H/G); sink [H]: one more term of the denominator."""
    per = q.shape[1] // k.shape[1]
    k, v = k.repeat_interleave(per, dim=1), v.repeat_interleave(per, dim=1)
    s = capped(torch.einsum("ihd,jhd->hij", q, k) * scale, softcap).masked_fill(~mask[None], -math.inf)
    m = s.max(dim=-1, keepdim=True).values
    if sink is not None:
        m = torch.maximum(m, sink[:, None, None])
    p = torch.exp(s - m)
    total = p.sum(dim=-1, keepdim=True)
    if sink is not None:
        total = total + torch.exp(sink[:, None, None] - m)
    return torch.einsum("hij,jhd->ihd", p / total, v)


def attention(h, w, m, eps, kind):
    H, G, D, V = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    T = h.shape[0]
    q, k, v = product(h, w["q"]).view(T, H, D), product(h, w["k"]).view(T, G, D), product(h, w["v"]).view(T, G, V)
    if kind == "attention":
        q, k = rms_norm(q, w["q.norm"], eps), rms_norm(k, w["k.norm"], eps)
        mask, sink = chunk_mask(T, m["mask"]["size"]), w["sink"]
    else:
        mask, sink = window_mask(T, m["mask"]["size"], m["mask"]["keep_first"]), None
    at = torch.arange(T)
    q, k = (stored(rotate(x, at, m["rot"]["base"], m["rot"]["dims"])) for x in (q, k))
    o = masked_attention(q, k, v, m["scale"], m["softcap"], mask, sink)
    if kind == "attention_2":
        o = o * sigmoid(product(h, w["g"]))[:, :, None]
    return product(o.reshape(T, H * V), w["o"])


# ---------------------------------------------------------------------------------------------------- feed-forward
def gelu_tanh(z):
    return 0.5 * z * (1 + torch.tanh(math.sqrt(2 / math.pi) * (z + 0.044715 * z ** 3)))


def dense(h, w):
    return product(gelu_tanh(product(h, w["gate"])) * product(h, w["up"]), w["down"])


def clamped_unit(h, w, limit):
    g = torch.clamp(product(h, w["gate"]), max=limit)
    u = torch.clamp(product(h, w["up"]), min=-limit, max=limit)
    return product(g * sigmoid(1.702 * g) * (u + 1), w["down"])


def choose(scores, correction, top, groups):
    """Experts [T, top] by corrected score, only from the best groups of neighbours (by the sum of a group's two best)."""
    c = scores + correction
    T, E = c.shape
    size = E // groups["count"]
    best = c.view(T, groups["count"], size).topk(min(2, size), dim=-1).values.sum(dim=-1)
    kept = torch.zeros_like(best, dtype=torch.bool).scatter(1, best.topk(groups["keep"], dim=-1).indices, True)
    c = c.masked_fill(~kept.repeat_interleave(size, dim=1), -math.inf)
    if _margins is not None:
        _margins.append(torch.minimum(_gap(c, top), _gap(best, groups["keep"]) / 2))
    return c.topk(top, dim=-1).indices


def _gap(x, n):
    """Between the n-th largest of a row and the next one."""
    s = torch.cat((x.sort(dim=-1, descending=True).values, torch.full((x.shape[0], 1), -math.inf, dtype=x.dtype)), dim=1)
    return s[:, n - 1] - s[:, n]


def route(h, router, correction, m):
    """(chosen experts, their weights)"""
    s = sigmoid(h @ router.T)
    chosen = choose(s, correction, m["top"], m["groups"])
    w = s.gather(1, chosen)
    return chosen, w / (w.sum(dim=-1, keepdim=True) + 1e-20) * m["scale"]


def mixture(h, w, m):
    chosen, weight = route(h, w["router"], w["correction"], m["router"])
    out = torch.zeros_like(h)
    for e in range(m["router"]["experts"]):
        t, slot = (chosen == e).nonzero(as_tuple=True)
        if t.numel():
            y = clamped_unit(h[t], {n: w[f"e{e}.{n}"] for n in ("gate", "up", "down")}, m["expert"]["limit"])
            out.index_add_(0, t, y * weight[t, slot][:, None])
    return out + clamped_unit(h, {n: w[f"shared.{n}"] for n in ("gate", "up", "down")}, m["shared"]["limit"])


# ---------------------------------------------------------------------------------------------------- the model
def _under(weights, prefix, dtype):
    return {k[len(prefix):]: v.to(dtype) for k, v in weights.items() if k.startswith(prefix)}


def forward(config, weights, tokens, dtype=torch.float64, layers_out=None):
    """Logits [T, vocab] of one sequence.  layers_out: a list that receives the residual stream after every layer."""
    eps = config["norm"]["eps"]
    x = embedding(tokens, weights["embed"].to(dtype), weights["bigram"].to(dtype), config["embedding"]["bigram"])
    for i, layer in enumerate(config["layers"]):
        pre = f"l{layer.get('weights_of', i)}."
        nw = {n: weights[pre + n].to(dtype) for n in ("norm1", "norm1b", "norm2", "norm2b") if pre + n in weights}
        y = attention(layer_norm(x, nw["norm1"], eps), _under(weights, pre + "mix.", dtype), layer["mixer"], eps, layer["type"])
        x = x + layer_norm(y, nw["norm1b"], eps)
        if layer.get("mlp") is not None:
            h, w = layer_norm(x, nw["norm2"], eps), _under(weights, pre + "mlp.", dtype)
            y = dense(h, w) if layer["mlp"]["kind"] == "dense" else mixture(h, w, layer["mlp"])
            x = x + layer_norm(y, nw["norm2b"], eps)
        if layers_out is not None:
            layers_out.append(x.clone())
    return product(layer_norm(x, weights["final.norm"].to(dtype), eps), weights["head"].to(dtype))


def greedy(config, weights, prompt, n, dtype=torch.float64):
    """n greedily chosen tokens after the prompt, recomputing the whole sequence for each."""
    seq = list(prompt)
    for _ in range(n):
        seq.append(int(forward(config, weights, seq, dtype)[-1].argmax()))
    return seq[len(prompt):]
