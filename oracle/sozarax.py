"""TEST INFRASTRUCTURE ONLY: a plain, slow restatement of the Sozarax design, one function per mechanism, on the CPU and (by
default) in float64.  Nothing here is shared with the product path: no caches, no chunks, no packed projections; the
recurrence runs token by token, attention is a full score matrix, experts are a loop over tokens.

Weights come as a dict of tensors under the checkpoint's names, the configuration as the dict of config.json.
"""
from __future__ import annotations

import contextlib
import math

import torch

_round = None      # see sixteen_bit_products


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


def silu(x):
    return x * sigmoid(x)


def unit_rms(x, eps):
    """x over the root of its mean square along the last dimension, eps inside the root."""
    return x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps)


def norm(x, w, eps):
    return unit_rms(x, eps) * w


# ---------------------------------------------------------------------------------------------------- time mixing
def shifted(h, before=None):
    """Row t is row t-1 of h; row 0 is `before` (zeros at the start of a sequence)."""
    first = torch.zeros_like(h[:1]) if before is None else before[None, :]
    return torch.cat((first, h[:-1]), dim=0)


def token_mix(h, mu, before=None):
    """A step of size mu from every row towards the row in front of it."""
    return h + (shifted(h, before) - h) * mu


def channel_decay(x, w1, w2, w0):
    """Decay per channel, between 0 and 1: exp(-exp(W2 tanh(W1 x) + w0))."""
    return torch.exp(-torch.exp(product(torch.tanh(product(x, w1)), w2) + w0))


def channel_recurrence(r, k, v, decay, bonus, state=None):
    """o_t = (S_(t-1) + (u k_t) v_t^T)^T r_t, then S_t = diag(decay_t) S_(t-1) + k_t v_t^T.
    r, k, decay [T, H, D], v [T, H, V], bonus u [H, D]; returns (o [T, H, V], final S [H, D, V])."""
    T, H, D = r.shape
    S = torch.zeros((H, D, v.shape[-1]), dtype=r.dtype) if state is None else state.clone()
    out = []
    for t in range(T):
        kv = k[t][:, :, None] * v[t][:, None, :]
        out.append(((S + bonus[:, :, None] * kv) * r[t][:, :, None]).sum(dim=1))
        S = decay[t][:, :, None] * S + kv
    return torch.stack(out), S


def time_mixing(h, w, m, eps):
    H, D = m["heads"], m["dim"]
    T = h.shape[0]
    mix = {n: token_mix(h, w["mu." + n]) for n in "rkvgw"}
    r, k, v = (product(mix[n], w[n]).view(T, H, D) for n in "rkv")
    decay = channel_decay(mix["w"], w["w1"], w["w2"], w["w0"]).view(T, H, D)
    o, _ = channel_recurrence(r, k, v, decay, w["u"])
    o = unit_rms(stored(o), eps).reshape(T, H * D) * w["norm"]
    return product(o * silu(product(mix["g"], w["g"])), w["o"])


# ---------------------------------------------------------------------------------------------------- attention
def query_temperature(positions, coef, every):
    p = positions.to(torch.float64)
    return 1 + coef * torch.log(torch.floor((p + 1) / every) + 1)


def distance_slopes(heads):
    return torch.pow(torch.tensor(2.0, dtype=torch.float64), -8.0 * (torch.arange(heads, dtype=torch.float64) + 1) / heads)


def biased_attention(q, k, v, scale, slopes):
    """Causal softmax over scale q.k - slope (i - j).  q [T, H, D], k [T, G, D], v [T, G, V]; head h reads group h / (H/G)."""
    T, H, _ = q.shape
    per = H // k.shape[1]
    k, v = k.repeat_interleave(per, dim=1), v.repeat_interleave(per, dim=1)
    i = torch.arange(T)
    s = torch.einsum("ihd,jhd->hij", q, k) * scale
    s = s - slopes.to(s.dtype)[:, None, None] * (i[:, None] - i[None, :])[None].to(s.dtype)
    s = s.masked_fill((i[None, :] > i[:, None])[None], -math.inf)
    p = torch.exp(s - s.max(dim=-1, keepdim=True).values)
    p = p / p.sum(dim=-1, keepdim=True)
    return torch.einsum("hij,jhd->ihd", p, v)


def attention(h, w, m, eps):
    H, G, D, V = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    T = h.shape[0]
    q = norm(product(h, w["q"]), w["q.norm"], eps)
    k = norm(product(h, w["k"]), w["k.norm"], eps)
    t = m["q_temp"]
    q = q * query_temperature(torch.arange(T), t["coef"], t["every"])[:, None].to(q.dtype)
    o = biased_attention(stored(q).view(T, H, D), stored(k).view(T, G, D), product(h, w["v"]).view(T, G, V), m["scale"], distance_slopes(H))
    return product(o.reshape(T, H * V), w["o"])


# ---------------------------------------------------------------------------------------------------- feed-forward
def squared_relu(x):
    return torch.clamp(x, min=0) ** 2


def dense(h, w):
    return product(squared_relu(product(h, w["up"])), w["down"])


def route(h, router, top):
    """(chosen experts [T, top], their sigmoid scores)"""
    return tuple(reversed(torch.topk(sigmoid(h @ router.T), top, dim=-1)))


def expert(x, w):
    return product(silu(product(x, w["gate"])) * product(x, w["up"]), w["down"])


def mixture(h, w, m):
    """Every chosen expert sees the input times its score."""
    chosen, score = route(h, w["router"], m["router"]["top"])
    out = torch.zeros_like(h)
    for e in range(m["router"]["experts"]):
        t, slot = (chosen == e).nonzero(as_tuple=True)
        if t.numel():
            out.index_add_(0, t, expert(h[t] * score[t, slot][:, None], {n: w[f"e{e}.{n}"] for n in ("gate", "up", "down")}))
    return out


# ---------------------------------------------------------------------------------------------------- the model
def _under(weights, prefix, dtype):
    return {k[len(prefix):]: v.to(dtype) for k, v in weights.items() if k.startswith(prefix)}


def layer_order(config):
    """Layer numbers in the order in which they run."""
    n, loop = len(config["layers"]), config.get("loop")
    if not loop:
        return list(range(n))
    return list(range(loop["start"])) + list(range(loop["start"], loop["stop"])) * loop["times"] + list(range(loop["stop"], n))


def forward(config, weights, tokens, dtype=torch.float64, layers_out=None):
    """Logits [T, vocab] of one sequence.  layers_out: a list that receives the residual stream after every layer run."""
    eps = config["norm"]["eps"]
    tokens = torch.as_tensor(tokens, dtype=torch.int64)
    x = weights["embed"].to(dtype)[tokens] * config["embedding"]["scale"]
    for i in layer_order(config):
        layer, pre = config["layers"][i], f"l{i}."
        nw = {n: weights[pre + n].to(dtype) for n in ("norm1", "norm1b", "norm2", "norm2b") if pre + n in weights}
        mixer = {"wkv": time_mixing, "attention": attention}[layer["type"]]
        y = mixer(norm(x, nw["norm1"], eps), _under(weights, pre + "mix.", dtype), layer["mixer"], eps)
        x = x + norm(y, nw["norm1b"], eps)
        if layer.get("mlp") is not None:
            h, w = norm(x, nw["norm2"], eps), _under(weights, pre + "mlp.", dtype)
            y = dense(h, w) if layer["mlp"]["kind"] == "dense" else mixture(h, w, layer["mlp"])
            x = x + norm(y, nw["norm2b"], eps)
        if layers_out is not None:
            layers_out.append(x.clone())
    return product(norm(x, weights["final.norm"].to(dtype), eps), weights["head"].to(dtype))


def greedy(config, weights, prompt, n, dtype=torch.float64):
    """n greedily chosen tokens after the prompt, recomputing the whole sequence for each."""
    seq = list(prompt)
    for _ in range(n):
        seq.append(int(forward(config, weights, seq, dtype)[-1].argmax()))
    return seq[len(prompt):]
