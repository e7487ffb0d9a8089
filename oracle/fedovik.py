"""TEST INFRASTRUCTURE ONLY: a plain, slow restatement of the Fedovik design, one function per mechanism, on the CPU and (by
default) in float64.  Nothing here is shared with the product path: no caches, no packed projections; attention is a full score
matrix, recurrences walk token by token.

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
    are the values marked stored(): what rounding alone does to the result of a 16-bit run."""
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


def softplus(x):
    return torch.clamp(x, min=0) + torch.log1p(torch.exp(-x.abs()))


def silu(x):
    return x * sigmoid(x)


def layer_norm(x, w, b, eps):
    d = x - x.mean(dim=-1, keepdim=True)
    return d / torch.sqrt((d * d).mean(dim=-1, keepdim=True) + eps) * w + b


def over_rms(x, eps):
    return x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps)


# ---------------------------------------------------------------------------------------------------- attention
def rotate_neighbours(x, positions, base, dims):
    """x [T, heads, D]: the pairs (2i, 2i + 1) of the first `dims` elements turn by position * base^(-2i/dims)."""
    f = torch.tensor([float(base) ** (-2.0 * i / dims) for i in range(dims // 2)], dtype=torch.float64)
    a = (positions.to(torch.float64)[:, None] * f)[:, None, :]
    c, s = a.cos().to(x.dtype), a.sin().to(x.dtype)
    out = x.clone()
    u, v = x[..., 0:dims:2], x[..., 1:dims:2]
    out[..., 0:dims:2], out[..., 1:dims:2] = u * c - v * s, v * c + u * s
    return out


def scores(q, k, scale):
    """[H, T, T] of q [T, H, D] and k [T, G, D]; head h reads group h / (H/G)."""
    k = k.repeat_interleave(q.shape[1] // k.shape[1], dim=1)
    return torch.einsum("ihd,jhd->hij", q, k) * scale


def weighted(p, v):
    """[T, H, V] of weights [H, T, T] and v [T, G, V]"""
    return torch.einsum("hij,jhd->ihd", p, v.repeat_interleave(p.shape[0] // v.shape[1], dim=1))


def distances(n):
    return torch.arange(n)[:, None] - torch.arange(n)[None, :]


def sigmoid_weights(s, bias):
    """Every key on its own: sigmoid(score + a number per head), zero for keys behind the query."""
    return sigmoid(s + bias[:, None, None]) * (distances(s.shape[1]) >= 0)


def log_distance_weights(s, r1, r2, window):
    """Softmax over the last `window` tokens of score - r1 ln(1 + r2 distance)."""
    d = distances(s.shape[1])
    bias = r1[:, None, None] * torch.log(1 + r2[:, None, None] * d.clamp(min=0).to(s.dtype))
    s = (s - bias).masked_fill((d < 0) | (d >= window), -math.inf)
    p = torch.exp(s - s.max(dim=-1, keepdim=True).values)
    return p / p.sum(dim=-1, keepdim=True)


def biased_product(h, w, name):
    return stored(product(h, w[name]) + w[name + ".b"])


def sigmoid_attention(h, w, m, eps):
    H, G, D, V, T = m["heads"], m["kv_heads"], m["dim"], m["vdim"], h.shape[0]
    q, k, v = biased_product(h, w, "q").view(T, H, D), biased_product(h, w, "k").view(T, G, D), biased_product(h, w, "v").view(T, G, V)
    q, k = (stored(rotate_neighbours(x, torch.arange(T), m["rot"]["base"], m["rot"]["dims"])) for x in (q, k))
    o = weighted(sigmoid_weights(scores(q, k, m["scale"]), w["pb"]), v).reshape(T, H * V)
    return biased_product(o * sigmoid(product(h, w["g"])), w, "o")


def log_distance_attention(h, w, m, eps):
    H, G, D, V, T = m["heads"], m["kv_heads"], m["dim"], m["vdim"], h.shape[0]
    q, k, v = biased_product(h, w, "q").view(T, H, D), biased_product(h, w, "k").view(T, G, D), biased_product(h, w, "v").view(T, G, V)
    q, k = stored(over_rms(q, eps) * w["q.norm"]), stored(over_rms(k, eps) * w["k.norm"])
    o = weighted(log_distance_weights(scores(q, k, m["scale"]), w["r1"], w["r2"], m["mask"]["size"]), v)
    return o.reshape(T, H * V)


# ---------------------------------------------------------------------------------------------------- gated delta rule
def short_convolution(x, w):
    """silu of a causal convolution per channel; w [channels, taps], the last tap for the current token."""
    taps = w.shape[1]
    padded = torch.cat((torch.zeros((taps - 1, x.shape[1]), dtype=x.dtype), x))
    return silu(sum(padded[i:i + x.shape[0]] * w[:, i] for i in range(taps)))


def unit(x):
    return x / torch.sqrt((x * x).sum(dim=-1, keepdim=True) + 1e-6)


def channel_decays(z, a_log, dt_bias, heads):
    """exp(-exp(A_log) softplus(z + dt_bias)), [T, heads, dim]"""
    return torch.exp(-torch.exp(a_log)[None, :, None] * softplus(z + dt_bias).view(z.shape[0], heads, -1))


def delta_rule(q, k, v, g, beta, S=None):
    """q, k [T, G, D], v [T, H, V], g [T, H, D], beta [T, H]: S <- g S; S <- S + k (beta (v - S^T k))^T; o = S^T q.  Returns (o [T, H, V],
    the last S [H, D, V])."""
    T, H, V = v.shape
    q, k = (x.repeat_interleave(H // x.shape[1], dim=1) for x in (q, k))
    S = torch.zeros((H, k.shape[2], V), dtype=v.dtype) if S is None else S
    out = []
    for t in range(T):
        S = g[t][:, :, None] * S
        u = beta[t][:, None] * (v[t] - torch.einsum("hdv,hd->hv", S, k[t]))
        S = S + k[t][:, :, None] * u[:, None, :]
        out.append(torch.einsum("hdv,hd->hv", S, q[t]))
    return torch.stack(out), S


def gated_delta(h, w, m, eps):
    H, G, D, V, T = m["heads"], m["kv_heads"], m["dim"], m["vdim"], h.shape[0]
    q, k, v = (stored(short_convolution(product(h, w[n]), w[n + ".conv"])) for n in "qkv")
    q, k = unit(q.view(T, G, D)) * D ** -0.5, unit(k.view(T, G, D))
    beta = sigmoid(product(h, w["b"]))
    g = channel_decays(product(product(h, w["a1"]), w["a2"]), w["A_log"], w["dt_bias"], H)
    o = stored(delta_rule(q, k, v.view(T, H, V), g, beta)[0])
    o = over_rms(o, eps) * w["norm"] * sigmoid(product(product(h, w["g1"]), w["g2"])).view(T, H, V)
    return o.reshape(T, H * V)


def parallel(h, w, m, eps):
    wl, wr = _under(w, "left."), _under(w, "right.")
    left = product(log_distance_attention(h, wl, m["left"], eps), wl["o"])
    right = product(gated_delta(h, wr, m["right"], eps), wr["o"])
    return m["left_scale"] * left + m["right_scale"] * right


# ---------------------------------------------------------------------------------------------------- matrix memory
def capped(x, cap):
    return cap * torch.tanh(x / cap)


def matrix_memory(q, k, v, i, f, state=None):
    """q, k [T, H, D], v [T, H, V], logarithms of the gates i, f [T, H]; everything relative to a running maximum m that starts at 0.
    Returns (o [T, H, V], the last (S [H, D, V], n [H, D], m [H]))."""
    T, H, V = v.shape
    if state is None:
        state = (torch.zeros((H, q.shape[2], V), dtype=v.dtype), torch.zeros((H, q.shape[2]), dtype=v.dtype), torch.zeros(H, dtype=v.dtype))
    S, n, m = state
    out = []
    for t in range(T):
        m_new = torch.maximum(f[t] + m, i[t])
        keep, take = torch.exp(f[t] + m - m_new), torch.exp(i[t] - m_new)
        m = m_new
        S = keep[:, None, None] * S + take[:, None, None] * k[t][:, :, None] * v[t][:, None, :]
        n = keep[:, None] * n + take[:, None] * k[t]
        den = torch.maximum((n * q[t]).sum(-1).abs(), torch.exp(-m)) + 1e-6
        out.append(torch.einsum("hdv,hd->hv", S, q[t]) / den[:, None])
    return torch.stack(out), (S, n, m)


def log_gates(i, f, cap):
    """(input gate, forget gate), both logarithms, from their projections."""
    return capped(i, cap), -softplus(-capped(f, cap))


def mlstm(h, w, m, eps):
    H, D, V, T = m["heads"], m["dim"], m["vdim"], h.shape[0]
    q, k, v = product(h, w["q"]).view(T, H, D) * D ** -0.5, product(h, w["k"]).view(T, H, D), product(h, w["v"]).view(T, H, V)
    i, f = log_gates(product(h, w["i"]) + w["i.b"], product(h, w["f"]) + w["f.b"], m["gate_cap"])
    o = over_rms(stored(matrix_memory(q, k, v, i, f)[0]), eps).reshape(T, H * V)
    return product(o * w["norm"] * sigmoid(product(h, w["g"])), w["o"])


MIXERS = {"attention": sigmoid_attention, "parallel": parallel, "mlstm": mlstm}


# ---------------------------------------------------------------------------------------------------- the model
def dense(h, w):
    return product(torch.clamp(product(h, w["gate"]), min=0) * product(h, w["up"]), w["down"])


def _under(weights, prefix, dtype=None):
    return {k[len(prefix):]: (v if dtype is None else v.to(dtype)) for k, v in weights.items() if k.startswith(prefix)}


def passes(config):
    """(layer number, None or the number of the pass that begins in front of it) in the order in which layers run."""
    loop = config.get("loop")
    n = len(config["layers"])
    if loop is None:
        return [(i, None) for i in range(n)]
    order = [(i, None) for i in range(loop["start"])]
    for t in range(loop["times"]):
        order += [(i, t if i == loop["start"] else None) for i in range(loop["start"], loop["stop"])]
    return order + [(i, None) for i in range(loop["stop"], n)]


def forward(config, weights, tokens, dtype=torch.float64, layers_out=None):
    """Logits [T, vocab] of one sequence.  layers_out: a list that receives the residual stream after every layer run."""
    eps = config["norm"]["eps"]
    table = weights["embed"].to(dtype)
    x = x0 = table[torch.as_tensor(tokens)] * config["embedding"]["scale"]
    norm = lambda x, n: layer_norm(x, weights[n].to(dtype), weights[n + ".b"].to(dtype), eps)      # noqa: E731
    for i, begins in passes(config):
        if begins is not None:
            x = product(torch.cat((x, x0), dim=-1), weights["loop.in"].to(dtype)) + weights["loop.step"].to(dtype)[begins]
        layer = config["layers"][i]
        h = norm(x, f"l{i}.norm1")
        y = MIXERS[layer["type"]](h, _under(weights, f"l{i}.mix.", dtype), layer["mixer"], eps)
        if layer.get("mlp") is not None:
            y = y + dense(h, _under(weights, f"l{i}.mlp.", dtype))
        x = x + y
        if layers_out is not None:
            layers_out.append(x.clone())
    return product(norm(x, "final.norm"), table)


def greedy(config, weights, prompt, n, dtype=torch.float64):
    """n greedily chosen tokens after the prompt, recomputing the whole sequence for each."""
    seq = list(prompt)
    for _ in range(n):
        seq.append(int(forward(config, weights, seq, dtype)[-1].argmax()))
    return seq[len(prompt):]
