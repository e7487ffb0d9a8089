"""TEST INFRASTRUCTURE ONLY: a plain, slow restatement of the Nepulix design, one function per mechanism, on the CPU
and (by default) in float64.  Nothing here is shared with the product path: no caches, no chunks, no absorbed products;
recurrences run token by token and attention is a full score matrix.

Weights come as a dict of tensors under the checkpoint's names, the configuration as the dict of config.json.
"""
from __future__ import annotations

import contextlib
import math

import torch

_round = None      # see sixteen_bit_products


@contextlib.contextmanager
def sixteen_bit_products(seed=0):
    """Inside, every matrix product takes and gives values rounded to bfloat16 (to nearest for seed 0, else stochastically):
    what rounding alone does to the result of a 16-bit run."""
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


def rms(x, eps):
    """x over the root of its mean square, eps inside the root."""
    return x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps)


def norm_unit_offset(x, w, eps):
    """RMS norm whose weight is stored around zero."""
    return rms(x, eps) * (1 + w)


def silu(x):
    return x / (1 + torch.exp(-x))


def softplus(x):
    return torch.where(x > 30, x, torch.log1p(torch.exp(torch.clamp(x, max=30.0))))


def angles(positions, base, dims, dtype=torch.float64):
    """[T, dims/2] rotation angles p * base^(-2i/dims)."""
    i = torch.arange(dims // 2, dtype=torch.float64)
    f = torch.pow(torch.tensor(float(base), dtype=torch.float64), -2.0 * i / dims)
    return (positions.to(torch.float64)[:, None] * f[None, :]).to(dtype)


def rotate_half(x, positions, base, dims):
    """x [T, H, D]: dimension i < dims/2 is paired with i + dims/2; dimensions from `dims` on pass unchanged."""
    a = angles(positions, base, dims, x.dtype)[:, None, :]
    u, v, rest = x[..., : dims // 2], x[..., dims // 2: dims], x[..., dims:]
    return torch.cat((u * a.cos() - v * a.sin(), v * a.cos() + u * a.sin(), rest), dim=-1)


def rotate_interleaved(x, positions, base, dims):
    """x [T, H, D]: dimension 2i is paired with 2i + 1; dimensions from `dims` on pass unchanged."""
    a = angles(positions, base, dims, x.dtype)[:, None, :]
    u, v = x[..., 0:dims:2], x[..., 1:dims:2]
    out = x.clone()
    out[..., 0:dims:2] = u * a.cos() - v * a.sin()
    out[..., 1:dims:2] = v * a.cos() + u * a.sin()
    return out


def decayed_recurrence(q, k, v, decay, state=None):
    """S_t = decay_t S_(t-1) + k_t v_t^T, o_t = S_t^T q_t.  q, k [T, H, D], v [T, H, V], decay [T, H];
    returns (o [T, H, V], final S [H, D, V])."""
    T, H, D = q.shape
    S = torch.zeros((H, D, v.shape[-1]), dtype=q.dtype) if state is None else state.clone()
    out = []
    for t in range(T):
        S = decay[t][:, None, None] * S + k[t][:, :, None] * v[t][:, None, :]
        out.append((S * q[t][:, :, None]).sum(dim=1))
    return torch.stack(out), S


def retention(h, w, m, eps, positions, state=None):
    """Returns (output [T, width], final state).  w: the mixer's tensors by their short names."""
    H, D, V = m["heads"], m["dim"], m["vdim"]
    T = h.shape[0]
    q = product(h, w["q"]).view(T, H, D)
    k = product(h, w["k"]).view(T, H, D)
    v = product(h, w["v"]).view(T, H, V)
    q = rotate_half(q, positions, m["rot"]["base"], m["rot"]["dims"])
    k = rotate_half(k, positions, m["rot"]["base"], m["rot"]["dims"]) * D ** -0.5
    decay = torch.tensor(m["decay"], dtype=h.dtype)[None, :].expand(T, H)
    o, S = decayed_recurrence(q, k, v, decay, state)
    o = rms(o, eps).reshape(T, H * V)
    return product(o * silu(product(h, w["g"])), w["o"]), S


def causal_conv(x, kernel, bias, before=None):
    """x [T, C], kernel [C, taps] (last column: the current row); `before` [taps-1, C] replaces the zeros before x."""
    taps = kernel.shape[1]
    pad = torch.zeros((taps - 1, x.shape[1]), dtype=x.dtype) if before is None else before
    full = torch.cat((pad, x), dim=0)
    out = bias[None, :].expand(x.shape[0], -1).clone()
    for j in range(taps):
        out = out + full[j: j + x.shape[0]] * kernel[:, j]
    return out


def group_rms(y, groups, eps):
    return rms(y.reshape(y.shape[0], groups, -1), eps).reshape(y.shape)


def mamba2(h, w, m, eps, positions, state=None):
    H, V, N, G = m["heads"], m["vdim"], m["state"], m["groups"]
    inner = H * V
    T = h.shape[0]
    p = product(h, w["in"])
    z, xbc, dt = p[:, :inner], p[:, inner: 2 * inner + 2 * G * N], p[:, 2 * inner + 2 * G * N:]
    xbc = silu(causal_conv(xbc, w["conv"], w["conv.b"]))
    x = xbc[:, :inner].reshape(T, H, V)
    B = xbc[:, inner: inner + G * N].reshape(T, G, N).repeat_interleave(H // G, dim=1)
    C = xbc[:, inner + G * N:].reshape(T, G, N).repeat_interleave(H // G, dim=1)
    dt = softplus(dt + w["dt_bias"])
    decay = torch.exp(-torch.exp(w["A_log"]) * dt)
    y, S = decayed_recurrence(C, B, x * dt[:, :, None], decay, state)
    y = (y + w["D"][None, :, None] * x).reshape(T, inner)
    y = group_rms(y * silu(z), m["norm_groups"], eps) * w["norm"]
    return product(y, w["o"]), S


def latent_attention(h, w, m, eps, positions, state=None):
    H, D, R, V, K = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    T = h.shape[0]
    cq = rms(product(h, w["dq"]), eps) * w["dq.norm"]
    q = product(cq, w["uq"]).view(T, H, D + R)
    down = product(h, w["dkv"])
    c = rms(down[:, :K], eps) * w["dkv.norm"]
    kr = rotate_interleaved(down[:, None, K:], positions, m["rot"]["base"], m["rot"]["dims"])[:, 0]
    qr = rotate_interleaved(q[..., D:], positions, m["rot"]["base"], m["rot"]["dims"])
    ku = product(c, w["uk"]).view(T, H, D)
    v = product(c, w["uv"]).view(T, H, V)
    s = (torch.einsum("ihd,jhd->hij", q[..., :D], ku) + torch.einsum("ihd,jd->hij", qr, kr)) * m["scale"]
    s = s.masked_fill(~torch.ones((T, T), dtype=torch.bool).tril(), -math.inf)
    p = torch.exp(s - s.max(dim=-1, keepdim=True).values)
    p = p / p.sum(dim=-1, keepdim=True)
    return product(torch.einsum("hij,jhd->ihd", p, v).reshape(T, H * V), w["o"]), None


def dense_ff(h, w, m):
    g = torch.clamp(product(h, w["gate"]), max=m["limit"])
    u = torch.clamp(product(h, w["up"]), min=-m["limit"], max=m["limit"])
    return product(g / (1 + torch.exp(-1.702 * g)) * (u + 1), w["down"])


MIXERS = {"retention": retention, "mamba2": mamba2, "latent_attention": latent_attention}


def _under(weights, prefix, dtype):
    return {k[len(prefix):]: v.to(dtype) for k, v in weights.items() if k.startswith(prefix)}


def forward(config, weights, tokens, dtype=torch.float64, layers_out=None):
    """Logits [T, vocab] of one sequence.  layers_out: a list that receives the residual stream after every layer."""
    eps = config["norm"]["eps"]
    tokens = torch.as_tensor(tokens, dtype=torch.int64)
    positions = torch.arange(tokens.numel())
    x = weights["embed"].to(dtype)[tokens]
    for i, layer in enumerate(config["layers"]):
        pre = f"l{i}."
        mix = MIXERS[layer["type"]](x, _under(weights, pre + "mix.", dtype), layer["mixer"], eps, positions)[0]
        x = x + norm_unit_offset(mix, weights[pre + "norm1"].to(dtype), eps)
        if layer.get("mlp") is not None:
            ff = dense_ff(x, _under(weights, pre + "mlp.", dtype), layer["mlp"])
            x = x + norm_unit_offset(ff, weights[pre + "norm2"].to(dtype), eps)
        if layers_out is not None:
            layers_out.append(x.clone())
    x = norm_unit_offset(x, weights["final.norm"].to(dtype), eps)
    return product(x, weights["embed"].to(dtype))


def greedy(config, weights, prompt, n, dtype=torch.float64):
    """n greedily chosen tokens after the prompt, recomputing the whole sequence for each."""
    seq = list(prompt)
    for _ in range(n):
        seq.append(int(forward(config, weights, seq, dtype)[-1].argmax()))
    return seq[len(prompt):]
