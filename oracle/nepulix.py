"""TEST INFRASTRUCTURE ONLY: a plain, slow restatement of the Nepulix design, one function per mechanism, on the CPU
and (by default) in float64.  Nothing here is shared with the product path: no caches, no chunks, no absorbed products;
recurrences run token by token and attention is a full score matrix.

Weights come as a dict of tensors under the checkpoint's names, the configuration as the dict of config.json.
"""
from __future__ import annotations

import math

import torch


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
    q = (h @ w["q"].T).view(T, H, D)
    k = (h @ w["k"].T).view(T, H, D)
    v = (h @ w["v"].T).view(T, H, V)
    q = rotate_half(q, positions, m["rot"]["base"], m["rot"]["dims"])
    k = rotate_half(k, positions, m["rot"]["base"], m["rot"]["dims"]) * D ** -0.5
    decay = torch.tensor(m["decay"], dtype=h.dtype)[None, :].expand(T, H)
    o, S = decayed_recurrence(q, k, v, decay, state)
    o = rms(o, eps).reshape(T, H * V)
    return (o * silu(h @ w["g"].T)) @ w["o"].T, S


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
    p = h @ w["in"].T
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
    return y @ w["o"].T, S


def latent_attention(h, w, m, eps, positions, state=None):
    H, D, R, V, K = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    T = h.shape[0]
    cq = rms(h @ w["dq"].T, eps) * w["dq.norm"]
    q = (cq @ w["uq"].T).view(T, H, D + R)
    down = h @ w["dkv"].T
    c = rms(down[:, :K], eps) * w["dkv.norm"]
    kr = rotate_interleaved(down[:, None, K:], positions, m["rot"]["base"], m["rot"]["dims"])[:, 0]
    qr = rotate_interleaved(q[..., D:], positions, m["rot"]["base"], m["rot"]["dims"])
    ku = (c @ w["uk"].T).view(T, H, D)
    v = (c @ w["uv"].T).view(T, H, V)
    s = (torch.einsum("ihd,jhd->hij", q[..., :D], ku) + torch.einsum("ihd,jd->hij", qr, kr)) * m["scale"]
    s = s.masked_fill(~torch.ones((T, T), dtype=torch.bool).tril(), -math.inf)
    p = torch.exp(s - s.max(dim=-1, keepdim=True).values)
    p = p / p.sum(dim=-1, keepdim=True)
    return torch.einsum("hij,jhd->ihd", p, v).reshape(T, H * V) @ w["o"].T, None


def dense_ff(h, w, m):
    g = torch.clamp(h @ w["gate"].T, max=m["limit"])
    u = torch.clamp(h @ w["up"].T, min=-m["limit"], max=m["limit"])
    return (g / (1 + torch.exp(-1.702 * g)) * (u + 1)) @ w["down"].T


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
    return x @ weights["embed"].to(dtype).T


def greedy(config, weights, prompt, n, dtype=torch.float64):
    """n greedily chosen tokens after the prompt, recomputing the whole sequence for each."""
    seq = list(prompt)
    for _ in range(n):
        seq.append(int(forward(config, weights, seq, dtype)[-1].argmax()))
    return seq[len(prompt):]
