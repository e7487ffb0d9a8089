"""Small Nepulix configurations and random weights for the tests."""
import torch


def retention(heads, dim, vdim, rot, base=10000.0, decay=None):
    if decay is None:
        decay = [1 - 2.0 ** (-2 - 1.3 * i) for i in range(heads)]
    return {"type": "retention", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "decay": decay, "rot": {"base": base, "dims": rot}}}


def mamba2(heads, vdim, state, groups, conv, norm_groups):
    return {"type": "mamba2", "mixer": {"heads": heads, "vdim": vdim, "state": state, "groups": groups, "conv": conv, "norm_groups": norm_groups}}


def latent(heads, dim, rot_dim, vdim, q_rank, kv_rank, scale=None, base=5000.0):
    return {"type": "latent_attention", "mixer": {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "q_rank": q_rank, "kv_rank": kv_rank,
                                                  "scale": scale or (dim + rot_dim) ** -0.5, "rot": {"base": base, "dims": rot_dim}}}


def config(width, vocab, layers, ff=None, limit=2.0, eps=1e-5):
    out = []
    for i, layer in enumerate(layers):
        layer = dict(layer)
        # every third layer goes without a feed-forward
        layer["mlp"] = None if ff is None or i % 3 == 2 else {"kind": "dense", "ff": ff + 8 * i, "limit": limit / (1 + i)}
        out.append(layer)
    return {"architecture": "Nepulix", "width": width, "vocab": vocab, "norm": {"eps": eps}, "layers": out}


CONFIGS = {
    # sizes that are no multiples of eight, a partial rotation whose half is odd, more norm groups than heads
    "odd": config(72, 101, [mamba2(6, 20, 26, 3, 4, 8), retention(3, 42, 25, 22), latent(5, 22, 6, 37, 51, 44), mamba2(4, 24, 12, 2, 2, 3)], ff=90),
    # head sizes of large models
    "large": config(256, 264, [retention(2, 128, 128, 128, 1e6), mamba2(8, 64, 128, 1, 4, 1), latent(18, 128, 64, 128, 192, 512)], ff=384, limit=7.0),
    # everything that can be one is one
    "ones": config(64, 96, [latent(1, 16, 8, 16, 16, 32), mamba2(1, 32, 16, 1, 1, 1), retention(1, 16, 32, 8)], ff=64, eps=1e-3),
    # heads of 256, values wider than keys, all decays different, latent first and last
    "wide": config(128, 200, [latent(3, 40, 24, 144, 72, 96, scale=0.21), retention(2, 200, 160, 96, 2e4, [0.9, 1.0]),
                              mamba2(6, 48, 72, 3, 5, 2), latent(2, 64, 16, 64, 64, 200)]),
}


def tensor_shapes(cfg):
    w = cfg["width"]
    shapes = {"embed": (cfg["vocab"], w), "final.norm": (w,)}
    for i, layer in enumerate(cfg["layers"]):
        m, p = layer["mixer"], f"l{i}."
        shapes[p + "norm1"] = (w,)
        if layer["type"] == "retention":
            h, d, v = m["heads"], m["dim"], m["vdim"]
            t = {"q": (h * d, w), "k": (h * d, w), "v": (h * v, w), "g": (h * v, w), "o": (w, h * v)}
        elif layer["type"] == "mamba2":
            h, inner, gn = m["heads"], m["heads"] * m["vdim"], m["groups"] * m["state"]
            ch = inner + 2 * gn
            t = {"in": (inner + ch + h, w), "conv": (ch, m["conv"]), "conv.b": (ch,), "dt_bias": (h,), "A_log": (h,), "D": (h,), "norm": (inner,), "o": (w, inner)}
        else:
            h, d, r, v, qr, kr = (m[k] for k in ("heads", "dim", "rot_dim", "vdim", "q_rank", "kv_rank"))
            t = {"dq": (qr, w), "dq.norm": (qr,), "uq": (h * (d + r), qr), "dkv": (kr + r, w), "dkv.norm": (kr,), "uk": (h * d, kr), "uv": (h * v, kr), "o": (w, h * v)}
        shapes.update({p + "mix." + k: s for k, s in t.items()})
        if layer["mlp"] is not None:
            ff = layer["mlp"]["ff"]
            shapes.update({p + "norm2": (w,), p + "mlp.gate": (ff, w), p + "mlp.up": (ff, w), p + "mlp.down": (w, ff)})
    return shapes


def random_weights(cfg, seed=0):
    """bfloat16 weights under the checkpoint's names; queries are scaled up so that attention is far from uniform."""
    g = torch.Generator().manual_seed(seed)
    out = {}
    for name, shape in tensor_shapes(cfg).items():
        t = torch.randn(shape, generator=g)
        leaf = name.split(".", 1)[1] if name[0] == "l" else name
        if name == "embed":
            t = t * 1.0
        elif leaf in ("norm1", "norm2") or name == "final.norm":
            t = t * 0.2
        elif leaf in ("mix.dq.norm", "mix.dkv.norm", "mix.norm", "mix.D"):
            t = 1 + 0.3 * t
        elif leaf == "mix.A_log":
            t = t * 0.7
        elif leaf in ("mix.dt_bias", "mix.conv.b"):
            t = t * 0.5 - (2.0 if leaf == "mix.dt_bias" else 0.0)
        elif leaf == "mix.conv":
            t = t * shape[1] ** -0.5
        elif len(shape) == 2:
            t = t * shape[1] ** -0.5 * (2.5 if leaf == "mix.uq" else 1.0)
        out[name] = t.to(torch.bfloat16)
    return out


def random_tokens(cfg, n, seed):
    return torch.randint(0, cfg["vocab"], (n,), generator=torch.Generator().manual_seed(seed)).tolist()


def logit_error(got, want):
    """Per position: root mean square of the difference (mean taken off), over the root mean square of all wanted logits."""
    d = got.double().cpu() - want.double()
    d = d - d.mean(dim=-1, keepdim=True)
    w = want.double() - want.double().mean(dim=-1, keepdim=True)
    return d.pow(2).mean(dim=-1).sqrt() / w.pow(2).mean().sqrt()


def write_checkpoint(folder, cfg, weights):
    import json
    from safetensors.torch import save_file
    folder.mkdir(parents=True, exist_ok=True)
    (folder / "config.json").write_text(json.dumps(cfg))
    save_file({k: v.contiguous() for k, v in weights.items()}, str(folder / "model.safetensors"))
