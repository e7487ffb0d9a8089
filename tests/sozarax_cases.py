"""Small Sozarax configurations and random weights for the tests."""
import torch


def wkv(heads, dim, rank):
    """rank: of the decay's two-step projection; only the tensors tell it."""
    return {"type": "wkv", "mixer": {"heads": heads, "dim": dim}, "rank": rank}


def attention(heads, kv_heads, dim, vdim, coef, every, scale=None):
    return {"type": "attention", "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale or dim ** -0.5,
                                           "q_temp": {"coef": coef, "every": every}}}


def dense(ff):
    return {"kind": "dense", "ff": ff}


def moe(ff, experts, top):
    return {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top}}


def config(width, vocab, layers, mlps, loop, scale, eps=1e-5):
    out, ranks = [], []
    for layer, mlp in zip(layers, mlps):
        ranks.append(layer.get("rank"))
        out.append({"type": layer["type"], "mixer": layer["mixer"], "mlp": mlp})
    return {"architecture": "Sozarax", "width": width, "vocab": vocab, "norm": {"eps": eps}, "embedding": {"scale": scale}, "layers": out,
            "loop": {"start": loop[0], "stop": loop[1], "times": loop[2]}}, ranks


MADE = {
    # sizes that are no multiples of eight; attention inside the loop; several experts per token; a layer without feed-forward
    "odd": config(72, 101, [attention(6, 3, 20, 13, 0.3, 7), wkv(3, 22, 5), attention(5, 5, 9, 33, 0.8, 40), wkv(2, 36, 19)],
                  [dense(90), moe(28, 5, 2), None, moe(17, 6, 3)], (0, 2, 2), 3.7),
    # head sizes of large models; the last layers loop
    "large": config(256, 264, [wkv(2, 128, 64), attention(24, 1, 128, 128, 0.1, 64), wkv(4, 64, 32)],
                    [moe(136, 16, 4), dense(512), moe(64, 40, 1)], (1, 3, 2), 16.0),
    # nearly everything that can be one is one (a dense hidden size of one would make its normed result a matter of one sign)
    "ones": config(64, 96, [wkv(1, 16, 1), attention(1, 1, 16, 8, 0.5, 1), wkv(1, 32, 8)], [moe(8, 1, 1), dense(24), moe(1, 2, 1)], (1, 2, 1), 1.0, eps=1e-3),
    # only recurrent layers, all looped, heads wider than the matrix-core kernels' smaller forms, every expert chosen
    "states": config(96, 120, [wkv(1, 200, 40), wkv(5, 20, 7)], [moe(24, 3, 3), dense(100)], (0, 2, 3), 0.5),
    # only attention, values wider than keys and keys wider than values, no loop at all
    "pages": config(128, 88, [attention(4, 2, 48, 144, 0.4, 30, 0.3), attention(18, 1, 160, 24, 0.2, 11), attention(3, 3, 40, 64, 0.0, 5)],
                    [dense(64), None, moe(40, 130, 2)], (2, 2, 1), 8.0),
}
CONFIGS = {k: v[0] for k, v in MADE.items()}


def tensor_shapes(name):
    cfg, ranks = MADE[name]
    w = cfg["width"]
    shapes = {"embed": (cfg["vocab"], w), "head": (cfg["vocab"], w), "final.norm": (w,)}
    for i, layer in enumerate(cfg["layers"]):
        m, p = layer["mixer"], f"l{i}."
        if layer["type"] == "wkv":
            hd, d = m["heads"] * m["dim"], ranks[i]
            t = {"mu." + n: (w,) for n in "rkvgw"}
            t.update({n: (hd, w) for n in "rkvg"})
            t.update({"w1": (d, w), "w2": (hd, d), "w0": (hd,), "u": (m["heads"], m["dim"]), "norm": (hd,), "o": (w, hd)})
        else:
            h, g, d, v = (m[k] for k in ("heads", "kv_heads", "dim", "vdim"))
            t = {"q": (h * d, w), "k": (g * d, w), "v": (g * v, w), "q.norm": (h * d,), "k.norm": (g * d,), "o": (w, h * v)}
        shapes.update({p + "mix." + k: s for k, s in t.items()})
        shapes.update({p + n: (w,) for n in ("norm1", "norm1b")})
        mlp = layer["mlp"]
        if mlp is not None:
            shapes.update({p + n: (w,) for n in ("norm2", "norm2b")})
            if mlp["kind"] == "dense":
                shapes.update({p + "mlp.up": (mlp["ff"], w), p + "mlp.down": (w, mlp["ff"])})
            else:
                ff = mlp["expert"]["ff"]
                shapes[p + "mlp.router"] = (mlp["router"]["experts"], w)
                for e in range(mlp["router"]["experts"]):
                    shapes.update({f"{p}mlp.e{e}.gate": (ff, w), f"{p}mlp.e{e}.up": (ff, w), f"{p}mlp.e{e}.down": (w, ff)})
    return shapes


CODE = 12      # channels that only the embedding writes and only the routers read, see random_weights


def random_weights(name, seed=0):
    """bfloat16 weights under the checkpoint's names.  Query norms are scaled up, so that attention is far from uniform; decays reach
    from almost nothing lost to almost everything; r and k lean towards each other, since a state's first outputs are divided by their
    own size and r.k near zero would make that a matter of rounding.  For the same reason no choice of experts is a close call: the
    routers read channels that no sublayer writes, where each token carries a code with a clear order of the experts."""
    cfg, g = CONFIGS[name], torch.Generator().manual_seed(seed)
    out = {}
    for n, shape in tensor_shapes(name).items():
        t = torch.randn(shape, generator=g)
        leaf = n.split(".", 1)[1] if n[0] == "l" else n
        if leaf == "mix.w0":
            t = 2.0 * t - 3.0
        elif leaf.startswith("mix.mu."):
            t = 0.5 + 0.4 * t
        elif leaf == "mix.u":
            t = 1 + 0.5 * t
        elif leaf == "mix.q.norm":
            t = 2.5 * (1 + 0.3 * t)
        elif len(shape) == 1:
            t = 1 + 0.3 * t
            if leaf in ("norm1b", "norm2b"):
                t[:CODE] = 0
        elif n == "embed":
            t = t / cfg["embedding"]["scale"]
        elif leaf == "mlp.router":
            t = t * CODE ** -0.5
            t[:, CODE:] = 0
        else:
            t = t * shape[1] ** -0.5
            if leaf == "mix.k" and n.replace("mix.k", "mix.r") in tensor_shapes(name):
                t = 0.6 * t      # and 0.8 of r, below
        out[n] = t.to(torch.bfloat16)
    for n in [n for n in out if n.endswith("mix.r")]:
        k = n[:-1] + "k"
        out[k] = (out[k].float() + 0.8 * out[n].float()).to(torch.bfloat16)
    routed = [(i, layer["mlp"]["router"]) for i, layer in enumerate(cfg["layers"]) if layer["mlp"] and layer["mlp"]["kind"] == "moe"]
    open_, codes = torch.arange(cfg["vocab"]), out["embed"][:, :CODE].float()
    read = {i: (out[f"l{i}.mlp.router"][:, :CODE].float() * out[f"l{i}.norm2"][:CODE].float()).T for i, _ in routed}
    usual = {i: (codes @ r).pow(2).mean().sqrt() for i, r in read.items()}
    for _ in range(400):
        clear = torch.ones(len(open_), dtype=torch.bool)
        for i, r in routed:
            if r["top"] < r["experts"]:
                best = (codes[open_] @ read[i]).topk(r["top"] + 1, dim=-1).values
                clear &= best[:, -2] - best[:, -1] > 0.1 * usual[i]
        open_ = open_[~clear]
        if not len(open_):
            break
        codes[open_] = (torch.randn((len(open_), CODE), generator=g) / cfg["embedding"]["scale"]).to(torch.bfloat16).float()
    assert not len(open_)
    out["embed"][:, :CODE] = codes.to(torch.bfloat16)
    return out


def random_tokens(cfg, n, seed):
    return torch.randint(0, cfg["vocab"], (n,), generator=torch.Generator().manual_seed(seed)).tolist()
