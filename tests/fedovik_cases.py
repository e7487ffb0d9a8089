"""Small Fedovik configurations and random weights for the tests."""
import torch


def memory(heads, dim, vdim, cap=15.0):
    return {"type": "mlstm", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "gate_cap": cap}}


def attention(heads, kv_heads, dim, vdim, rot, scale, base=1e4):
    return {"type": "attention", "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale, "rot": {"base": base, "dims": rot}}}


def parallel(left, right, left_scale, right_scale):
    """left: (heads, kv_heads, dim, vdim, window, scale), right: (heads, kv_heads, dim, vdim, taps)"""
    names = ("heads", "kv_heads", "dim", "vdim")
    return {"type": "parallel", "mixer": {"left": {**dict(zip(names, left)), "mask": {"size": left[4]}, "scale": left[5]},
                                          "right": {**dict(zip(names, right)), "conv": right[4]}, "left_scale": left_scale, "right_scale": right_scale}}


def config(width, vocab, layers, loop=None, embedding_scale=1.5, eps=1e-5):
    """layers: (mixer, size of the feed-forward or None); loop: (start, stop, times)"""
    out = [{**mixer, "mlp": None if ff is None else {"kind": "dense", "ff": ff}} for mixer, ff in layers]
    cfg = {"architecture": "Fedovik", "width": width, "vocab": vocab, "norm": {"eps": eps}, "embedding": {"scale": embedding_scale}, "layers": out}
    if loop is not None:
        cfg["loop"] = dict(zip(("start", "stop", "times"), loop))
    return cfg


CONFIGS = {
    # sizes that are no multiples of eight, a loop in the middle with three passes, a layer without a feed-forward, three taps
    "odd": config(76, 101, [(attention(6, 3, 22, 13, 14, 0.3), 50), (memory(3, 20, 26, 7.0), None),
                            (parallel((4, 2, 18, 21, 25, 0.4), (6, 2, 12, 15, 3), 0.7, 1.2), 36), (memory(2, 9, 5, 30.0), 41)], (1, 3, 3)),
    # head sizes of large models, a loop over everything
    "large": config(192, 264, [(parallel((24, 1, 128, 128, 64, 0.1), (4, 2, 128, 128, 4), 1.3, 0.6), 384), (memory(2, 128, 128), 512),
                               (attention(16, 8, 128, 128, 128, 0.09, 5e5), 256)], (0, 3, 2), embedding_scale=3.0),
    # nearly everything that can be one is one: a token that sees itself only, a convolution of the current token, one pass
    "ones": config(64, 96, [(memory(1, 16, 8, 2.0), 24), (parallel((1, 1, 16, 8, 1, 1.0), (1, 1, 8, 8, 1), 1.0, 1.0), 16), (attention(1, 1, 8, 1, 2, 1.0), 8)], (1, 2, 1),
                   embedding_scale=1.0, eps=1e-3),
    # sizes beyond those of the matrix-core kernels, groups of many heads, windows wider than a prompt, a loop that ends with the last
    # layer, values of one element in the delta rule
    "wide": config(128, 88, [(memory(1, 260, 300, 15.0), 96), (parallel((18, 1, 40, 280, 4000, 0.2), (2, 1, 264, 24, 5), 0.5, 0.8), 64),
                             (parallel((3, 3, 72, 16, 33, 0.2), (5, 1, 16, 1, 2), 1.1, -0.9), None), (attention(2, 1, 160, 48, 80, 0.1, 3e3), 40)], (2, 4, 2)),
    # no loop
    "plain": config(96, 72, [(attention(4, 4, 64, 40, 48, 0.15), 64), (parallel((2, 2, 32, 64, 70, 0.25), (3, 3, 64, 72, 4), 0.9, 1.0), 48), (memory(4, 64, 64), 64)]),
}


def tensor_shapes(cfg):
    w, shapes = cfg["width"], {}
    shapes["embed"] = (cfg["vocab"], w)
    loop = cfg.get("loop")
    if loop is not None:
        shapes.update({"loop.in": (w, 2 * w), "loop.step": (loop["times"], w)})

    def attention_shapes(m):
        h, g, d, v = (m[k] for k in ("heads", "kv_heads", "dim", "vdim"))
        t = {"q": (h * d, w), "k": (g * d, w), "v": (g * v, w), "q.b": (h * d,), "k.b": (g * d,), "v.b": (g * v,), "o": (w, h * v)}
        t.update({"q.norm": (d,), "k.norm": (d,), "r1": (h,), "r2": (h,)} if "mask" in m else {"pb": (h,), "g": (h * v, w), "o.b": (w,)})
        return t

    for i, layer in enumerate(cfg["layers"]):
        m, p = layer["mixer"], f"l{i}."
        shapes.update({p + "norm1": (w,), p + "norm1.b": (w,)})
        if layer["type"] == "attention":
            t = attention_shapes(m)
        elif layer["type"] == "mlstm":
            h, d, v = m["heads"], m["dim"], m["vdim"]
            t = {"q": (h * d, w), "k": (h * d, w), "v": (h * v, w), "g": (h * v, w), "o": (w, h * v), "norm": (h * v,)}
            t.update({n: (h, w) for n in "if"})
            t.update({n + ".b": (h,) for n in "if"})
        else:
            r = m["right"]
            h, g, d, v = (r[k] for k in ("heads", "kv_heads", "dim", "vdim"))
            low_a, low_g = 9 + i, 16      # sizes that only the tensors tell
            rows = {"q": g * d, "k": g * d, "v": h * v}
            right = {"b": (h, w), "A_log": (h,), "norm": (v,), "a1": (low_a, w), "a2": (h * d, low_a), "dt_bias": (h * d,), "g1": (low_g, w), "g2": (h * v, low_g),
                     "o": (w, h * v), **{n: (k, w) for n, k in rows.items()}, **{n + ".conv": (k, r["conv"]) for n, k in rows.items()}}
            t = {**{"left." + n: s for n, s in attention_shapes(m["left"]).items()}, **{"right." + n: s for n, s in right.items()}}
        shapes.update({p + "mix." + n: s for n, s in t.items()})
        if layer["mlp"] is not None:
            ff = layer["mlp"]["ff"]
            shapes.update({p + "mlp.gate": (ff, w), p + "mlp.up": (ff, w), p + "mlp.down": (w, ff)})
    shapes.update({"final.norm": (w,), "final.norm.b": (w,)})
    return shapes


def random_weights(cfg, seed=0):
    """bfloat16 weights under the checkpoint's names.  Queries are scaled up, so that scores matter; decays and gates are spread from
    short to long memory; biases and passes' vectors are as large as what they are added to."""
    g = torch.Generator().manual_seed(seed)
    out = {}
    for n, shape in tensor_shapes(cfg).items():
        t = torch.randn(shape, generator=g)
        leaf = n.split(".", 1)[1] if n[0] == "l" and n[1].isdigit() else n
        name = leaf.rsplit("mix.", 1)[-1].replace("left.", "").replace("right.", "")
        if n == "embed":
            t = t + 0.2
        elif n == "loop.in":
            t = t * (2 * cfg["width"]) ** -0.5 * 1.2
        elif n == "loop.step":
            pass
        elif name == "pb":
            t = t - 4
        elif name == "r1":      # far tokens of a window keep some weight
            t = 0.3 * t.abs() + 0.05
        elif name == "r2":
            t = t.abs() + 0.1
        elif name == "i.b":
            t = 2 * t
        elif name == "f.b":
            t = 2 * t + 4
        elif name == "dt_bias":
            t = 2 * t - 4
        elif name == "A_log":
            t = 0.7 * t
        elif name in ("norm", "q.norm", "k.norm") or leaf in ("norm1", "final.norm"):
            t = 1 + 0.3 * t
            if name == "q.norm":
                t = 2 * t
        elif len(shape) == 1:
            t = 0.5 * t
        elif name.endswith(".conv"):
            t = t * shape[1] ** -0.5
        else:
            t = t * shape[1] ** -0.5
            if name in ("q", "i", "f", "b", "g", "g2") or leaf == "mix.left.o":
                t = 2 * t
        out[n] = t.to(torch.bfloat16)
    return out


def random_tokens(cfg, n, seed):
    return torch.randint(0, cfg["vocab"], (n,), generator=torch.Generator().manual_seed(seed)).tolist()
