"""Small Lulizen configurations, random weights and tokens for the tests."""
import torch

from oracle import lulizen as O


def chunked(heads, kv_heads, dim, vdim, rot, size, scale, softcap, base=1e4):
    return {"type": "attention", "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale, "softcap": softcap,
                                           "rot": {"base": base, "dims": rot}, "mask": {"size": size}}}


def windowed(heads, kv_heads, dim, vdim, rot, size, keep, scale, softcap, base=3e3):
    layer = chunked(heads, kv_heads, dim, vdim, rot, size, scale, softcap, base)
    layer["mixer"]["mask"]["keep_first"] = keep
    return dict(layer, type="attention_2")


def dense(ff):
    return {"kind": "dense", "ff": ff}


def moe(ff, experts, top, count, keep, shared_ff, limit=1.2, shared_limit=0.9, scale=1.7):
    return {"kind": "moe", "expert": {"ff": ff, "limit": limit}, "shared": {"ff": shared_ff, "limit": shared_limit},
            "router": {"experts": experts, "top": top, "groups": {"count": count, "keep": keep}, "scale": scale}}


def config(width, vocab, layers, bigram, eps=1e-5):
    """layers: (mixer, feed-forward or None), or the number of a layer whose tensors run again."""
    out = []
    for x in layers:
        out.append(dict(out[x], weights_of=x) if isinstance(x, int) else {**x[0], "mlp": x[1]})
    return {"architecture": "Lulizen", "width": width, "vocab": vocab, "norm": {"eps": eps}, "layers": out,
            "embedding": {"bigram": dict(zip(("buckets", "mul_prev", "mul_cur"), bigram))}}


CONFIGS = {
    # sizes that are no multiples of eight, a rotation of an odd number of pairs, groups of two and of one, a layer without a
    # feed-forward, tensors that run three times
    "odd": config(76, 101, [(windowed(6, 3, 22, 13, 14, 25, 5, 0.5, 9.0), moe(20, 6, 3, 3, 2, 36)), (chunked(4, 2, 19, 33, 6, 37, 0.3, 5.0), None),
                            (chunked(5, 5, 10, 9, 10, 50, 0.4, 12.0), moe(17, 5, 2, 5, 2, 9)), 0, 1, 0], (67, 13, 5)),
    # head sizes of large models, the second kind of attention first, one kv head and many, a cap beyond what needs no reference
    "large": config(256, 264, [(chunked(24, 1, 128, 128, 128, 64, 0.09, 100.0, 5e5), moe(136, 16, 4, 4, 2, 200, 7.0, 5.0, 2.2)),
                               (windowed(16, 8, 128, 128, 64, 128, 40, 0.08, 50.0), dense(512)),
                               (windowed(8, 2, 64, 64, 32, 33, 32, 0.12, 30.0), moe(64, 40, 6, 8, 3, 64, 2.0, 3.0, 1.0))], (1021, 7, 3)),
    # nearly everything that can be one is one: a token that sees itself only, or itself and the first
    "ones": config(64, 96, [(windowed(1, 1, 16, 8, 2, 1, 1, 1.0, 1.0), moe(8, 1, 1, 1, 1, 24, scale=1.0)), (chunked(1, 1, 32, 8, 32, 1, 0.4, 2.0), dense(24)),
                            (windowed(2, 1, 24, 16, 24, 30, 0, 0.4, 20.0), moe(8, 4, 1, 4, 1, 16))], (1, 1, 1), eps=1e-3),
    # values wider than the matrix-core kernels cover, keys wider than values, many experts in small groups, windows wider than a prompt
    "wide": config(128, 88, [(chunked(3, 3, 48, 280, 48, 1000, 0.25, 15.0), moe(24, 130, 2, 65, 60, 40)), (windowed(18, 1, 160, 24, 80, 4000, 3, 0.12, 25.0), dense(96)),
                             (chunked(2, 1, 72, 40, 40, 90, 0.2, 8.0), moe(40, 14, 6, 2, 1, 56))], (500, 11, -3)),
}


def tensor_shapes(cfg):
    w, b = cfg["width"], cfg["embedding"]["bigram"]["buckets"]
    shapes = {"embed": (cfg["vocab"], w), "bigram": (b + 1, w), "head": (cfg["vocab"], w), "final.norm": (w,)}
    for i, layer in enumerate(cfg["layers"]):
        if "weights_of" in layer:
            continue
        m, p, mlp = layer["mixer"], f"l{i}.", layer["mlp"]
        h, g, d, v = (m[k] for k in ("heads", "kv_heads", "dim", "vdim"))
        t = {"q": (h * d, w), "k": (g * d, w), "v": (g * v, w), "o": (w, h * v)}
        t.update({"q.norm": (d,), "k.norm": (d,), "sink": (h,)} if layer["type"] == "attention" else {"g": (h, w)})
        shapes.update({p + "mix." + k: s for k, s in t.items()})
        shapes.update({p + n: (w,) for n in (("norm1", "norm1b") if mlp is None else ("norm1", "norm1b", "norm2", "norm2b"))})
        if mlp is None:
            continue
        units = {"": mlp["ff"]} if mlp["kind"] == "dense" else {"shared.": mlp["shared"]["ff"], **{f"e{e}.": mlp["expert"]["ff"] for e in range(mlp["router"]["experts"])}}
        for n, ff in units.items():
            shapes.update({f"{p}mlp.{n}gate": (ff, w), f"{p}mlp.{n}up": (ff, w), f"{p}mlp.{n}down": (w, ff)})
        if mlp["kind"] == "moe":
            shapes.update({p + "mlp.router": (mlp["router"]["experts"], w), p + "mlp.correction": (mlp["router"]["experts"],)})
    return shapes


CODE = 12      # channels that only the embedding writes and only the routers read, see settled_tokens


def random_weights(cfg, seed=0):
    """bfloat16 weights under the checkpoint's names.  Queries are scaled up, so that attention is far from uniform and caps are felt;
    sinks are as large as usual sums; the mean of a row is far from zero."""
    g = torch.Generator().manual_seed(seed)
    out = {}
    for n, shape in tensor_shapes(cfg).items():
        t = torch.randn(shape, generator=g)
        leaf = n.split(".", 1)[1] if n[0] == "l" else n
        if leaf == "mix.sink":
            t = 1.5 * t + 1.0
        elif leaf == "mlp.correction":
            t = 0.3 * t
        elif leaf == "mix.q.norm":
            t = 2.5 * (1 + 0.3 * t)
        elif len(shape) == 1:
            t = 1 + 0.3 * t
            if leaf in ("norm1b", "norm2b"):
                t[:CODE] = 0
        elif n in ("embed", "bigram"):
            t = t + 0.3
        elif leaf == "mlp.router":
            t = t * 1.5 * CODE ** -0.5
            t[:, CODE:] = 0
        else:
            t = t * shape[1] ** -0.5
            if leaf == "mix.q" and n + ".norm" not in tensor_shapes(cfg):
                t = t * 2.5
        out[n] = t.to(torch.bfloat16)
    return out


def random_tokens(cfg, n, seed):
    return torch.randint(0, cfg["vocab"], (n,), generator=torch.Generator().manual_seed(seed)).tolist()


def settled_tokens(cfg, w, n, seed, gap=4e-3):
    """Random tokens for which no choice of experts is a close call that rounding may tip.  The routers read channels that no sublayer
    writes, so that a choice hangs on a token and the one in front; tokens with a close one are drawn anew."""
    g = torch.Generator().manual_seed(seed)
    s = torch.randint(0, cfg["vocab"], (n,), generator=g).tolist()
    for _ in range(200):
        with O.watching_choices() as margins:
            O.forward(cfg, w, s)
        if not margins:
            return s
        close = (torch.stack(margins).min(0).values < gap).nonzero().flatten().tolist()
        if not close:
            return s
        for i in close:
            s[i] = int(torch.randint(0, cfg["vocab"], (), generator=g))
    raise AssertionError("no tokens with clear choices found")
