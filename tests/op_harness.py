"""What the GPU tests of single operators share: fetching an operator, errors and limits, queries and pages for attention."""
import torch


def op(name):
    from nano_vllm_ninetoothed_amd import mops
    return mops.get_op(name, "hip")


def rel(got, want):
    got = got.double().cpu()
    assert torch.isfinite(got).all()
    return ((got - want).norm() / want.norm()).item()


def limit(dtype, f32=1e-6, bf16=3e-3):
    return f32 if dtype == torch.float32 else bf16


def i32(x, gpu):
    return torch.tensor(x, dtype=torch.int32, device=gpu)


def bounds(counts):
    cu = [0]
    for n in counts:
        cu.append(cu[-1] + n)
    return cu


def paged_case(gpu, dtype, H, G, d, v, lens, bs, seed, far=()):
    """Random queries, keys and values of several sequences in shuffled pages that hold garbage elsewhere.  far: positions whose key
    looks like the last query, so that it stands out of all others."""
    from nano_vllm_ninetoothed_amd.mops.hip.attention_ops import padded
    g = torch.Generator().manual_seed(seed)
    blocks = [-(-n // bs) for n in lens]
    total = sum(blocks) + 2
    perm = torch.randperm(total, generator=g).tolist()
    kp, vp = (torch.full((total, bs, G, padded(s)), float("nan"), dtype=dtype) for s in (d, v))
    table = torch.full((len(lens), max(max(blocks), 1)), -1, dtype=torch.int32)
    seqs = []
    for i, n in enumerate(lens):
        q, k, val = torch.randn((n, H, d), generator=g), torch.randn((n, G, d), generator=g), torch.randn((n, G, v), generator=g)
        for p in far:
            if p < n:
                k[p] = 3 * q[-1].view(G, H // G, d)[:, 0]
        q, k, val = q.to(dtype), k.to(dtype), val.to(dtype)
        for b in range(blocks[i]):
            table[i, b] = page = perm.pop()
            m = min(bs, n - b * bs)
            kp[page, :m], vp[page, :m] = 0, 0
            kp[page, :m, :, :d], vp[page, :m, :, :v] = k[b * bs:b * bs + m], val[b * bs:b * bs + m]
        seqs.append((q, k, val))
    return seqs, kp.to(gpu), vp.to(gpu), table.to(gpu)


def padded_rows(q, d):
    return torch.nn.functional.pad(q, (0, -d % 8)).contiguous()
