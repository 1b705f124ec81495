"""Small Kazozen configurations and random checkpoints for the tests (the checkpoint's config.json layout and tensor names)."""
import math

import torch


def dense(ff=20, limit=1.2):
    return {"kind": "dense", "ff": ff, "limit": limit}


def moe(experts=6, top=2, ff=12, count=2, keep=1, limit=0.8):
    """count = 0: the router has no groups."""
    r = {"experts": experts, "top": top}
    if count:
        r["groups"] = {"count": count, "keep": keep}
    return {"kind": "moe", "router": r, "expert": {"ff": ff, "limit": limit}}


def attention(heads=4, kv_heads=2, dim=8, vdim=6, size=11, keep=3, rot=None, base=300.0, scaling=(4.0, 24, 4.0, 0.5), scale=None, kv_from=None, mlp=None):
    """rot: rotated dims (None: all that pair up); scaling: (factor, original, fast, slow) or None."""
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "mask": {"size": size, "keep_first": keep},
         "rot": {"base": base, "dims": dim // 2 * 2 if rot is None else rot}, "scale": scale if scale is not None else 1.0 / math.sqrt(dim)}
    if scaling:
        m["rot"]["scaling"] = dict(zip(("factor", "original", "fast", "slow"), scaling))
    if kv_from is not None:
        m["kv_from"] = kv_from
    return {"type": "attention", "mixer": m, "mlp": mlp}


def config(layers, width=24, vocab=40, eps=1e-5, scale=3.0, bigram=(31, 7, 5), softcap=9.0):
    emb = {"scale": scale}
    if bigram:
        emb["bigram"] = dict(zip(("buckets", "mul_prev", "mul_cur"), bigram))
    return {"architecture": "Kazozen", "vocab": vocab, "width": width, "norm": {"eps": eps}, "logit_softcap": softcap, "embedding": emb, "layers": layers}


def random_checkpoint(cfg, seed=0, gain=1.0, embed=0.3):
    """bf16 tensors under the checkpoint's names.  gain multiplies the norm weights of the keys (scores that stand out)."""
    g = torch.Generator().manual_seed(seed)
    W = cfg["width"]

    def mat(*shape, s=1.0):
        return (torch.randn(*shape, generator=g) * (s / math.sqrt(shape[-1]))).to(torch.bfloat16)

    def vec(k, mean=0.0, std=0.2):
        return (mean + std * torch.randn(k, generator=g)).to(torch.bfloat16)
    S = {"embed": (torch.randn(cfg["vocab"], W, generator=g) * embed).to(torch.bfloat16), "final.norm": vec(W, 1.0, 0.3), "final.norm.b": vec(W)}
    bg = cfg["embedding"].get("bigram")
    if bg:
        S["bigram"] = (torch.randn(bg["buckets"] + 1, W, generator=g) * 0.6).to(torch.bfloat16)
    for i, L in enumerate(cfg["layers"]):
        m, p, q, mlp = L["mixer"], f"l{i}.mix.", f"l{i}.mlp.", L.get("mlp")
        H, G, d, e = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
        for s in (1, 2) if mlp else (1,):
            S.update({f"l{i}.norm{s}": vec(W, 0.6, 0.2), f"l{i}.norm{s}.b": vec(W)})
        S.update({p + "q": mat(H * d, W), p + "q.b": vec(H * d), p + "q.norm": vec(H * d, 1.0, 0.3), p + "g": mat(H * e, W), p + "sink": vec(H, 0.5, 1.0),
                  p + "o": mat(W, H * e)})
        if m.get("kv_from") is None:
            S.update({p + "k": mat(G * d, W), p + "k.b": vec(G * d), p + "k.norm": vec(G * d, gain, 0.3), p + "v": mat(G * e, W), p + "v.b": vec(G * e)})
        if mlp is None:
            continue
        if mlp["kind"] == "dense":
            S.update({q + "gate": mat(mlp["ff"], W), q + "up": mat(mlp["ff"], W), q + "down": mat(W, mlp["ff"])})
        else:
            f, n = mlp["expert"]["ff"], mlp["router"]["experts"]
            for j in range(n):
                S.update({f"{q}e{j}.gate": mat(f, W), f"{q}e{j}.up": mat(f, W), f"{q}e{j}.down": mat(W, f)})
            S[q + "router"], S[q + "correction"] = mat(n, W), vec(n, -0.3, 0.4)
    return S
