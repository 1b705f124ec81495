"""Small Gaparax configurations and random checkpoints for the tests (the checkpoint's config.json layout and tensor names)."""
import math

import torch


def dense(ff=20):
    return {"kind": "dense", "ff": ff}


def moe(experts=6, top=2, ff=12, count=3, keep=2, scale=1.7):
    return {"kind": "moe", "router": {"experts": experts, "top": top, "groups": {"count": count, "keep": keep}, "scale": scale},
            "expert": {"ff": ff}}


def attention(heads=4, kv_heads=2, dim=8, vdim=6, size=13, bias_max=11, rows=8, softcap=6.0, scale=None, mlp=None):
    """rows is no config key: it is the height of the bias table in the checkpoint (random_checkpoint reads it here)."""
    return {"type": "attention", "_rows": rows, "mlp": mlp,
            "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "mask": {"size": size}, "bias_max": bias_max,
                      "softcap": softcap, "scale": scale if scale is not None else 1.0 / math.sqrt(dim)}}


def latent(heads=3, dim=8, rot_dim=6, vdim=10, kv_rank=12, base=300.0, scaling=(4.0, 24, 4.0, 0.5), scale=None, mlp=None):
    """scaling: (factor, original, fast, slow) or None; rot_dim = 0: no rotated part."""
    m = {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "kv_rank": kv_rank,
         "scale": scale if scale is not None else 1.0 / math.sqrt(dim + rot_dim)}
    if rot_dim:
        m["rot"] = {"base": base, "dims": rot_dim}
        if scaling:
            m["rot"]["scaling"] = dict(zip(("factor", "original", "fast", "slow"), scaling))
    return {"type": "latent_attention", "mixer": m, "mlp": mlp}


def config(layers, width=24, vocab=40, eps=1e-5, streams=2):
    return {"architecture": "Gaparax", "vocab": vocab, "width": width, "streams": streams, "norm": {"eps": eps}, "layers": layers}


def public(cfg):
    """The config as a checkpoint folder holds it (without the helpers' private keys)."""
    c = dict(cfg)
    c["layers"] = [{k: v for k, v in L.items() if not k.startswith("_")} for L in cfg["layers"]]
    return c


def random_checkpoint(cfg, seed=0, gain=1.0, bias_std=1.0):
    """bf16 tensors under the checkpoint's names.  gain sharpens the query and key projections of latent attention (those of the other
    mixer are normed: its temperatures carry the gain); bias_std is the spread of the distance biases."""
    g = torch.Generator().manual_seed(seed)
    W, n = cfg["width"], cfg["streams"]

    def mat(*shape, s=1.0):
        return (torch.randn(*shape, generator=g) * (s / math.sqrt(shape[-1]))).to(torch.bfloat16)

    def vec(k, mean=0.0, std=0.2):
        return (mean + std * torch.randn(k, generator=g)).to(torch.bfloat16)
    S = {"embed": (torch.randn(cfg["vocab"], W, generator=g) * 0.7).to(torch.bfloat16), "head": mat(cfg["vocab"], W), "final.norm": vec(W, 1.0, 0.3)}
    for i, L in enumerate(cfg["layers"]):
        m, p, q, mlp = L["mixer"], f"l{i}.mix.", f"l{i}.mlp.", L.get("mlp")
        H, d, e = m["heads"], m["dim"], m["vdim"]
        for s in (1, 2) if mlp else (1,):
            S.update({f"l{i}.norm{s}": vec(W, 1.0, 0.3), f"l{i}.rg{s}": mat(W, W), f"l{i}.rg{s}.b": vec(W, 0.5, 0.5),
                      f"l{i}.hc{s}.in": vec(n, 1.0 / n, 0.4), f"l{i}.hc{s}.out": vec(n, 1.0, 0.4),
                      f"l{i}.hc{s}.mix": (torch.eye(n) * 0.8 + 0.3 * torch.randn(n, n, generator=g)).to(torch.bfloat16)})
        if L["type"] == "attention":
            G = m["kv_heads"]
            S.update({p + "q": mat(H * d, W), p + "k": mat(G * d, W), p + "v": mat(G * e, W), p + "g": mat(H * e, W), p + "o": mat(W, H * e),
                      p + "q.norm": vec(d, 1.0, 0.3), p + "k.norm": vec(d, 1.0, 0.3), p + "temp": vec(H, gain, 0.3), p + "pb": vec(H, -1.5, 0.7),
                      p + "rel": (torch.randn(L["_rows"], H, generator=g) * bias_std).to(torch.bfloat16)})
        else:
            r, R = m["rot_dim"], m["kv_rank"]
            S.update({p + "q": mat(H * (d + r), W, s=gain), p + "dkv": mat(R + r, W, s=gain), p + "dkv.norm": vec(R, 1.0, 0.3), p + "uk": mat(H * d, R),
                      p + "uv": mat(H * e, R), p + "sink": vec(H, 0.5, 1.0), p + "o": mat(W, H * e)})
        if mlp is None:
            continue
        if mlp["kind"] == "dense":
            S.update({q + "up": mat(mlp["ff"], W, s=1.5), q + "down": mat(W, mlp["ff"])})
        else:
            f = mlp["expert"]["ff"]
            for j in range(mlp["router"]["experts"]):
                S.update({f"{q}e{j}.gate": mat(f, W, s=2.0), f"{q}e{j}.up": mat(f, W, s=2.0), f"{q}e{j}.down": mat(W, f)})
            S[q + "router"] = mat(mlp["router"]["experts"], W, s=3.0)
    return S
