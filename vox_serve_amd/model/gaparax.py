"""Gaparax: a decoder-only language model on the hybrid engine (`engine_hybrid.HybridEngine`).

A checkpoint is a folder with `config.json` and `model.safetensors`.  config.json:
  architecture "Gaparax"; vocab, width; streams; norm.eps;
  layers[i] = {type: "attention" | "latent_attention", mixer: {...},
               mlp: null | {kind: "dense", ff} | {kind: "moe", router: {experts, top, groups: {count, keep}, scale}, expert: {ff}}}.
Tensors (bf16, linear weights [out, in]): embed, head, final.norm, and per layer l<i>.norm1, l<i>.norm2, l<i>.hc<q>.{in, out, mix},
l<i>.rg<q>, l<i>.rg<q>.b (q = 1 mixer, 2 feed-forward), l<i>.mix.*, l<i>.mlp.*.

The residual stream is `streams` copies x_s, all the embedding at the start.  Sublayer q reads u = sum_s in[s] x_s; with n = norm u its
result y = f(n) * sigmoid(rg n + b) enters as x_t <- sum_s mix[s, t] x_s + out[t] y; the head reads the norm of the sum of the streams.
The mixers:
  attention         grouped-query attention inside chunks of mask.size positions; q and k RMS-normed per head (weights shared by the
                    heads); z = softcap * tanh(q.k * scale * temp_h / softcap) + rel[bucket(distance), h]; every visible key weighs
                    sigmoid(z + pb_h), without a softmax; the concatenated heads times sigmoid(g n); output projection.
  latent_attention  q = heads of [dim plain | rot_dim rotated]; dkv n = key / value latent (kv_rank, RMS norm, weight) | one rotated key
                    part shared by the heads, both all the cache keeps; plain keys uk latent and values uv latent per head; rotate-half
                    rotary with the frequency-dependent scaling of rot.scaling; softmax over all earlier tokens with a learned sink per
                    head in the denominator; output projection.
The dense feed-forward is down(relu(up n)^2).  The routed one takes a softmax over all experts, keeps the best groups of neighbouring
experts, the `top` largest scores inside them are the weights (times router.scale); experts are silu gated units.
The plugin fuses each mixer's projections and the gate on its result into the engine's row order at load time.
"""
from typing import Dict

import torch

from ..engine_hybrid import HybridCfg, MixerCfg, MoECfg
from .hybrid_lm import HybridLM

ARCHITECTURE = "Gaparax"
NO_LIMIT = float("inf")         # the experts' units are not clamped


def _ff_from_dict(i: int, mlp) -> dict:
    """-> the MixerCfg fields of the layer's feed-forward."""
    if mlp is None:
        return {}
    kind = mlp.get("kind")
    if kind == "dense":
        return dict(ff=int(mlp["ff"]), ff_kind="up_down", ff_act="relu2")
    if kind != "moe":
        raise ValueError(f"layer {i}: feed-forward kind {kind!r} is not part of this design")
    r = mlp["router"]
    experts, top, gr = int(r["experts"]), int(r["top"]), r.get("groups") or {"count": 1, "keep": 1}
    count, keep = int(gr["count"]), int(gr["keep"])
    if count < 1 or experts % count or not 1 <= keep <= count or not 1 <= top <= keep * (experts // count):
        raise ValueError(f"layer {i}: {top} of {experts} experts from {keep} of {count} groups")
    scale = r.get("scale")
    return dict(moe=MoECfg(experts=experts, identity=0, top=top, ff=int(mlp["expert"]["ff"]), limit=NO_LIMIT, act_alpha=1.0, score="softmax",
                           renorm=False, up_offset=0.0, groups=count, keep=keep, weight_scale=1.0 if scale is None else float(scale)))


def config_from_dict(d: dict) -> HybridCfg:
    if d.get("architecture") != ARCHITECTURE:
        raise ValueError(f"not a {ARCHITECTURE} config: architecture = {d.get('architecture')!r}")
    layers = []
    for i, l in enumerate(d["layers"]):
        t, m = l["type"], l["mixer"]
        common = dict(scale=float(m["scale"]), res_gate=True, **_ff_from_dict(i, l.get("mlp")))
        H, dim, vdim = int(m["heads"]), int(m["dim"]), int(m["vdim"])
        if t == "attention":
            G = int(m["kv_heads"])
            if H % G:
                raise ValueError(f"layer {i}: {G} key heads do not divide {H} heads")
            layers.append(MixerCfg("sigmoid_attention", H, dim, vdim, kv_heads=G, chunk=int(m["mask"]["size"]), score_cap=float(m["softcap"]),
                                   dist_max=int(m["bias_max"]), out_gate=True, **common))
        elif t == "latent_attention":
            rot = m.get("rot") or {}
            dims, sc = int(rot.get("dims", 0)), rot.get("scaling")
            if dims > int(m["rot_dim"]):
                raise ValueError(f"layer {i}: {dims} rotated dims in a part of {m['rot_dim']}")
            layers.append(MixerCfg("latent_attention", H, dim, vdim, kv_rank=int(m["kv_rank"]), rot_dim=int(m["rot_dim"]), rot_dims=dims,
                                   rot_base=float(rot.get("base", 10000.0)), head_gate=False,
                                   rot_yarn=tuple(float(sc[k]) for k in ("factor", "original", "fast", "slow")) if sc else None, **common))
        else:
            raise ValueError(f"layer {i}: unknown mixer type {t!r}")
    return HybridCfg(int(d["width"]), int(d["vocab"]), float(d["norm"]["eps"]), layers, None, norm_kind="rms_groups", norm_groups=1,
                     streams=int(d["streams"]))


def pack_weights(S: Dict[str, torch.Tensor], cfg: HybridCfg) -> Dict:
    """Checkpoint tensors -> the engine's fused layout."""
    layers = []
    for i, m in enumerate(cfg.layers):
        p, q = f"l{i}.mix.", f"l{i}.mlp."
        subs = (1, 2) if (m.moe is not None or m.ff) else (1,)
        lw = dict(norm1=S[f"l{i}.norm1"], norm2=S.get(f"l{i}.norm2"), w_out=S[p + "o"], w_gate_in=S[f"l{i}.rg1"], b_gate_in=S[f"l{i}.rg1.b"],
                  w_gate_ff=S.get(f"l{i}.rg2"), b_gate_ff=S.get(f"l{i}.rg2.b"))
        for n in ("in", "out", "mix"):
            lw["hc_" + n] = [S[f"l{i}.hc{s}.{n}"] for s in subs]
        if tuple(lw["hc_mix"][0].shape) != (cfg.streams, cfg.streams):
            raise ValueError(f"layer {i}: streams are mixed by {tuple(lw['hc_mix'][0].shape)}, config says {cfg.streams}")
        if m.kind == "sigmoid_attention":
            lw.update(w_in=torch.cat([S[p + n] for n in ("q", "k", "v", "g")], 0).contiguous(), q_norm=S[p + "q.norm"], k_norm=S[p + "k.norm"],
                      head_temp=S[p + "temp"], dist_table=S[p + "rel"], weight_bias=S[p + "pb"])
        else:
            H, d, R = m.heads, m.dim, m.kv_rank
            lw.update(w_in=torch.cat([S[p + "q"], S[p + "dkv"]], 0).contiguous(), kv_lat_norm=S[p + "dkv.norm"], w_uv=S[p + "uv"], sinks=S[p + "sink"],
                      # per head the transpose of its rows of uk: [H][R][d], so that (plain query) x (this) is the query against the latent
                      w_ukT=S[p + "uk"].view(H, d, R).transpose(1, 2).contiguous())
        if m.moe is not None:
            e = m.moe
            lw["moe"] = dict(router=S[q + "router"], correction=None,
                             w_gate_up=torch.stack([torch.cat([S[f"{q}e{j}.gate"], S[f"{q}e{j}.up"]], 0) for j in range(e.experts)]).contiguous(),
                             w_down=torch.stack([S[f"{q}e{j}.down"] for j in range(e.experts)]).contiguous())
        elif m.ff:
            lw.update(w_up=S[q + "up"], w_down=S[q + "down"])
        layers.append(lw)
    return dict(embedding=S["embed"], head=S["head"], final_norm=S["final.norm"], loop_in=None, layers=layers)


def synth_weights(cfg: HybridCfg, seed: int = 0, bias_rows: int = 32) -> Dict[str, torch.Tensor]:
    """Random checkpoint tensors (bf16, the checkpoint's names) for a config: benchmarks."""
    g = torch.Generator().manual_seed(seed)
    W, n = cfg.width, cfg.streams

    def lin(*shape):
        return (torch.randn(*shape, generator=g) / shape[-1] ** 0.5).to(torch.bfloat16)

    def vec(k, mean=0.0, std=0.1):
        return (mean + std * torch.randn(k, generator=g)).to(torch.bfloat16)
    S = {"embed": (torch.randn(cfg.vocab, W, generator=g) * 0.5).to(torch.bfloat16), "head": lin(cfg.vocab, W), "final.norm": vec(W, 1.0)}
    for i, m in enumerate(cfg.layers):
        p, q = f"l{i}.mix.", f"l{i}.mlp."
        H, d, e = m.heads, m.dim, m.vdim
        for s in (1, 2) if (m.moe is not None or m.ff) else (1,):
            S.update({f"l{i}.norm{s}": vec(W, 1.0), f"l{i}.rg{s}": lin(W, W), f"l{i}.rg{s}.b": vec(W), f"l{i}.hc{s}.in": vec(n, 1.0 / n),
                      f"l{i}.hc{s}.out": vec(n, 1.0), f"l{i}.hc{s}.mix": (torch.eye(n) + 0.05 * torch.randn(n, n, generator=g)).to(torch.bfloat16)})
        if m.kind == "sigmoid_attention":
            G = m.kv_heads
            S.update({p + "q": lin(H * d, W), p + "k": lin(G * d, W), p + "v": lin(G * e, W), p + "g": lin(H * e, W), p + "q.norm": vec(d, 1.0),
                      p + "k.norm": vec(d, 1.0), p + "temp": vec(H, 1.0), p + "rel": lin(bias_rows, H), p + "pb": vec(H, -4.0)})
        else:
            S.update({p + "q": lin(H * (d + m.rot_dim), W), p + "dkv": lin(m.kv_rank + m.rot_dim, W), p + "dkv.norm": vec(m.kv_rank, 1.0),
                      p + "uk": lin(H * d, m.kv_rank), p + "uv": lin(H * e, m.kv_rank), p + "sink": vec(H)})
        S[p + "o"] = lin(W, H * e)
        if m.moe is not None:
            x = m.moe
            for j in range(x.experts):
                S.update({f"{q}e{j}.gate": lin(x.ff, W), f"{q}e{j}.up": lin(x.ff, W), f"{q}e{j}.down": lin(W, x.ff)})
            S[q + "router"] = lin(x.experts, W)
        elif m.ff:
            S.update({q + "up": lin(m.ff, W), q + "down": lin(W, m.ff)})
    return S


class GaparaxModel(HybridLM):
    """The text-only plugin of `hybrid_lm.HybridLM` with this design's config reader and weight packer."""

    default_name = "gaparax"
    config_from_dict = staticmethod(config_from_dict)
    pack_weights = staticmethod(pack_weights)
