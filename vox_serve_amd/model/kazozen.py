"""Kazozen: a decoder-only language model on the hybrid engine (`engine_hybrid.HybridEngine`).

A checkpoint is a folder with `config.json` and `model.safetensors`.  config.json:
  architecture "Kazozen"; vocab, width; norm.eps; logit_softcap; embedding = {scale, bigram: {buckets, mul_prev, mul_cur}};
  layers[i] = {type: "attention", mixer: {heads, kv_heads, dim, vdim, scale, mask: {size, keep_first},
                                          rot: {base, dims, scaling: {factor, original, fast, slow}}, kv_from},
               mlp: null | {kind: "dense", ff, limit} | {kind: "moe", router: {experts, top, groups: {count, keep}}, expert: {ff, limit}}}.
Tensors (bf16, linear weights [out, in]): embed, bigram, final.norm, final.norm.b, and per layer l<i>.norm1, l<i>.norm1.b, l<i>.norm2,
l<i>.norm2.b, l<i>.mix.*, l<i>.mlp.*.

x0 = embed[token] * scale + bigram[pair of the previous token and this one].  Sublayers read the stream as it is and only what they return
is normed: x += norm1(mixer(x)); x += norm2(ff(x)), layer norms with weight and bias.  Logits = cap * tanh(embed . norm(x) / cap).
  attention   grouped-query softmax attention; biases in the q, k, v projections; q and k RMS-normed over the whole projection, then rotated
              (interleaved pairs, frequency-dependent scaling); a position sees the last mask.size tokens and the first mask.keep_first of its
              sequence; a learned sink per head in the denominator; the concatenated heads times sigmoid(g x); output projection.  A layer
              with kv_from = j has no k and v of its own and reads layer j's cache.
  units       down(a * sigmoid(1.702 a) * (b + 1)), a = min(gate x, limit), b = clamp(up x, -limit, limit), as the dense feed-forward and as
              the experts.
  router      scores sigmoid(z); choices by score + correction inside the groups.keep groups of neighbours whose two best choices have the
              largest sum; the chosen experts' plain scores are the weights.
The plugin fuses each mixer's projections into the engine's row order at load time.
"""
from typing import Dict

import torch

from ..engine_hybrid import HybridCfg, MixerCfg, MoECfg
from .hybrid_lm import HybridLM

ARCHITECTURE = "Kazozen"
SLOPE = 1.702           # of the sigmoid inside the gated units


def _ff_from_dict(i: int, mlp) -> dict:
    """-> the MixerCfg fields of the layer's feed-forward."""
    if mlp is None:
        return {}
    kind = mlp.get("kind")
    if kind == "dense":
        return dict(ff=int(mlp["ff"]), ff_kind="gated", ff_act="swish", ff_limit=float(mlp["limit"]), ff_alpha=SLOPE, ff_up_offset=1.0)
    if kind != "moe":
        raise ValueError(f"layer {i}: feed-forward kind {kind!r} is not part of this design")
    r = mlp["router"]
    experts, top, gr = int(r["experts"]), int(r["top"]), r.get("groups") or {"count": 1, "keep": 1}
    count, keep = int(gr["count"]), int(gr["keep"])
    if count < 1 or experts % count or not 1 <= keep <= count or not 1 <= top <= keep * (experts // count):
        raise ValueError(f"layer {i}: {top} of {experts} experts from {keep} of {count} groups")
    return dict(moe=MoECfg(experts=experts, identity=0, top=top, ff=int(mlp["expert"]["ff"]), limit=float(mlp["expert"]["limit"]), act_alpha=SLOPE,
                           score="sigmoid", renorm=False, up_offset=1.0, groups=count, keep=keep, group_best_two=True))


def config_from_dict(d: dict) -> HybridCfg:
    if d.get("architecture") != ARCHITECTURE:
        raise ValueError(f"not a {ARCHITECTURE} config: architecture = {d.get('architecture')!r}")
    layers = []
    for i, l in enumerate(d["layers"]):
        if l["type"] != "attention":
            raise ValueError(f"layer {i}: unknown mixer type {l['type']!r}")
        m = l["mixer"]
        H, G, dim, vdim = int(m["heads"]), int(m["kv_heads"]), int(m["dim"]), int(m["vdim"])
        if G < 1 or H % G:
            raise ValueError(f"layer {i}: {G} key heads do not divide {H} heads")
        mask, rot, src = m.get("mask") or {}, m.get("rot") or {}, m.get("kv_from")
        dims, sc = int(rot.get("dims", 0)), rot.get("scaling")
        if dims % 2 or not 0 <= dims <= dim:
            raise ValueError(f"layer {i}: {dims} rotated dims of {dim}")
        if src is not None:
            src = int(src)
            if not 0 <= src < i or layers[src].kv_from is not None or (layers[src].kv_heads, layers[src].dim, layers[src].vdim) != (G, dim, vdim):
                raise ValueError(f"layer {i}: cannot use the keys and values of layer {src}")
        layers.append(MixerCfg("window_attention", H, dim, vdim, kv_heads=G, scale=float(m["scale"]), window=int(mask.get("size") or 0),
                               keep_first=int(mask.get("keep_first") or 0), rot_dims=dims, rot_base=float(rot.get("base", 10000.0)),
                               rot_yarn=tuple(float(sc[k]) for k in ("factor", "original", "fast", "slow")) if sc else None, kv_from=src,
                               out_gate=True, qk_norm_whole=True, block="post_norm", **_ff_from_dict(i, l.get("mlp"))))
    emb = d.get("embedding") or {}
    bg, scale = emb.get("bigram"), emb.get("scale")
    return HybridCfg(int(d["width"]), int(d["vocab"]), float(d["norm"]["eps"]), layers, None, norm_kind="layer",
                     embed_scale=1.0 if scale is None else float(scale), logit_softcap=float(d.get("logit_softcap") or 0.0),
                     bigram=(int(bg["buckets"]), int(bg["mul_prev"]), int(bg["mul_cur"])) if bg else None)


def pack_weights(S: Dict[str, torch.Tensor], cfg: HybridCfg) -> Dict:
    """Checkpoint tensors -> the engine's fused layout."""
    layers = []
    for i, m in enumerate(cfg.layers):
        p, q = f"l{i}.mix.", f"l{i}.mlp."
        rows = ("q", "g") if m.kv_from is not None else ("q", "k", "v", "g")
        bias = [S[p + n + ".b"].float() if n != "g" else torch.zeros(S[p + n].shape[0]) for n in rows]
        lw = dict(norm1=S[f"l{i}.norm1"], norm1_b=S[f"l{i}.norm1.b"], norm2=S.get(f"l{i}.norm2"), norm2_b=S.get(f"l{i}.norm2.b"),
                  w_in=torch.cat([S[p + n] for n in rows], 0).contiguous(), b_in=torch.cat([b.to(S[p + "q"].device) for b in bias], 0).contiguous(),
                  w_out=S[p + "o"], q_norm=S[p + "q.norm"], k_norm=S.get(p + "k.norm"), sinks=S[p + "sink"])
        if m.moe is not None:
            e = m.moe
            lw["moe"] = dict(router=S[q + "router"], correction=S.get(q + "correction"),
                             w_gate_up=torch.stack([torch.cat([S[f"{q}e{j}.gate"], S[f"{q}e{j}.up"]], 0) for j in range(e.experts)]).contiguous(),
                             w_down=torch.stack([S[f"{q}e{j}.down"] for j in range(e.experts)]).contiguous())
        elif m.ff:
            lw.update(w_up=torch.cat([S[q + "gate"], S[q + "up"]], 0).contiguous(), w_down=S[q + "down"])
        layers.append(lw)
    return dict(embedding=S["embed"], head=S["embed"], bigram=S.get("bigram"), final_norm=S["final.norm"], final_norm_b=S["final.norm.b"], loop_in=None,
                layers=layers)


def synth_weights(cfg: HybridCfg, seed: int = 0) -> Dict[str, torch.Tensor]:
    """Random checkpoint tensors (bf16, the checkpoint's names) for a config: benchmarks."""
    g = torch.Generator().manual_seed(seed)
    W = cfg.width

    def lin(*shape):
        return (torch.randn(*shape, generator=g) / shape[-1] ** 0.5).to(torch.bfloat16)

    def vec(k, mean=0.0, std=0.1):
        return (mean + std * torch.randn(k, generator=g)).to(torch.bfloat16)
    S = {"embed": lin(cfg.vocab, W), "final.norm": vec(W, 1.0), "final.norm.b": vec(W)}
    if cfg.bigram:
        S["bigram"] = (torch.randn(cfg.bigram[0] + 1, W, generator=g) * 0.5).to(torch.bfloat16)
    for i, m in enumerate(cfg.layers):
        p, q = f"l{i}.mix.", f"l{i}.mlp."
        H, G, d, e = m.heads, m.kv_heads, m.dim, m.vdim
        S.update({f"l{i}.norm1": vec(W, 1.0), f"l{i}.norm1.b": vec(W), p + "q": lin(H * d, W), p + "q.b": vec(H * d), p + "q.norm": vec(H * d, 1.0),
                  p + "g": lin(H * e, W), p + "sink": vec(H), p + "o": lin(W, H * e)})
        if m.kv_from is None:
            S.update({p + "k": lin(G * d, W), p + "k.b": vec(G * d), p + "k.norm": vec(G * d, 1.0), p + "v": lin(G * e, W), p + "v.b": vec(G * e)})
        if m.moe is not None or m.ff:
            S.update({f"l{i}.norm2": vec(W, 1.0), f"l{i}.norm2.b": vec(W)})
        if m.moe is not None:
            x = m.moe
            for j in range(x.experts):
                S.update({f"{q}e{j}.gate": lin(x.ff, W), f"{q}e{j}.up": lin(x.ff, W), f"{q}e{j}.down": lin(W, x.ff)})
            S[q + "router"], S[q + "correction"] = lin(x.experts, W), vec(x.experts)
        elif m.ff:
            S.update({q + "gate": lin(m.ff, W), q + "up": lin(m.ff, W), q + "down": lin(W, m.ff)})
    return S


class KazozenModel(HybridLM):
    """The text-only plugin of `hybrid_lm.HybridLM` with this design's config reader and weight packer."""

    default_name = "kazozen"
    config_from_dict = staticmethod(config_from_dict)
    pack_weights = staticmethod(pack_weights)
