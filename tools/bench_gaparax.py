"""Prefill and decode throughput of the Gaparax design (random weights) at layer sizes of a real model, beside the framework's closest
existing model, Dipivik (latent attention and routed feed-forwards on the same engine), at the same width and number of layers.  bf16,
one GPU; both are driven directly (plan upload + one native step).

    python tools/bench_gaparax.py [--sizes 1024,2048] [--prompt 512,2048] [--batch 1,8] [--steps 30] [--warmup 5]

Gaparax layers per block of four: latent attention (heads = width/128 of 128 plain + 64 rotated dims, values of 128, cached latent
width/4 + 64 rotated key dims, scaled rotary) with a dense relu-squared feed-forward of 4 x width | latent attention with a routed
feed-forward of 8 experts in 4 groups of which 2 are kept, 2 per token, expert width = width | sigmoid-weighted attention (heads = width/128 on a quarter as
many key heads, 128 dims, chunks of 2048 positions, distance biases up to 2048) with the dense feed-forward | the same with the routed
one.  Two residual streams, a gate of width x width on every sublayer.  Vocabulary 32 000.  Prints one JSON object.
"""
import argparse
import json
import os
import sys

sys.path.insert(0, os.path.dirname(os.path.dirname(os.path.abspath(__file__))))
from tools.bench_dipivik import dipivik_cfg
from tools.bench_dipivik import step_bytes as dipivik_step_bytes
from tools.bench_sirodra import bench_hybrid_cfg


def gaparax_cfg(width, blocks, vocab, experts=8, top=2, chunk=2048):
    from vox_serve_amd.engine_hybrid import HybridCfg, MixerCfg, MoECfg
    h = width // 128

    def moe():
        return dict(moe=MoECfg(experts=experts, identity=0, top=top, ff=width, limit=float("inf"), act_alpha=1.0, score="softmax", renorm=False,
                               up_offset=0.0, groups=4, keep=2, weight_scale=1.5))

    def dense():
        return dict(ff=4 * width, ff_kind="up_down", ff_act="relu2")

    def lat(ff):
        return MixerCfg("latent_attention", h, 128, 128, kv_rank=width // 4, rot_dim=64, rot_dims=64, rot_base=1e5, rot_yarn=(8.0, 4096.0, 24.0, 2.0),
                        scale=192 ** -0.5, head_gate=False, res_gate=True, **ff)

    def sig(ff):
        return MixerCfg("sigmoid_attention", h, 128, 128, kv_heads=max(1, h // 4), chunk=chunk, score_cap=30.0, dist_max=chunk, scale=128 ** -0.5,
                        out_gate=True, res_gate=True, **ff)
    layers = []
    for _ in range(blocks):
        layers += [lat(dense()), lat(moe()), sig(dense()), sig(moe())]
    return HybridCfg(width, vocab, 1e-5, layers, None, norm_kind="rms_groups", norm_groups=1, streams=2)


def step_bytes(cfg):
    """bf16 weight bytes a one-row decode step streams: all mixers, the gates, the chosen experts, router (fp32), head."""
    W = cfg.width
    n = cfg.vocab * W
    for m in cfg.layers:
        n += m.n_in * W + W * m.heads * m.vdim + 2 * W * W
        if m.kind == "latent_attention":
            n += m.heads * m.kv_rank * (m.dim + m.vdim)
        e = m.moe
        n += 2 * m.ff * W if e is None else 3 * e.top * e.ff * W + 2 * e.experts * W
    return 2 * n


def run(sizes=(1024, 2048), prompts=(512, 2048), batches=(1, 8), blocks=3, vocab=32000, ctx=1024, steps=30, warmup=5, device="cuda:0", only=None):
    from vox_serve_amd.model import dipivik, gaparax
    res = {"workload": "Gaparax layer pattern (latent attention + dense FF | latent + routed FF | chunked sigmoid attention + dense | the same + "
                       "routed) x %d blocks vs the Dipivik pattern of the same depth, bf16, random weights, decode context %d" % (blocks, ctx),
           "sizes": {}}
    for W in sizes:
        ent = {}
        if only in (None, "gaparax"):
            cfg = gaparax_cfg(W, blocks, vocab)
            packed = gaparax.pack_weights(gaparax.synth_weights(cfg), cfg)
            ent["gaparax"] = bench_hybrid_cfg(cfg, packed, step_bytes(cfg), prompts, batches, ctx, steps, warmup, device)
        if only in (None, "dipivik"):
            cfg = dipivik_cfg(W, blocks, vocab)
            packed = dipivik.pack_weights(dipivik.synth_weights(cfg), cfg)
            ent["dipivik"] = bench_hybrid_cfg(cfg, packed, dipivik_step_bytes(cfg), prompts, batches, ctx, steps, warmup, device)
        res["sizes"][str(W)] = ent
    return res


if __name__ == "__main__":
    ap = argparse.ArgumentParser()
    ap.add_argument("--sizes", default="1024,2048")
    ap.add_argument("--prompt", default="512,2048")
    ap.add_argument("--batch", default="1,8")
    ap.add_argument("--blocks", type=int, default=3)
    ap.add_argument("--steps", type=int, default=30)
    ap.add_argument("--warmup", type=int, default=5)
    ap.add_argument("--only", default=None, choices=[None, "gaparax", "dipivik"])
    a = ap.parse_args()
    ints = lambda s: tuple(int(x) for x in s.split(","))
    print(json.dumps(run(ints(a.sizes), ints(a.prompt), ints(a.batch), a.blocks, steps=a.steps, warmup=a.warmup, only=a.only)))
