"""Prefill and decode throughput of the Kazozen design (random weights) at layer sizes of a real model, beside the framework's closest
existing model, Gaparax (grouped attention with an output gate and group-limited routing on the same engine), at the same width and number of
layers.  bf16, one GPU; both are driven directly (plan upload + one native step).

    python tools/bench_kazozen.py [--sizes 1024,2048] [--prompt 512,2048] [--batch 1,8] [--steps 30] [--warmup 5]

Kazozen layers per block of four: window attention (heads = width/128 on a quarter as many key heads, 128 dims, window of 1024 tokens, four
kept first tokens, scaled rotary) with a dense gated feed-forward of 8/3 x width | the same on the keys and values of the layer before with
a routed feed-forward of 8 experts in 4 groups of which 2 are kept, 2 per token, expert width = width | the two once more.  A bigram
embedding of 4096 rows, a tied head with a soft cap.  Vocabulary 32 000.  Prints one JSON object.
"""
import argparse
import json
import os
import sys

sys.path.insert(0, os.path.dirname(os.path.dirname(os.path.abspath(__file__))))
from tools.bench_gaparax import gaparax_cfg
from tools.bench_gaparax import step_bytes as gaparax_step_bytes
from tools.bench_sirodra import bench_hybrid_cfg


def kazozen_cfg(width, blocks, vocab, experts=8, top=2, window=1024):
    from vox_serve_amd.engine_hybrid import HybridCfg, MixerCfg, MoECfg
    h = width // 128

    def attn(kv_from, **ff):
        return MixerCfg("window_attention", h, 128, 128, kv_heads=max(1, h // 4), window=window, keep_first=4, scale=128 ** -0.5, rot_dims=128,
                        rot_base=1e6, rot_yarn=(4.0, 4096.0, 32.0, 1.0), kv_from=kv_from, out_gate=True, qk_norm_whole=True, block="post_norm", **ff)

    def moe():
        return dict(moe=MoECfg(experts=experts, identity=0, top=top, ff=width, limit=7.0, act_alpha=1.702, score="sigmoid", renorm=False, up_offset=1.0,
                               groups=4, keep=2, group_best_two=True))
    dense = dict(ff=(8 * width // 3 + 255) // 256 * 256, ff_kind="gated", ff_act="swish", ff_limit=7.0, ff_alpha=1.702, ff_up_offset=1.0)
    layers = []
    for _ in range(2 * blocks):
        layers += [attn(None, **dense), attn(len(layers), **moe())]
    return HybridCfg(width, vocab, 1e-5, layers, None, norm_kind="layer", embed_scale=width ** 0.5, logit_softcap=30.0, bigram=(4096, 1009, 17))


def step_bytes(cfg):
    """bf16 weight bytes a one-row decode step streams: all mixers, the dense units or chosen experts, router (fp32), head."""
    W = cfg.width
    n = cfg.vocab * W
    for m in cfg.layers:
        e = m.moe
        n += m.n_in * W + W * m.heads * m.vdim + (3 * m.ff * W if e is None else 3 * e.top * e.ff * W + 2 * e.experts * W)
    return 2 * n


def run(sizes=(1024, 2048), prompts=(512, 2048), batches=(1, 8), blocks=3, vocab=32000, ctx=1024, steps=30, warmup=5, device="cuda:0", only=None):
    from vox_serve_amd.model import gaparax, kazozen
    res = {"workload": "Kazozen layer pattern (window attention + dense FF | the same on shared keys and values + routed FF, twice) x %d blocks vs the "
                       "Gaparax pattern of the same depth, bf16, random weights, decode context %d" % (blocks, ctx), "sizes": {}}
    for W in sizes:
        ent = {}
        for name, mod, make, nbytes in (("kazozen", kazozen, kazozen_cfg, step_bytes), ("gaparax", gaparax, gaparax_cfg, gaparax_step_bytes)):
            if only in (None, name):
                cfg = make(W, blocks, vocab)
                ent[name] = bench_hybrid_cfg(cfg, mod.pack_weights(mod.synth_weights(cfg), cfg), nbytes(cfg), prompts, batches, ctx, steps, warmup, device)
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
    ap.add_argument("--only", default=None, choices=[None, "kazozen", "gaparax"])
    a = ap.parse_args()
    ints = lambda s: tuple(int(x) for x in s.split(","))
    print(json.dumps(run(ints(a.sizes), ints(a.prompt), ints(a.batch), a.blocks, steps=a.steps, warmup=a.warmup, only=a.only)))
