"""Host-side pieces of the Gaparax path that need no GPU: the config reader, the fused weight layout, the tables the engine is given
(scaled rotary frequencies, distance biases), the registry entry, and identities and sensitivities of the oracle itself (causality,
chunks, streams, the sink, the routing groups)."""
import copy
import math

import pytest
import torch

from oracle import gaparax_ref as GR
from tests import gaparax_util as P

F32_BAR = 2e-4


def rel_err(got, want):
    d = got - want
    d = d - d.mean(-1, keepdim=True)
    w = want - want.mean(-1, keepdim=True)
    return float((d.pow(2).mean(-1).sqrt() / w.pow(2).mean().sqrt()).max())


def tokens(n, vocab, seed):
    return torch.randint(0, vocab, (n,), generator=torch.Generator().manual_seed(seed)).tolist()


def small():
    return P.config([P.latent(heads=3, dim=6, rot_dim=4, vdim=5, kv_rank=9, scale=0.4, mlp=P.dense(14)),
                     P.attention(heads=6, kv_heads=3, dim=8, vdim=10, size=7, bias_max=12, rows=6, softcap=9.0, scale=0.3, mlp=P.moe()),
                     P.latent(heads=2, scaling=None, mlp=None)], streams=3)


def test_config_reader_takes_every_size_and_constant():
    from vox_serve_amd.model.gaparax import config_from_dict
    c = config_from_dict(P.public(small()))
    assert (c.width, c.vocab, c.eps, c.norm_kind, c.norm_groups, c.norm_one_plus, c.streams, c.loop) == (24, 40, 1e-5, "rms_groups", 1, False, 3, None)
    a, b, d = c.layers
    assert (a.kind, a.heads, a.dim, a.rot_dim, a.rot_dims, a.vdim, a.kv_rank, a.q_rank, a.scale, a.head_gate, a.res_gate, a.window) == \
        ("latent_attention", 3, 6, 4, 4, 5, 9, 0, 0.4, False, True, 0)
    assert a.rot_base == 300.0 and a.rot_yarn == (4.0, 24.0, 4.0, 0.5) and d.rot_yarn is None
    assert (a.ff, a.ff_kind, a.ff_act, a.moe, a.block) == (14, "up_down", "relu2", None, "sequential")
    assert (b.kind, b.heads, b.kv_heads, b.dim, b.vdim, b.chunk, b.dist_max, b.score_cap, b.scale, b.out_gate, b.res_gate) == \
        ("sigmoid_attention", 6, 3, 8, 10, 7, 12, 9.0, 0.3, True, True)
    e = b.moe
    assert (e.experts, e.identity, e.top, e.ff, e.shared_ff, e.groups, e.keep, e.weight_scale) == (6, 0, 2, 12, 0, 3, 2, 1.7)
    assert (e.score, e.renorm, e.scale_input, e.limit, e.act_alpha, e.up_offset, e.expert_form) == ("softmax", False, False, math.inf, 1.0, 0.0, "gated")
    assert (d.ff, d.moe) == (0, None)
    assert a.n_in == 3 * 10 + 13 and a.cache_values() == 13 and a.state_floats(24) == 0
    assert b.n_in == 48 + 24 + 30 + 60 and b.cache_values() == 3 * 18 and b.state_floats(24) == 0
    plain = P.public(small())
    del plain["layers"][1]["mlp"]["router"]["groups"], plain["layers"][1]["mlp"]["router"]["scale"]
    e = config_from_dict(plain).layers[1].moe
    assert (e.groups, e.keep, e.weight_scale) == (1, 1, 1.0)


@pytest.mark.parametrize("break_it", [
    lambda c: c.update(architecture="Other"),
    lambda c: c["layers"][0].update(type="other"),
    lambda c: c["layers"][0]["mlp"].update(kind="other"),
    lambda c: c["layers"][1]["mixer"].update(kv_heads=4),
    lambda c: c["layers"][0]["mixer"]["rot"].update(dims=6),
    lambda c: c["layers"][1]["mlp"]["router"]["groups"].update(count=4),
    lambda c: c["layers"][1]["mlp"]["router"]["groups"].update(keep=4),
    lambda c: c["layers"][1]["mlp"]["router"].update(top=5),
])
def test_config_reader_refuses(break_it):
    from vox_serve_amd.model.gaparax import config_from_dict
    bad = copy.deepcopy(P.public(small()))
    break_it(bad)
    with pytest.raises(ValueError):
        config_from_dict(bad)


def test_pack_weights_layout():
    from vox_serve_amd.model.gaparax import config_from_dict, pack_weights
    cfg = small()
    S = P.random_checkpoint(cfg, seed=3)
    w = pack_weights(S, config_from_dict(P.public(cfg)))
    a, b, d = w["layers"]
    assert tuple(a["w_in"].shape) == (43, 24) and torch.equal(a["w_in"][:30], S["l0.mix.q"]) and torch.equal(a["w_in"][30:], S["l0.mix.dkv"])
    assert a["w_gate_in"] is S["l0.rg1"] and a["b_gate_ff"] is S["l0.rg2.b"] and a["sinks"] is S["l0.mix.sink"] and a["w_up"] is S["l0.mlp.up"]
    # a plain query against the expanded key of a latent = the folded query against the latent itself
    q, c = torch.randn(3, 6), torch.randn(9)
    k = (S["l0.mix.uk"].float() @ c).view(3, 6)
    for h in range(3):
        assert torch.allclose(q[h] @ k[h], (a["w_ukT"][h].float() @ q[h]) @ c, atol=1e-4)
    assert tuple(b["w_in"].shape) == (162, 24) and torch.equal(b["w_in"][48:72], S["l1.mix.k"]) and torch.equal(b["w_in"][102:], S["l1.mix.g"])
    assert b["head_temp"] is S["l1.mix.temp"] and b["dist_table"] is S["l1.mix.rel"] and b["weight_bias"] is S["l1.mix.pb"]
    assert tuple(b["moe"]["w_gate_up"].shape) == (6, 24, 24) and torch.equal(b["moe"]["w_gate_up"][2][12:], S["l1.mlp.e2.up"])
    assert tuple(b["moe"]["w_down"].shape) == (6, 24, 12) and b["moe"]["router"] is S["l1.mlp.router"]
    assert len(b["hc_in"]) == 2 and b["hc_mix"][1] is S["l1.hc2.mix"] and len(d["hc_out"]) == 1 and d["norm2"] is None
    assert w["head"] is S["head"] and w["embedding"] is S["embed"]
    narrow = dict(S, **{"l0.hc1.mix": torch.eye(2)})
    with pytest.raises(ValueError):
        pack_weights(narrow, config_from_dict(P.public(cfg)))


def test_synthetic_weights_fit_the_reader():
    from vox_serve_amd.model.gaparax import config_from_dict, pack_weights, synth_weights
    c = config_from_dict(P.public(small()))
    S = synth_weights(c)
    R = P.random_checkpoint(small())
    assert set(S) == set(R) and all(tuple(S[k].shape) == tuple(R[k].shape) for k in S if not k.endswith(".rel"))
    assert len(pack_weights(S, c)["layers"]) == 3


def test_registry_names_the_design():
    from vox_serve_amd.model import MODEL_REGISTRY, get_model_class
    assert "gaparax" in MODEL_REGISTRY and get_model_class("Gaparax") is MODEL_REGISTRY["gaparax"]


@pytest.mark.parametrize("dims,base,sc", [(8, 300.0, (4.0, 24, 4.0, 0.5)), (32, 1e4, (8.0, 4096, 32.0, 1.0)), (16, 50.0, (2.0, 4000, 64.0, 1.0)), (4, 1e6, (1.0, 100, 8.0, 2.0)),
                                          (8, 100.0, (2.0, 50, 1.01, 1.0))])
def test_scaled_rotary_frequencies(dims, base, sc):
    """The engine's table against the oracle's; fast pairs keep their frequency, slow ones are divided by the factor."""
    from vox_serve_amd.engine_hybrid import yarn_frequencies
    got, mag = yarn_frequencies(dims, base, *[float(x) for x in sc])
    want, wmag = GR.yarn_frequencies(dims, base, dict(zip(("factor", "original", "fast", "slow"), sc)))
    assert torch.allclose(got.double(), torch.tensor(want, dtype=torch.float64), rtol=1e-6) and math.isclose(mag, wmag)
    for i, f in enumerate(want):
        plain = base ** (-2.0 * i / dims)
        assert plain / sc[0] * (1 - 1e-12) <= f <= plain * (1 + 1e-12)


@pytest.mark.parametrize("rows,far,longest", [(8, 20, 100), (7, 33, 100), (16, 16, 12), (2, 9, 50), (32, 300, 120), (6, 3, 40), (12, 500, 1000)])
def test_distance_bias_table(rows, far, longest):
    """One entry per distance below `longest`, or up to the distance from which the last row holds; a clamped reader sees the oracle's
    bucket at every distance."""
    from vox_serve_amd.engine_hybrid import distance_bias
    table = torch.randn(rows, 3)
    t = distance_bias(table, far, longest)
    assert t.shape[0] == 3 and 1 <= t.shape[1] <= longest
    for n in range(longest):
        assert torch.equal(t[:, min(n, t.shape[1] - 1)], table[GR.distance_bucket(n, rows, far)] if far > rows // 2 else table[min(n, rows // 2)
                           if n < rows // 2 else rows - 1])


def test_distance_buckets_of_the_oracle():
    assert [GR.distance_bucket(n, 8, 32) for n in (0, 1, 3, 4, 5, 7, 8, 16, 31, 32, 1000)] == [0, 1, 3, 4, 4, 5, 5, 6, 7, 7, 7]


def test_oracle_is_causal_and_chunks_are_separate():
    cfg = small()
    S = P.random_checkpoint(cfg, seed=5)
    toks = tokens(30, 40, 6)
    full = GR.forward(cfg, S, toks)
    assert torch.allclose(GR.forward(cfg, S, toks[:17]), full[:17], atol=1e-12)
    other = list(toks)
    other[20] = (other[20] + 1) % 40
    assert torch.allclose(GR.forward(cfg, S, other)[:20], full[:20], atol=1e-12)
    assert not torch.allclose(GR.forward(cfg, S, other)[20:], full[20:], atol=1e-6)
    # attention layers alone: a token moves its own chunk only, and a chunk's logits are those of the chunk as a sequence of its own
    solo = P.config([P.attention(size=7), P.attention(size=7, kv_heads=4, mlp=P.dense())])
    S = P.random_checkpoint(solo, seed=6)
    full = GR.forward(solo, S, toks)
    other = list(toks)
    other[9] = (other[9] + 1) % 40
    moved = (GR.forward(solo, S, other) - full).abs().amax(-1) > 1e-9
    assert moved[9:14].any() and not moved[:9].any() and not moved[14:].any()
    assert torch.allclose(GR.forward(solo, S, toks[14:21]), full[14:21], atol=1e-12)


def test_oracle_streams():
    """One stream with weights of one is the plain residual sum; streams that are never mixed and read by halves are too."""
    cfg = P.config([P.attention(mlp=P.dense()), P.latent(mlp=None)], streams=1)
    S = P.random_checkpoint(cfg, seed=7)
    for k in [k for k in S if ".hc" in k]:
        S[k] = torch.ones_like(S[k])
    toks = tokens(20, 40, 8)
    one = GR.forward(cfg, S, toks)
    Sd = {k: v.double() for k, v in S.items()}
    x = Sd["embed"][torch.tensor(toks)]
    for i, q in ((0, 1), (0, 2), (1, 1)):
        Q = GR.sub(Sd, f"l{i}.")
        n = GR.rms_norm(x, Q[f"norm{q}"], cfg["norm"]["eps"])
        m = cfg["layers"][i]["mixer"]
        y = GR.dense_ff(GR.sub(Q, "mlp."), n) if q == 2 else (GR.attention_mixer if i == 0 else GR.latent_mixer)(GR.sub(Q, "mix."), n, m, cfg["norm"]["eps"])
        x = x + y * GR.residual_gate(Q, q, n)
    assert torch.allclose(GR.rms_norm(x, Sd["final.norm"], cfg["norm"]["eps"]) @ Sd["head"].T, one, atol=1e-10)
    two = copy.deepcopy(cfg)
    two["streams"] = 2
    T = dict(S)
    for k in [k for k in S if ".hc" in k]:
        T[k] = torch.eye(2) if k.endswith("mix") else torch.full((2,), 0.5 if k.endswith("in") else 1.0)
    assert torch.allclose(GR.forward(two, T, toks), one, atol=1e-4)        # (twice the stream: the final norm's eps alone tells them apart)


def test_oracle_tells_the_mechanisms_apart():
    """A mechanism left out or one off moves the logits by far more than the bar."""
    cfg = P.config([P.latent(heads=3, mlp=P.moe()), P.attention(size=13, mlp=P.dense())], streams=2)
    S = P.random_checkpoint(cfg, seed=9, gain=2.0)
    toks = tokens(60, 40, 10)
    want = GR.forward(cfg, S, toks)

    def moved(**names):
        orig = {k: getattr(GR, k) for k in names}
        try:
            for k, f in names.items():
                setattr(GR, k, f(orig[k]))
            return rel_err(GR.forward(cfg, S, toks), want)
        finally:
            for k, f in orig.items():
                setattr(GR, k, f)
    bar = 50 * F32_BAR
    assert moved(chunk_mask=lambda f: lambda T, size: f(T, size + 1)) > bar
    assert moved(chunk_mask=lambda f: lambda T, size: f(T, 10 ** 6)) > bar
    assert moved(distance_bucket=lambda f: lambda n, r, far: f(n + 1, r, far)) > bar
    assert moved(softcap=lambda f: lambda s, cap: s) > bar
    assert moved(sink_softmax=lambda f: lambda s, sink: torch.softmax(s, -1)) > bar
    assert moved(residual_gate=lambda f: lambda Q, q, n: 1.0) > bar
    assert moved(write_streams=lambda f: lambda xs, mix, out, y: f(xs, mix.T, out, y)) > bar
    assert moved(read_streams=lambda f: lambda xs, w: xs[0]) > bar
    assert moved(rotate_halves=lambda f: lambda x, pos, fr, mag: f(x, pos, fr, 1.0)) > bar
    assert moved(relu_squared=lambda f: lambda z: torch.clamp(z, min=0.0)) > bar
    assert moved(route=lambda f: lambda Q, n, r: f(Q, n, dict(r, scale=1.0))) > bar
    assert moved(route=lambda f: lambda Q, n, r: f(Q, n, dict(r, groups={"count": 3, "keep": 1}))) > bar


def test_oracle_rotation_depends_on_distance():
    """Rotated queries against rotated keys depend on how far apart they are, not on where they stand; the pairs' scale enters squared."""
    fr, mag = GR.yarn_frequencies(6, 300.0, {"factor": 4.0, "original": 24, "fast": 4.0, "slow": 0.5})
    q, k = torch.randn(1, 1, 8, dtype=torch.float64), torch.randn(1, 1, 8, dtype=torch.float64)

    def score(i, j, m=mag):
        return float((GR.rotate_halves(q, torch.tensor([i]), fr, m) * GR.rotate_halves(k, torch.tensor([j]), fr, m)).sum())
    assert math.isclose(score(17, 5), score(112, 100), rel_tol=1e-9) and not math.isclose(score(17, 5), score(17, 6), rel_tol=1e-3)
    tail = float((q[..., 6:] * k[..., 6:]).sum())
    assert math.isclose(score(17, 5) - tail, mag ** 2 * (score(17, 5, 1.0) - tail), rel_tol=1e-9)


def test_oracle_sink_and_weights_in_closed_form():
    s = torch.tensor([[0.3, -0.2, float("-inf")]], dtype=torch.float64)
    sink = torch.tensor(0.7, dtype=torch.float64)
    den = math.exp(0.7) + math.exp(0.3) + math.exp(-0.2)
    assert torch.allclose(GR.sink_softmax(s, sink), torch.tensor([[math.exp(0.3) / den, math.exp(-0.2) / den, 0.0]], dtype=torch.float64))
    # sigmoid attention with silent scores: every visible key weighs sigmoid(bias + offset), nothing is normalised
    cfg = P.config([P.attention(heads=1, kv_heads=1, dim=4, vdim=4, size=6, bias_max=6, rows=4)], width=8)
    S = {k: v.double() for k, v in P.random_checkpoint(cfg, seed=11).items()}
    Q = GR.sub(S, "l0.mix.")
    Q["temp"] = torch.zeros(1, dtype=torch.float64)
    n = torch.randn(5, 8, dtype=torch.float64)
    v = n @ Q["v"].T
    want = torch.zeros(5, 4, dtype=torch.float64)
    for i in range(5):
        for j in range(i + 1):
            want[i] += torch.sigmoid(Q["rel"][GR.distance_bucket(i - j, 4, 6), 0] + Q["pb"][0]) * v[j]
    want = (want * torch.sigmoid(n @ Q["g"].T)) @ Q["o"].T
    assert torch.allclose(GR.attention_mixer(Q, n, cfg["layers"][0]["mixer"], 1e-5), want)


def test_oracle_routing_groups():
    z = torch.log(torch.tensor([[0.30, 0.01, 0.20, 0.19, 0.02, 0.28]], dtype=torch.float64))
    Q = {"router": torch.eye(6, dtype=torch.float64)}
    pick = lambda **r: [(j, round(float(w), 6)) for j, w in GR.route(Q, z, dict({"experts": 6, "top": 2, "scale": 2.0}, **r))[0]]
    assert pick() == [(0, 0.6), (5, 0.56)]
    assert pick(groups={"count": 3, "keep": 1}) == [(0, 0.6), (1, 0.02)]
    assert pick(groups={"count": 3, "keep": 2}, top=3) == [(0, 0.6), (5, 0.56), (4, 0.04)]
    assert pick(groups={"count": 2, "keep": 1}, top=3) == [(0, 0.6), (2, 0.4), (1, 0.02)]
