"""Host-side pieces of the Kazozen path that need no GPU: the config reader, the fused weight layout, the registry entry, and identities and
sensitivities of the oracle itself (causality, windows and kept tokens, shared keys, the sink, the routing groups, the bigram rows)."""
import copy
import math

import pytest
import torch

from oracle import kazozen_ref as KR
from tests import kazozen_util as P

F32_BAR = 2e-4


def rel_err(got, want):
    d = got - want
    d = d - d.mean(-1, keepdim=True)
    w = want - want.mean(-1, keepdim=True)
    return float((d.pow(2).mean(-1).sqrt() / w.pow(2).mean().sqrt()).max())


def tokens(n, vocab, seed):
    return torch.randint(0, vocab, (n,), generator=torch.Generator().manual_seed(seed)).tolist()


def small():
    return P.config([P.attention(heads=6, kv_heads=3, dim=8, vdim=10, size=7, keep=2, scale=0.3, mlp=P.dense(14, 0.9)),
                     P.attention(heads=6, kv_heads=3, dim=8, vdim=10, size=9, keep=0, scale=0.4, kv_from=0, mlp=P.moe()),
                     P.attention(heads=2, kv_heads=2, rot=6, scaling=None, mlp=None)])


def test_config_reader_takes_every_size_and_constant():
    from vox_serve_amd.model.kazozen import config_from_dict
    c = config_from_dict(small())
    assert (c.width, c.vocab, c.eps, c.norm_kind, c.norm_one_plus, c.streams, c.loop, c.embed_scale, c.logit_softcap, c.logit_scale, c.bigram) == \
        (24, 40, 1e-5, "layer", False, 0, None, 3.0, 9.0, 1.0, (31, 7, 5))
    a, b, d = c.layers
    assert (a.kind, a.heads, a.kv_heads, a.dim, a.vdim, a.window, a.keep_first, a.scale, a.out_gate, a.qk_norm_whole, a.block, a.kv_from) == \
        ("window_attention", 6, 3, 8, 10, 7, 2, 0.3, True, True, "post_norm", None)
    assert (a.rot_dims, a.rot_base, a.rot_yarn) == (8, 300.0, (4.0, 24.0, 4.0, 0.5)) and (d.rot_dims, d.rot_yarn) == (6, None)
    assert (a.ff, a.ff_kind, a.ff_act, a.ff_limit, a.ff_alpha, a.ff_up_offset, a.moe) == (14, "gated", "swish", 0.9, 1.702, 1.0, None)
    assert (b.kv_from, b.window, b.keep_first, b.scale, b.ff) == (0, 9, 0, 0.4, 0)
    e = b.moe
    assert (e.experts, e.identity, e.top, e.ff, e.shared_ff, e.groups, e.keep, e.group_best_two, e.weight_scale) == (6, 0, 2, 12, 0, 2, 1, True, 1.0)
    assert (e.score, e.renorm, e.scale_input, e.limit, e.act_alpha, e.up_offset, e.expert_form) == ("sigmoid", False, False, 0.8, 1.702, 1.0, "gated")
    assert (d.ff, d.moe) == (0, None)
    assert a.n_in == 48 + 24 + 30 + 60 and a.cache_values() == 3 * 18 and a.state_floats(24) == 0
    assert b.n_in == 48 + 60 and b.cache_values() == 0
    plain = small()
    del plain["layers"][1]["mlp"]["router"]["groups"], plain["embedding"]["bigram"], plain["logit_softcap"]
    c = config_from_dict(plain)
    assert (c.layers[1].moe.groups, c.layers[1].moe.keep, c.bigram, c.logit_softcap) == (1, 1, None, 0.0)


@pytest.mark.parametrize("break_it", [
    lambda c: c.update(architecture="Other"),
    lambda c: c["layers"][0].update(type="other"),
    lambda c: c["layers"][0]["mlp"].update(kind="other"),
    lambda c: c["layers"][0]["mixer"].update(kv_heads=4),
    lambda c: c["layers"][0]["mixer"]["rot"].update(dims=10),
    lambda c: c["layers"][0]["mixer"]["rot"].update(dims=3),
    lambda c: c["layers"][1]["mixer"].update(kv_from=1),
    lambda c: c["layers"][1]["mixer"].update(kv_from=2),
    lambda c: c["layers"][1]["mixer"].update(vdim=9),
    lambda c: c["layers"][2]["mixer"].update(kv_from=1),
    lambda c: c["layers"][1]["mlp"]["router"]["groups"].update(count=4),
    lambda c: c["layers"][1]["mlp"]["router"]["groups"].update(keep=3),
    lambda c: c["layers"][1]["mlp"]["router"].update(top=4),
])
def test_config_reader_refuses(break_it):
    from vox_serve_amd.model.kazozen import config_from_dict
    bad = copy.deepcopy(small())
    break_it(bad)
    with pytest.raises(ValueError):
        config_from_dict(bad)


def test_pack_weights_layout():
    from vox_serve_amd.model.kazozen import config_from_dict, pack_weights
    cfg = small()
    S = P.random_checkpoint(cfg, seed=3)
    w = pack_weights(S, config_from_dict(cfg))
    a, b, d = w["layers"]
    assert tuple(a["w_in"].shape) == (162, 24) and torch.equal(a["w_in"][48:72], S["l0.mix.k"]) and torch.equal(a["w_in"][72:102], S["l0.mix.v"])
    assert torch.equal(a["w_in"][102:], S["l0.mix.g"]) and torch.equal(a["b_in"][48:72], S["l0.mix.k.b"].float()) and not a["b_in"][102:].any()
    assert tuple(b["w_in"].shape) == (108, 24) and torch.equal(b["w_in"][48:], S["l1.mix.g"]) and torch.equal(b["b_in"][:48], S["l1.mix.q.b"].float())
    assert b["k_norm"] is None and a["k_norm"] is S["l0.mix.k.norm"] and b["sinks"] is S["l1.mix.sink"]
    assert a["norm1_b"] is S["l0.norm1.b"] and a["norm2_b"] is S["l0.norm2.b"] and d["norm2"] is None and d["norm2_b"] is None
    assert torch.equal(a["w_up"][:14], S["l0.mlp.gate"]) and torch.equal(a["w_up"][14:], S["l0.mlp.up"]) and a["w_down"] is S["l0.mlp.down"]
    assert tuple(b["moe"]["w_gate_up"].shape) == (6, 24, 24) and torch.equal(b["moe"]["w_gate_up"][2][12:], S["l1.mlp.e2.up"])
    assert tuple(b["moe"]["w_down"].shape) == (6, 24, 12) and b["moe"]["router"] is S["l1.mlp.router"] and b["moe"]["correction"] is S["l1.mlp.correction"]
    assert w["head"] is w["embedding"] is S["embed"] and w["bigram"] is S["bigram"] and w["final_norm_b"] is S["final.norm.b"]


def test_synthetic_weights_fit_the_reader():
    from vox_serve_amd.model.kazozen import config_from_dict, pack_weights, synth_weights
    c = config_from_dict(small())
    S = synth_weights(c)
    R = P.random_checkpoint(small())
    assert set(S) == set(R) and all(tuple(S[k].shape) == tuple(R[k].shape) for k in S)
    assert len(pack_weights(S, c)["layers"]) == 3


def test_registry_names_the_design():
    from vox_serve_amd.model import MODEL_REGISTRY, get_model_class
    assert "kazozen" in MODEL_REGISTRY and get_model_class("Kazozen") is MODEL_REGISTRY["kazozen"]


def test_bigram_rows_of_the_oracle_and_of_the_engines_reduced_hash():
    from vox_serve_amd.engine_hybrid import reduced_bigram
    toks = tokens(50, 1000, 4)
    bg = {"buckets": 97, "mul_prev": 1234567, "mul_cur": 98765}
    rows = KR.pair_rows(toks, bg)
    n, a, b = reduced_bigram((bg["buckets"], bg["mul_prev"], bg["mul_cur"]))
    assert rows[0] == 97 and rows[1:] == [(p * a + t * b) % n for p, t in zip(toks, toks[1:])]


def test_visibility_of_the_oracle():
    v = KR.visible(9, 3, 2)
    assert [j for j in range(9) if v[7, j]] == [0, 1, 5, 6, 7] and [j for j in range(9) if v[3, j]] == [0, 1, 2, 3] and [j for j in range(9) if v[0, j]] == [0]
    assert torch.equal(KR.visible(9, 9, 0), torch.ones(9, 9, dtype=torch.bool).tril()) and torch.equal(KR.visible(9, 1, 0), torch.eye(9, dtype=torch.bool))
    assert torch.equal(KR.visible(9, 1, 9), torch.ones(9, 9, dtype=torch.bool).tril())


def test_oracle_is_causal_and_windows_end():
    cfg = small()
    S = P.random_checkpoint(cfg, seed=5)
    toks = tokens(30, 40, 6)
    full = KR.forward(cfg, S, toks)
    assert torch.allclose(KR.forward(cfg, S, toks[:17]), full[:17], atol=1e-12)
    other = list(toks)
    other[20] = (other[20] + 1) % 40
    assert torch.allclose(KR.forward(cfg, S, other)[:20], full[:20], atol=1e-12)
    assert not torch.allclose(KR.forward(cfg, S, other)[20:], full[20:], atol=1e-6)
    # one attention layer without pairs: a token moves the positions that see it and no others; a kept one moves all that follow
    solo = P.config([P.attention(size=6, keep=2)], bigram=None)
    S = P.random_checkpoint(solo, seed=6)
    full = KR.forward(solo, S, toks)
    for at, last in ((12, 17), (2, 7), (1, 29)):
        other = list(toks)
        other[at] = (other[at] + 1) % 40
        moved = (KR.forward(solo, S, other) - full).abs().amax(-1) > 1e-9
        assert moved[at:last + 1].all() and not moved[:at].any() and not moved[last + 1:].any()


def test_oracle_shared_keys():
    """A layer on another one's keys and values = the same layer with that layer's cache handed over; its own norms and projections of keys do
    not exist."""
    cfg = P.config([P.attention(), P.attention(kv_from=0, size=4)])
    S = P.random_checkpoint(cfg, seed=7)
    assert not any(k.startswith("l1.mix.k") or k.startswith("l1.mix.v") for k in S)
    Sd = {k: v.double() for k, v in S.items()}
    toks = tokens(20, 40, 8)
    tr = []
    KR.forward(cfg, S, toks, tr)
    x, eps = KR.embed(cfg, Sd, toks), cfg["norm"]["eps"]
    kv = KR.keys_values(KR.sub(Sd, "l0.mix."), x, cfg["layers"][0]["mixer"], eps)
    for i in (0, 1):
        Q = KR.sub(Sd, f"l{i}.")
        x = x + KR.layer_norm(KR.attention_mixer(KR.sub(Q, "mix."), x, cfg["layers"][i]["mixer"], eps, kv), Q["norm1"], Q["norm1.b"], eps)
        assert torch.allclose(x, tr[i], atol=1e-12)


def test_oracle_tells_the_mechanisms_apart():
    """A mechanism left out or one off moves the logits by far more than the bar."""
    cfg = P.config([P.attention(heads=3, kv_heads=1, size=13, keep=3, mlp=P.moe()), P.attention(heads=3, kv_heads=1, size=13, keep=3, kv_from=0, mlp=P.dense(20, 0.6))])
    S = P.random_checkpoint(cfg, seed=9, gain=2.0)
    toks = tokens(60, 40, 10)
    want = KR.forward(cfg, S, toks)

    def moved(**names):
        orig = {k: getattr(KR, k) for k in names}
        try:
            for k, f in names.items():
                setattr(KR, k, f(orig[k]))
            return rel_err(KR.forward(cfg, S, toks), want)
        finally:
            for k, f in orig.items():
                setattr(KR, k, f)
    bar = 50 * F32_BAR
    assert moved(visible=lambda f: lambda T, size, keep: f(T, size + 1, keep)) > bar
    assert moved(visible=lambda f: lambda T, size, keep: f(T, size, keep + 1)) > bar
    assert moved(visible=lambda f: lambda T, size, keep: f(T, size, 0)) > bar
    assert moved(visible=lambda f: lambda T, size, keep: f(T, 10 ** 6, keep)) > bar
    assert moved(softcap=lambda f: lambda z, cap: z) > bar
    assert moved(sink_softmax=lambda f: lambda s, sink: torch.softmax(s, -1)) > bar
    assert moved(rotate_pairs=lambda f: lambda x, pos, fr, mag: f(x, pos, fr, 1.0)) > bar
    assert moved(rotate_pairs=lambda f: lambda x, pos, fr, mag: f(x, pos + pos // 9, fr, mag)) > bar
    assert moved(layer_norm=lambda f: lambda x, w, b, eps: f(x, w, torch.zeros_like(b), eps)) > bar
    assert moved(layer_norm=lambda f: lambda x, w, b, eps: KR.rms_norm(x, w, eps) + b) > bar
    assert moved(pair_rows=lambda f: lambda t, bg: f(t, dict(bg, mul_prev=bg["mul_cur"], mul_cur=bg["mul_prev"]))) > bar
    assert moved(clamped_unit=lambda f: lambda Q, x, limit: f(Q, x, 1e9)) > bar
    assert moved(route=lambda f: lambda Q, x, r: f(Q, x, dict(r, groups={"count": 1, "keep": 1}))) > bar
    assert moved(route=lambda f: lambda Q, x, r: f(dict(Q, correction=torch.zeros_like(Q["correction"])), x, r)) > bar
    for name in ("l0.mix.q.b", "l0.mix.v.b", "l0.mix.g", "l1.mix.q.norm"):
        assert rel_err(KR.forward(cfg, dict(S, **{name: torch.zeros_like(S[name]) + (1 if "norm" in name else 0)}), toks), want) > bar, name
    # (a key bias shared by all keys cancels in a softmax without rotation; with it, and with the norm, it shows)
    assert rel_err(KR.forward(cfg, dict(S, **{"l0.mix.k.b": torch.zeros_like(S["l0.mix.k.b"])}), toks), want) > bar


def test_oracle_rotation_depends_on_distance():
    """Rotated queries against rotated keys depend on how far apart they are, not on where they stand; the pairs' scale enters squared."""
    fr, mag = KR.frequencies(6, 300.0, {"factor": 4.0, "original": 24, "fast": 4.0, "slow": 0.5})
    g = torch.Generator().manual_seed(3)
    q, k = torch.randn(1, 1, 8, dtype=torch.float64, generator=g), torch.randn(1, 1, 8, dtype=torch.float64, generator=g)

    def score(i, j, m=mag):
        return float((KR.rotate_pairs(q, torch.tensor([i]), fr, m) * KR.rotate_pairs(k, torch.tensor([j]), fr, m)).sum())
    assert math.isclose(score(17, 5), score(112, 100), rel_tol=1e-9) and not math.isclose(score(17, 5), score(17, 6), rel_tol=1e-3)
    tail = float((q[..., 6:] * k[..., 6:]).sum())
    assert math.isclose(score(17, 5) - tail, mag ** 2 * (score(17, 5, 1.0) - tail), rel_tol=1e-9)


def test_oracle_sink_and_unit_in_closed_form():
    s = torch.tensor([[0.3, -0.2, float("-inf")]], dtype=torch.float64)
    sink = torch.tensor(0.7, dtype=torch.float64)
    den = math.exp(0.7) + math.exp(0.3) + math.exp(-0.2)
    assert torch.allclose(KR.sink_softmax(s, sink), torch.tensor([[math.exp(0.3) / den, math.exp(-0.2) / den, 0.0]], dtype=torch.float64))
    one = torch.ones(1, 1, dtype=torch.float64)
    for gate, up, want in ((0.5, 0.25, 0.5 / (1 + math.exp(-0.851)) * 1.25), (3.0, -3.0, 0.8 / (1 + math.exp(-1.702 * 0.8)) * 0.2),
                           (-3.0, 3.0, -3.0 / (1 + math.exp(1.702 * 3.0)) * 1.8)):
        assert math.isclose(float(KR.clamped_unit({"gate": one * gate, "up": one * up, "down": one}, one, 0.8)), want, rel_tol=1e-12)


def test_oracle_routing_groups():
    p = torch.tensor([[0.30, 0.05, 0.22, 0.21, 0.06, 0.38]], dtype=torch.float64)
    Q = {"router": torch.eye(6, dtype=torch.float64), "correction": torch.zeros(6, dtype=torch.float64)}
    z = torch.log(p / (1 - p))
    pick = lambda **r: [(j, round(float(w), 6)) for j, w in KR.route(Q, z, dict({"experts": 6, "top": 2}, **r))[0]]
    assert pick() == [(5, 0.38), (0, 0.3)]
    # pairs (.35, .43, .44): the best single score is in the last group too, but the middle one beats the first
    assert pick(groups={"count": 3, "keep": 1}) == [(5, 0.38), (4, 0.06)]
    assert pick(groups={"count": 3, "keep": 2}, top=3) == [(5, 0.38), (2, 0.22), (3, 0.21)]
    # triples: two best .52 against .59
    assert pick(groups={"count": 2, "keep": 1}, top=3) == [(5, 0.38), (3, 0.21), (4, 0.06)]
    Q["correction"] = torch.tensor([-2.0, -2.0, -2.0, -3.0, -3.0, -3.0], dtype=torch.float64)
    assert pick(groups={"count": 2, "keep": 1}, top=2) == [(0, 0.3), (2, 0.22)]
