"""Float64 restatement of the Gaparax design, one function per mechanism, for the tests.  It shares no code with the engine: plain
loops over tokens and heads on the CPU, no cache, a whole sequence at a time.

Notation: n = a normed row, W_x = tensor `<prefix>x` ([out, in], applied as W n), T tokens, H heads, G key heads, d key dims, e value
dims, R the width of the cached latent, r the rotated dims.  Checkpoint layout: see vox_serve_amd/model/gaparax.py.
"""
import math

import torch


def silu(z):
    return z * torch.sigmoid(z)


def relu_squared(z):
    return torch.clamp(z, min=0.0) ** 2


def rms_norm(x, w, eps):
    return x / torch.sqrt(x.pow(2).mean(-1, keepdim=True) + eps) * w


def sub(P, prefix):
    return {k[len(prefix):]: v for k, v in P.items() if k.startswith(prefix)}


# ---- the residual stream: several copies, mixed at every sublayer ----------------------------------------------------------------

def read_streams(xs, w_in):
    """What a sublayer sees of the streams: sum_s w_in[s] x_s."""
    u = torch.zeros_like(xs[0])
    for s, x in enumerate(xs):
        u = u + w_in[s] * x
    return u


def write_streams(xs, mix, w_out, y):
    """x_t <- sum_s mix[s][t] x_s + w_out[t] y, every new stream from the old ones."""
    return [sum(mix[s, t] * xs[s] for s in range(len(xs))) + w_out[t] * y for t in range(len(xs))]


def residual_gate(P, q, n):
    return torch.sigmoid(n @ P[f"rg{q}"].T + P[f"rg{q}.b"])


# ---- attention with independent key weights ----------------------------------------------------------------------------------------

def distance_bucket(n, rows, far):
    """Row of the bias table for a key n tokens back: exact below rows/2, logarithmic up to `far`, the last row beyond."""
    half = rows // 2
    if n < half:
        return n
    return min(rows - 1, half + math.floor(math.log(n / half) / math.log(far / half) * (rows - half)))


def chunk_mask(T, size):
    """visible[i][j]: j <= i and both in the same chunk of `size` tokens counted from the sequence's start."""
    i = torch.arange(T)
    return (i.view(-1, 1) >= i.view(1, -1)) & ((i // size).view(-1, 1) == (i // size).view(1, -1))


def softcap(s, cap):
    return cap * torch.tanh(s / cap)


def attention_mixer(P, n, m, eps):
    H, G, d, e = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    T = n.shape[0]
    q = rms_norm((n @ P["q"].T).view(T, H, d), P["q.norm"], eps)
    k = rms_norm((n @ P["k"].T).view(T, G, d), P["k.norm"], eps)
    v = (n @ P["v"].T).view(T, G, e)
    visible = chunk_mask(T, m["mask"]["size"])
    rows = P["rel"].shape[0]
    dist = (torch.arange(T).view(-1, 1) - torch.arange(T).view(1, -1)).clamp(min=0)
    bucket = torch.tensor([distance_bucket(x, rows, m["bias_max"]) for x in range(T)])[dist]
    out = torch.zeros(T, H, e, dtype=n.dtype)
    for h in range(H):
        g = h // (H // G)
        s = (q[:, h] @ k[:, g].T) * m["scale"] * P["temp"][h]
        s = softcap(s, m["softcap"]) + P["rel"][:, h][bucket]
        w = torch.where(visible, torch.sigmoid(s + P["pb"][h]), torch.zeros_like(s))
        out[:, h] = w @ v[:, g]
    return (out.reshape(T, H * e) * torch.sigmoid(n @ P["g"].T)) @ P["o"].T


# ---- latent attention with a sink ---------------------------------------------------------------------------------------------------

def yarn_frequencies(dims, base, sc):
    """-> (one frequency per pair, the factor of cos and sin)."""
    f = [base ** (-2.0 * i / dims) for i in range(dims // 2)]
    if not sc:
        return f, 1.0

    def dim_of(turns):
        return dims * math.log(sc["original"] / (2.0 * math.pi * turns)) / (2.0 * math.log(base))
    lo, hi = max(math.floor(dim_of(sc["fast"])), 0), min(math.ceil(dim_of(sc["slow"])), dims - 1)
    out = []
    for i, fi in enumerate(f):
        ramp = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        out.append(fi / sc["factor"] * ramp + fi * (1.0 - ramp))
    return out, 0.1 * math.log(sc["factor"]) + 1.0


def rotate_halves(x, positions, freqs, mag):
    """x [T, heads, r]: dims i and i + len(freqs) turn together by position * freqs[i], the pair scaled by mag; later dims pass."""
    half = len(freqs)
    y = x.clone()
    for i, f in enumerate(freqs):
        a = positions.to(x.dtype) * f
        c, s = (torch.cos(a) * mag).unsqueeze(1), (torch.sin(a) * mag).unsqueeze(1)
        u, v = x[..., i], x[..., i + half]
        y[..., i] = u * c - v * s
        y[..., i + half] = v * c + u * s
    return y


def sink_softmax(scores, sink):
    """exp(s_j) / (exp(sink) + sum_j exp(s_j)) over the last axis (-inf entries are masked keys)."""
    m = torch.clamp(scores.max(-1, keepdim=True).values, min=float(sink))
    w = torch.exp(scores - m)
    return w / (torch.exp(sink - m) + w.sum(-1, keepdim=True))


def latent_mixer(P, n, m, eps):
    H, d, r, e, R = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    T = n.shape[0]
    q = (n @ P["q"].T).view(T, H, d + r)
    ckr = n @ P["dkv"].T
    c = rms_norm(ckr[:, :R], P["dkv.norm"], eps)
    rot = m.get("rot") or {}
    freqs, mag = yarn_frequencies(rot["dims"], rot["base"], rot.get("scaling")) if rot.get("dims") else ([], 1.0)
    pos = torch.arange(T)
    qr = rotate_halves(q[..., d:], pos, freqs, mag)
    kr = rotate_halves(ckr[:, R:].unsqueeze(1), pos, freqs, mag)[:, 0]
    k = (c @ P["uk"].T).view(T, H, d)
    v = (c @ P["uv"].T).view(T, H, e)
    causal = torch.ones(T, T, dtype=torch.bool).tril()
    out = torch.zeros(T, H, e, dtype=n.dtype)
    for h in range(H):
        s = (q[:, h, :d] @ k[:, h].T + qr[:, h] @ kr.T) * m["scale"]
        out[:, h] = sink_softmax(s.masked_fill(~causal, float("-inf")), P["sink"][h]) @ v[:, h]
    return out.reshape(T, H * e) @ P["o"].T


# ---- feed-forwards --------------------------------------------------------------------------------------------------------------------

def dense_ff(P, n):
    return relu_squared(n @ P["up"].T) @ P["down"].T


def expert_unit(P, n):
    return (silu(n @ P["gate"].T) * (n @ P["up"].T)) @ P["down"].T


def route(P, n, router):
    """-> per token a list of (expert, weight): softmax scores; the groups with the largest best score stay; the largest scores inside
    them are chosen; weights are their scores times a constant."""
    s = torch.softmax(n @ P["router"].T, -1)
    gr = router.get("groups") or {"count": 1, "keep": 1}
    per = router["experts"] // gr["count"]
    picks = []
    for t in range(n.shape[0]):
        row = s[t].tolist()
        best = [max(row[g * per:(g + 1) * per]) for g in range(gr["count"])]
        kept = sorted(range(gr["count"]), key=lambda g: -best[g])[: gr["keep"]]
        pool = [j for j in range(router["experts"]) if j // per in kept]
        chosen = sorted(pool, key=lambda j: -row[j])[: router["top"]]
        picks.append([(j, s[t, j] * router.get("scale", 1.0)) for j in chosen])
    return picks


def moe_ff(P, n, mlp):
    out = torch.zeros_like(n)
    for t, chosen in enumerate(route(P, n, mlp["router"])):
        for j, w in chosen:
            out[t] += w * expert_unit(sub(P, f"e{j}."), n[t:t + 1])[0]
    return out


def forward(cfg, S, tokens, trace=None):
    """-> logits [T, vocab] (float64) of one whole sequence.  trace: a list that receives the sum of the streams after every layer."""
    S = {k: v.double() for k, v in S.items()}
    eps = cfg["norm"]["eps"]
    e = S["embed"][torch.as_tensor(tokens, dtype=torch.long)]
    xs = [e.clone() for _ in range(cfg["streams"])]
    for i, L in enumerate(cfg["layers"]):
        P = sub(S, f"l{i}.")
        for q in (1, 2):
            if q == 2 and not L.get("mlp"):
                break
            n = rms_norm(read_streams(xs, P[f"hc{q}.in"]), P[f"norm{q}"], eps)
            if q == 1:
                y = (attention_mixer if L["type"] == "attention" else latent_mixer)(sub(P, "mix."), n, L["mixer"], eps)
            else:
                y = dense_ff(sub(P, "mlp."), n) if L["mlp"]["kind"] == "dense" else moe_ff(sub(P, "mlp."), n, L["mlp"])
            xs = write_streams(xs, P[f"hc{q}.mix"], P[f"hc{q}.out"], y * residual_gate(P, q, n))
        if trace is not None:
            trace.append(sum(xs))
    return rms_norm(sum(xs), S["final.norm"], eps) @ S["head"].T
