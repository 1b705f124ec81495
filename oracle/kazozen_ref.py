"""Float64 restatement of the Kazozen design, one function per mechanism, for the tests.  It shares no code with the engine: plain
loops over tokens and heads on the CPU, no cache, a whole sequence at a time.

Notation: x = rows of the residual stream (every sublayer reads them as they are), W_a = tensor `<prefix>a` ([out, in], applied as W x),
T tokens, H query heads, G key heads, d key dims, e value dims.  Checkpoint layout: see vox_serve_amd/model/kazozen.py.
"""
import math

import torch

SLOPE = 1.702           # of the sigmoid inside the gated units


def rms_norm(x, w, eps):
    return x / torch.sqrt(x.pow(2).mean(-1, keepdim=True) + eps) * w


def layer_norm(x, w, b, eps):
    c = x - x.mean(-1, keepdim=True)
    return c / torch.sqrt(c.pow(2).mean(-1, keepdim=True) + eps) * w + b


def sub(P, prefix):
    return {k[len(prefix):]: v for k, v in P.items() if k.startswith(prefix)}


# ---- the embedding of a token and of the pair it forms with its predecessor -----------------------------------------------------------

def pair_rows(tokens, bigram):
    """Row of the pair table per token; the last row for a token without a predecessor."""
    n, a, b = bigram["buckets"], bigram["mul_prev"], bigram["mul_cur"]
    return [n if i == 0 else (int(tokens[i - 1]) * a + int(t) * b) % n for i, t in enumerate(tokens)]


def embed(cfg, S, tokens):
    emb = cfg["embedding"]
    x = S["embed"][torch.as_tensor(tokens, dtype=torch.long)] * emb["scale"]
    if emb.get("bigram"):
        x = x + S["bigram"][torch.tensor(pair_rows(tokens, emb["bigram"]))]
    return x


# ---- attention over a window and the first tokens ------------------------------------------------------------------------------------------

def visible(T, size, keep_first):
    """seen[i][j]: j <= i, and j among the last `size` tokens up to i or among the first `keep_first` of the sequence."""
    i, j = torch.arange(T).view(-1, 1), torch.arange(T).view(1, -1)
    return (j <= i) & ((i - j < size) | (j < keep_first))


def frequencies(dims, base, sc):
    """-> (one frequency per pair, the factor of cos and sin).  sc: scaling with factor, original, fast, slow, or nothing."""
    f = [base ** (-2.0 * i / dims) for i in range(dims // 2)]
    if not sc:
        return f, 1.0

    def place(turns):
        return dims * math.log(sc["original"] / (2.0 * math.pi * turns)) / (2.0 * math.log(base))
    lo, hi = max(math.floor(place(sc["fast"])), 0), min(math.ceil(place(sc["slow"])), dims - 1)
    out = []
    for i, fi in enumerate(f):
        t = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        out.append(fi / sc["factor"] * t + fi * (1.0 - t))
    return out, 0.1 * math.log(sc["factor"]) + 1.0


def rotate_pairs(x, positions, freqs, mag):
    """x [T, heads, d]: dims 2i and 2i + 1 turn together by position * freqs[i], the pair scaled by mag; later dims pass."""
    y = x.clone()
    for i, f in enumerate(freqs):
        a = positions.to(x.dtype) * f
        c, s = (torch.cos(a) * mag).unsqueeze(1), (torch.sin(a) * mag).unsqueeze(1)
        u, v = x[..., 2 * i], x[..., 2 * i + 1]
        y[..., 2 * i] = u * c - v * s
        y[..., 2 * i + 1] = v * c + u * s
    return y


def sink_softmax(scores, sink):
    """exp(s_j) / (exp(sink) + sum_j exp(s_j)) over the last axis (-inf entries are masked keys)."""
    m = torch.clamp(scores.max(-1, keepdim=True).values, min=float(sink))
    w = torch.exp(scores - m)
    return w / (torch.exp(sink - m) + w.sum(-1, keepdim=True))


def turned(P, x, name, heads, m, eps):
    """Queries or keys: projection with its bias, one norm over all heads at once, rotation."""
    y = rms_norm(x @ P[name].T + P[name + ".b"], P[name + ".norm"], eps).view(x.shape[0], heads, m["dim"])
    rot = m.get("rot") or {}
    freqs, mag = frequencies(rot["dims"], rot["base"], rot.get("scaling")) if rot.get("dims") else ([], 1.0)
    return rotate_pairs(y, torch.arange(x.shape[0]), freqs, mag)


def keys_values(P, x, m, eps):
    return turned(P, x, "k", m["kv_heads"], m, eps), (x @ P["v"].T + P["v.b"]).view(x.shape[0], m["kv_heads"], m["vdim"])


def attention_mixer(P, x, m, eps, kv):
    H, G, T = m["heads"], m["kv_heads"], x.shape[0]
    q, (k, v) = turned(P, x, "q", H, m, eps), kv
    seen = visible(T, m["mask"]["size"], m["mask"]["keep_first"])
    out = torch.zeros(T, H, v.shape[-1], dtype=x.dtype)
    for h in range(H):
        g = h // (H // G)
        s = (q[:, h] @ k[:, g].T) * m["scale"]
        out[:, h] = sink_softmax(s.masked_fill(~seen, float("-inf")), P["sink"][h]) @ v[:, g]
    return (out.reshape(T, -1) * torch.sigmoid(x @ P["g"].T)) @ P["o"].T


# ---- feed-forwards --------------------------------------------------------------------------------------------------------------------

def clamped_unit(P, x, limit):
    g = torch.clamp(x @ P["gate"].T, max=limit)
    u = torch.clamp(x @ P["up"].T, min=-limit, max=limit)
    return (g * torch.sigmoid(SLOPE * g) * (u + 1.0)) @ P["down"].T


def route(P, x, router):
    """-> per token a list of (expert, weight).  Choices by score + correction: the groups with the largest sum of their two best stay, the
    best choices inside them are taken; a weight is the plain score."""
    s = torch.sigmoid(x @ P["router"].T)
    c = s + P["correction"]
    gr = router.get("groups") or {"count": 1, "keep": 1}
    per = router["experts"] // gr["count"]
    picks = []
    for t in range(x.shape[0]):
        row = c[t].tolist()
        rank = [sum(sorted(row[g * per:(g + 1) * per])[-2:]) for g in range(gr["count"])]
        kept = sorted(range(gr["count"]), key=lambda g: -rank[g])[: gr["keep"]]
        pool = [j for j in range(router["experts"]) if j // per in kept]
        picks.append([(j, s[t, j]) for j in sorted(pool, key=lambda j: -row[j])[: router["top"]]])
    return picks


def moe_ff(P, x, mlp):
    out = torch.zeros_like(x)
    for t, chosen in enumerate(route(P, x, mlp["router"])):
        for j, w in chosen:
            out[t] += w * clamped_unit(sub(P, f"e{j}."), x[t:t + 1], mlp["expert"]["limit"])[0]
    return out


def softcap(z, cap):
    return cap * torch.tanh(z / cap) if cap else z


def forward(cfg, S, tokens, trace=None):
    """-> logits [T, vocab] (float64) of one whole sequence.  trace: a list that receives the residual stream after every layer."""
    S = {k: v.double() for k, v in S.items()}
    eps = cfg["norm"]["eps"]
    x = embed(cfg, S, tokens)
    made = {}
    for i, L in enumerate(cfg["layers"]):
        P, m, mlp = sub(S, f"l{i}."), L["mixer"], L.get("mlp")
        if m.get("kv_from") is None:
            made[i] = keys_values(sub(P, "mix."), x, m, eps)
        y = attention_mixer(sub(P, "mix."), x, m, eps, made[i if m.get("kv_from") is None else m["kv_from"]])
        x = x + layer_norm(y, P["norm1"], P["norm1.b"], eps)
        if mlp:
            y = clamped_unit(sub(P, "mlp."), x, mlp["limit"]) if mlp["kind"] == "dense" else moe_ff(sub(P, "mlp."), x, mlp)
            x = x + layer_norm(y, P["norm2"], P["norm2.b"], eps)
        if trace is not None:
            trace.append(x)
    return softcap(layer_norm(x, S["final.norm"], S["final.norm.b"], eps) @ S["embed"].T, cfg.get("logit_softcap"))
