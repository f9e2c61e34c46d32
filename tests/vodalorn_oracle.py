"""A plain, slow float64 implementation of the Vodalorn decoder, written from its
equations: one function per mechanism, whole sequences at once, no cache, no
batching, no code shared with ``loqa_hub_amd``. The tests compare the framework
(reference ops on the CPU, HIP kernels on the GPU) with it.

Notation: T tokens, width d, H heads, G key/value heads, head sizes D (queries,
keys) and Dv (values); positions p = 0 .. T - 1.
"""
import math

import torch

F64 = torch.float64


# ----------------------------------------------------------------- configs
def window(heads=4, kv_heads=2, dim=12, vdim=10, size=7, rot_dims=8, base=100.0, scale=None):
    return {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim,
            "scale": scale if scale is not None else dim ** -0.5, "mask": {"size": size},
            "rot": {"dims": rot_dims, "base": base}}


def retention(heads=3, dim=8, vdim=10, rot_dims=6, base=300.0, decay=None):
    return {"heads": heads, "dim": dim, "vdim": vdim, "rot": {"dims": rot_dims, "base": base},
            "decay": list(decay) if decay else [1.0 - 2.0 ** (-2 - h) for h in range(heads)]}


def parallel(left=None, right=None):
    return "parallel", {"left": left or window(), "right": right or retention()}


def delta(heads=4, kv_heads=2, dim=8, vdim=6, conv=4, decay_rank=5, gate_rank=7):
    """The two ranks are read from tensor shapes, not from the config: they sit
    under a key that :func:`make_config` strips."""
    return "channel_delta", {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim,
                             "conv": conv, "_ranks": (decay_rank, gate_rank)}


def dense_ff(ff=40):
    return {"kind": "dense", "ff": ff}


def moe_ff(ff=20, experts=6, top=2, groups=3, keep=2, scale=1.7, limit=1.1):
    r = {"experts": experts, "top": top, "scale": scale}
    if groups:
        r["groups"] = {"count": groups, "keep": keep}
    return {"kind": "moe", "expert": {"ff": ff, "limit": limit}, "router": r}


def make_config(layers, width=32, vocab=50, eps=1e-5, mult=0.6, side=6, bigram=(37, 31, 7),
                loop=None):
    """``bigram`` = (buckets, mul_prev, mul_cur); ``loop`` = (start, stop, times)."""
    out = {"architecture": "Vodalorn", "vocab": vocab, "width": width, "norm": {"eps": eps},
           "residual_mult": mult, "token_side": {"dim": side},
           "embedding": {"bigram": dict(zip(("buckets", "mul_prev", "mul_cur"), bigram))},
           "layers": [{"type": t, "mixer": m, "mlp": f} for (t, m), f in layers]}
    if loop:
        out["loop"] = dict(zip(("start", "stop", "times"), loop))
    return out


def public(cfg):
    """``cfg`` as a config.json holds it (without the tests' own keys)."""
    return dict(cfg, layers=[dict(L, mixer={k: v for k, v in L["mixer"].items() if k[0] != "_"})
                             for L in cfg["layers"]])


def make_weights(cfg, seed=0):
    """Random weights in checkpoint naming whose values are exact in bfloat16."""
    g = torch.Generator().manual_seed(seed)
    d, n = cfg["width"], len(cfg["layers"])
    S = cfg["token_side"]["dim"]
    sd = {}

    def put(name, t):
        sd[name] = t.to(torch.bfloat16).float()

    def mat(name, rows, cols, gain=1.0):
        put(name, torch.randn(rows, cols, generator=g) * gain / cols ** 0.5)

    def vec(name, n, mean=0.0, std=0.1):
        put(name, mean + torch.randn(n, generator=g) * std)

    def norm(name):
        vec(name, d, 1.0, 0.2)
        vec(name + ".b", d, 0.0, 0.2)

    put("embed", torch.randn(cfg["vocab"], d, generator=g))
    put("bigram", torch.randn(cfg["embedding"]["bigram"]["buckets"] + 1, d, generator=g))
    put("side.embed", torch.randn(cfg["vocab"], n * S, generator=g))
    if cfg.get("loop"):
        mat("loop.in", d, 2 * d, 1.4)
        put("loop.step", torch.randn(cfg["loop"]["times"], d, generator=g) * 0.5)
    for i, L in enumerate(cfg["layers"]):
        p, m, f = f"l{i}.", L["mixer"], L["mlp"]
        norm(p + "norm1")
        q = p + "mix."
        if L["type"] == "channel_delta":
            H, G, D, Dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
            Ra, Rg = m["_ranks"]
            for t, c in (("q", G * D), ("k", G * D), ("v", H * Dv)):
                mat(q + t, c, d, 2.0)
                put(q + t + ".conv", torch.randn(c, m["conv"], generator=g) * 0.5)
            mat(q + "b", H, d, 2.0)
            vec(q + "A_log", H, -0.5, 0.7)
            vec(q + "dt_bias", H * D, -0.5, 0.5)
            mat(q + "a1", Ra, d); mat(q + "a2", H * D, Ra, 2.0)
            mat(q + "g1", Rg, d); mat(q + "g2", H * Dv, Rg, 2.0)
            vec(q + "norm", Dv, 1.0, 0.2)
            mat(q + "o", d, H * Dv, 2.0)
        else:
            a, r = m["left"], m["right"]
            H, G, D, Dv = a["heads"], a["kv_heads"], a["dim"], a["vdim"]
            for t, c in (("q", H * D), ("k", G * D), ("v", G * Dv)):
                mat(q + "left." + t, c, d, 2.0)
                vec(q + "left." + t + ".b", c, 0.0, 0.5)
            mat(q + "left.o", d, H * Dv, 2.0)
            vec(q + "left.out", d, 1.0, 0.2)
            H, D, Dv = r["heads"], r["dim"], r["vdim"]
            for t, c in (("q", H * D), ("k", H * D), ("v", H * Dv), ("g", H * Dv)):
                mat(q + "right." + t, c, d, 2.0)
            mat(q + "right.o", d, H * Dv, 2.0)
            vec(q + "right.out", d, 1.0, 0.2)
        if f is not None:
            norm(p + "norm2")
            if f["kind"] == "dense":
                mat(p + "mlp.up", f["ff"], d, 1.5)
                mat(p + "mlp.down", d, f["ff"], 1.5)
            else:
                for e in range(f["router"]["experts"]):
                    ff = f["expert"]["ff"]
                    mat(f"{p}mlp.e{e}.gate", ff, d, 2.0); mat(f"{p}mlp.e{e}.up", ff, d, 2.0)
                    mat(f"{p}mlp.e{e}.down", d, ff, 2.0)
                mat(p + "mlp.router", f["router"]["experts"], d, 3.0)
        mat(p + "side.gate", S, d, 1.5)
        mat(p + "side.proj", d, S)
        vec(p + "side.norm", d, 1.0, 0.2)
    norm("final.norm")
    mat("head", cfg["vocab"], d, 2.0)
    return sd


# -------------------------------------------------------------- mechanisms
def over_rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def layer_norm(x, w, b, eps):
    c = x - x.mean(-1, keepdim=True)
    return c / torch.sqrt((c * c).mean(-1, keepdim=True) + eps) * w + b


def silu(x):
    return x * torch.sigmoid(x)


def gelu_tanh(z):
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def softplus(z):
    return torch.clamp(z, min=0.0) + torch.log1p(torch.exp(-z.abs()))


def bigram_rows(tokens, buckets, mul_prev, mul_cur):
    """The row of the pair table for every token of a sequence: a hash of the
    previous and the current token; the extra last row for the first token."""
    return [buckets if i == 0 else (tokens[i - 1] * mul_prev + t * mul_cur) % buckets
            for i, t in enumerate(tokens)]


def embedding(sd, cfg, tokens):
    b = cfg["embedding"]["bigram"]
    rows = bigram_rows(tokens, b["buckets"], b["mul_prev"], b["mul_cur"])
    return sd["embed"][torch.tensor(tokens)] + sd["bigram"][torch.tensor(rows)]


def rotate_halves(x, dims, base):
    """x [T, heads, size]: of the first ``dims`` entries, i turns with i + dims / 2
    by the angle p * base^(-2 i / dims)."""
    if dims == 0:
        return x
    n = dims // 2
    p = torch.arange(x.shape[0], dtype=F64)
    f = torch.tensor([base ** (-2.0 * i / dims) for i in range(n)], dtype=F64)
    a = p[:, None] * f[None, :]
    c, s = torch.cos(a)[:, None, :], torch.sin(a)[:, None, :]
    u, v = x[..., :n], x[..., n:dims]
    return torch.cat([u * c - v * s, v * c + u * s, x[..., dims:]], -1)


def window_softmax(q, k, v, scale, size):
    """q [T, H, D], k [T, G, D], v [T, G, Dv]; query i sees key j when
    0 <= i - j < size."""
    T, H, _ = q.shape
    G = k.shape[1]
    dist = torch.arange(T)[:, None] - torch.arange(T)[None, :]
    hidden = (dist < 0) | (dist >= size)
    out = torch.zeros(T, H, v.shape[2], dtype=F64)
    for h in range(H):
        g = h // (H // G)
        s = ((q[:, h] @ k[:, g].T) * scale).masked_fill(hidden, -math.inf)
        out[:, h] = torch.softmax(s, -1) @ v[:, g]
    return out


def retention_scan(q, k, v, decay):
    """q, k [T, H, D], v [T, H, Dv]: S <- decay_h S + k v^T, o = S^T q."""
    T, H, D = q.shape
    out = torch.zeros(T, H, v.shape[2], dtype=F64)
    for h in range(H):
        S = torch.zeros(D, v.shape[2], dtype=F64)
        for t in range(T):
            S = decay[h] * S + torch.outer(k[t, h], v[t, h])
            out[t, h] = S.T @ q[t, h]
    return out


def short_conv(x, w):
    """x [T, C], w [C, taps]: per channel, the last tap is the current token's."""
    T, taps = x.shape[0], w.shape[1]
    xp = torch.cat([torch.zeros(taps - 1, x.shape[1], dtype=F64), x])
    return sum(xp[j:j + T] * w[:, j] for j in range(taps))


def unit(x):
    return x / torch.sqrt((x * x).sum(-1, keepdim=True) + 1e-6)


def channel_delta_scan(q, k, v, g, beta):
    """q, k [T, G, D], v [T, H, Dv], g [T, H, D] (a decay per key channel), beta
    [T, H]: S <- diag(g) S; u = beta (v - S^T k); S <- S + k u^T; o = S^T q."""
    T, H, Dv = v.shape
    r = H // q.shape[1]
    out = torch.zeros(T, H, Dv, dtype=F64)
    for h in range(H):
        S = torch.zeros(q.shape[2], Dv, dtype=F64)
        for t in range(T):
            kt = k[t, h // r]
            S = g[t, h][:, None] * S
            u = beta[t, h] * (v[t, h] - S.T @ kt)
            S = S + torch.outer(kt, u)
            out[t, h] = S.T @ q[t, h // r]
    return out


def mixer_window(sd, p, m, h):
    T = h.shape[0]
    H, G, D, Dv, r = m["heads"], m["kv_heads"], m["dim"], m["vdim"], m["rot"]
    q = (h @ sd[p + "q"].T + sd[p + "q.b"]).view(T, H, D)
    k = (h @ sd[p + "k"].T + sd[p + "k.b"]).view(T, G, D)
    v = (h @ sd[p + "v"].T + sd[p + "v.b"]).view(T, G, Dv)
    q, k = rotate_halves(q, r["dims"], r["base"]), rotate_halves(k, r["dims"], r["base"])
    o = window_softmax(q, k, v, m["scale"], m["mask"]["size"])
    return o.reshape(T, H * Dv) @ sd[p + "o"].T


def mixer_retention(sd, p, m, h, eps):
    T = h.shape[0]
    H, D, Dv, r = m["heads"], m["dim"], m["vdim"], m["rot"]
    q = rotate_halves((h @ sd[p + "q"].T).view(T, H, D), r["dims"], r["base"])
    k = rotate_halves((h @ sd[p + "k"].T).view(T, H, D), r["dims"], r["base"]) / math.sqrt(D)
    o = retention_scan(q, k, (h @ sd[p + "v"].T).view(T, H, Dv), m["decay"])
    return (over_rms(o, eps).reshape(T, H * Dv) * silu(h @ sd[p + "g"].T)) @ sd[p + "o"].T


def mixer_parallel(sd, p, m, h, eps):
    p = p + "mix."
    left = mixer_window(sd, p + "left.", m["left"], h)
    right = mixer_retention(sd, p + "right.", m["right"], h, eps)
    return 0.5 * (over_rms(left, eps) * sd[p + "left.out"] + over_rms(right, eps) * sd[p + "right.out"])


def mixer_channel_delta(sd, p, m, h, eps):
    p = p + "mix."
    T = h.shape[0]
    H, G, D, Dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q, k, v = (silu(short_conv(h @ sd[p + t].T, sd[p + t + ".conv"])) for t in "qkv")
    q = unit(q.view(T, G, D)) / math.sqrt(D)
    k = unit(k.view(T, G, D))
    beta = torch.sigmoid(h @ sd[p + "b"].T)
    z = ((h @ sd[p + "a1"].T) @ sd[p + "a2"].T + sd[p + "dt_bias"]).view(T, H, D)
    g = torch.exp(-torch.exp(sd[p + "A_log"])[:, None] * softplus(z))
    o = over_rms(channel_delta_scan(q, k, v.view(T, H, Dv), g, beta), eps) * sd[p + "norm"]
    gate = torch.sigmoid((h @ sd[p + "g1"].T) @ sd[p + "g2"].T)
    return (o.reshape(T, H * Dv) * gate) @ sd[p + "o"].T


def ff_dense(sd, p, h):
    return (torch.relu(h @ sd[p + "mlp.up"].T) ** 2) @ sd[p + "mlp.down"].T


def clamped_glu(gate, up, limit):
    g, u = torch.clamp(gate, max=limit), torch.clamp(up, -limit, limit)
    return g * torch.sigmoid(1.702 * g) * (u + 1.0)


def route(z, f):
    """(expert, weight) pairs of one token from its router logits z [E]: softmax
    scores, the best groups by their largest score, the best experts in them,
    weights renormalised over the chosen ones and scaled."""
    r = f["router"]
    E, grp = r["experts"], r.get("groups") or {"count": 1, "keep": 1}
    s = torch.softmax(z, -1)
    per = E // grp["count"]
    best = sorted(range(grp["count"]), key=lambda j: -float(s[j * per:(j + 1) * per].max()))
    ok = [e for j in best[:grp["keep"]] for e in range(j * per, (j + 1) * per)]
    chosen = sorted(ok, key=lambda e: -float(s[e]))[:r["top"]]
    tot = sum(float(s[e]) for e in chosen) + 1e-20
    return [(e, float(s[e]) / tot * r["scale"]) for e in chosen]


def ff_moe(sd, p, f, h):
    z = h @ sd[p + "mlp.router"].T
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e, w in route(z[t], f):
            q = f"{p}mlp.e{e}."
            a = clamped_glu(sd[q + "gate"] @ h[t], sd[q + "up"] @ h[t], f["expert"]["limit"])
            out[t] += w * (sd[q + "down"] @ a)
    return out


def side_input(sd, p, x, e, eps):
    """The per-token side input of a layer, to be added to the residual."""
    y = (gelu_tanh(x @ sd[p + "side.gate"].T) * e) @ sd[p + "side.proj"].T
    return over_rms(y, eps) * sd[p + "side.norm"]


# ------------------------------------------------------------------ model
def schedule(cfg):
    """(layer, pass number when the run opens a pass of the repeated stretch)."""
    n, lp = len(cfg["layers"]), cfg.get("loop")
    if not lp:
        return [(i, None) for i in range(n)]
    out = [(i, None) for i in range(lp["start"])]
    for t in range(lp["times"]):
        out += [(i, t if i == lp["start"] else None) for i in range(lp["start"], lp["stop"])]
    return out + [(i, None) for i in range(lp["stop"], n)]


def forward(cfg, sd, tokens, trail=None):
    """f64 logits [T, vocab] of one whole sequence; ``trail`` collects the
    residual stream after every layer run."""
    sd = {k: v.to(F64) for k, v in sd.items()}
    eps, mult, S = cfg["norm"]["eps"], cfg["residual_mult"], cfg["token_side"]["dim"]
    x0 = embedding(sd, cfg, list(tokens))
    e = sd["side.embed"][torch.tensor(list(tokens))]
    x = x0
    for i, opens in schedule(cfg):
        L, p = cfg["layers"][i], f"l{i}."
        if opens is not None:
            x = torch.cat([x, x0], -1) @ sd["loop.in"].T + sd["loop.step"][opens]
        h = layer_norm(x, sd[p + "norm1"], sd[p + "norm1.b"], eps)
        mix = mixer_parallel if L["type"] == "parallel" else mixer_channel_delta
        x = x + mult * mix(sd, p, L["mixer"], h, eps)
        f = L["mlp"]
        if f is not None:
            h = layer_norm(x, sd[p + "norm2"], sd[p + "norm2.b"], eps)
            x = x + mult * (ff_dense(sd, p, h) if f["kind"] == "dense" else ff_moe(sd, p, f, h))
        x = x + mult * side_input(sd, p, x, e[:, i * S:(i + 1) * S], eps)
        if trail is not None:
            trail.append(x)
    return layer_norm(x, sd["final.norm"], sd["final.norm.b"], eps) @ sd["head"].T
