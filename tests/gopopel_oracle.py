"""A plain, slow float64 implementation of the Gopopel decoder, written from its
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
def biased(heads=4, kv_heads=2, dim=12, vdim=10, window=6, scale=None, v_mix=True):
    """Windowed attention with a linear distance bias and a learned sink."""
    return "attention", {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim,
                         "scale": scale if scale is not None else dim ** -0.5,
                         "mask": {"size": window}, "v_mix": v_mix}


def latent(heads=3, dim=8, rot_dim=4, vdim=10, kv_rank=12, q_rank=14, window=9, scale=None,
           base=100.0):
    return "latent_attention", {
        "heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "kv_rank": kv_rank,
        "q_rank": q_rank, "scale": scale if scale is not None else (dim + rot_dim) ** -0.5,
        "mask": {"size": window}, "rot": {"dims": rot_dim, "base": base}}


def dense_ff(ff=40):
    return {"kind": "dense", "ff": ff}


def make_config(layers, width=32, vocab=50, eps=1e-5, embed_scale=1.7):
    return {"architecture": "Gopopel", "vocab": vocab, "width": width, "norm": {"eps": eps},
            "embedding": {"scale": embed_scale},
            "layers": [{"type": t, "mixer": m, "mlp": f} for (t, m), f in layers]}


def make_weights(cfg, seed=0):
    """Random weights in checkpoint naming whose values are exact in bfloat16."""
    g = torch.Generator().manual_seed(seed)
    d = cfg["width"]
    sd = {}

    def put(name, t):
        sd[name] = t.to(torch.bfloat16).float()

    def mat(name, rows, cols, gain=1.0):
        put(name, torch.randn(rows, cols, generator=g) * gain / cols ** 0.5)

    def vec(name, n, mean=0.0, std=0.1):
        put(name, mean + torch.randn(n, generator=g) * std)

    def norm(name):
        vec(name, d, 1.0, 0.2)
        vec(name + ".b", d, 0.0, 0.1)
        put(name + ".alpha", 0.4 + 0.4 * torch.rand((), generator=g))

    put("embed", torch.randn(cfg["vocab"], d, generator=g))
    for i, L in enumerate(cfg["layers"]):
        p, m = f"l{i}.", L["mixer"]
        norm(p + "norm1")
        q = p + "mix."
        if L["type"] == "attention":
            H, G, D, Dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
            mat(q + "q", H * D, d, 2.0); mat(q + "k", G * D, d, 2.0); mat(q + "v", G * Dv, d, 2.0)
            vec(q + "q.norm", D, 1.2, 0.3); vec(q + "k.norm", D, 1.2, 0.3)
            put(q + "vmix", 0.2 + 0.6 * torch.rand((), generator=g))
            vec(q + "sink", H, 0.0, 1.0)
            mat(q + "o", d, H * Dv, 2.0)
        else:
            H, D, Dr, Dv = m["heads"], m["dim"], m["rot_dim"], m["vdim"]
            R, Rq = m["kv_rank"], m["q_rank"]
            mat(q + "dq", Rq, d, 2.0); vec(q + "dq.norm", Rq, 1.0, 0.2)
            mat(q + "uq", H * (D + Dr), Rq, 2.0)
            mat(q + "dkv", R + Dr, d, 2.0); vec(q + "dkv.norm", R, 1.0, 0.2)
            mat(q + "uk", H * D, R, 2.0); mat(q + "uv", H * Dv, R, 2.0)
            mat(q + "g", H * Dv, d, 2.0)
            mat(q + "o", d, H * Dv, 2.0)
        f = L["mlp"]
        if f is not None:
            mat(p + "mlp.up", f["ff"], d, 1.5)
            mat(p + "mlp.down", d, f["ff"], 1.5)
    norm("final.norm")
    mat("head", cfg["vocab"], d, 2.0)
    return sd


# -------------------------------------------------------------- mechanisms
def dynamic_tanh(x, w, b, alpha):
    """An elementwise squashing norm: no statistics of the row."""
    return torch.tanh(alpha * x) * w + b


def norm_plain(x, w, eps):
    """x divided by its root mean square over the last axis (eps inside the
    root), times a plain weight."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps) * w


def rotate_pairs(x, dims, base, pos=None):
    """x [T, heads, size]: entries 2i and 2i + 1 of the first ``dims`` turn
    together by the angle p * base^(-2 i / dims)."""
    T = x.shape[0]
    if dims == 0:
        return x
    p = torch.arange(T, dtype=F64) if pos is None else pos.to(F64)
    f = torch.tensor([base ** (-2.0 * i / dims) for i in range(dims // 2)], dtype=F64)
    a = p[:, None] * f[None, :]
    c, s = torch.cos(a)[:, None, :], torch.sin(a)[:, None, :]
    y = x.clone()
    u, v = x[..., 0:dims:2], x[..., 1:dims:2]
    y[..., 0:dims:2] = u * c - v * s
    y[..., 1:dims:2] = v * c + u * s
    return y


def slopes(H):
    """Geometric slopes of the distance bias, 2^(-8/H), 2^(-16/H), ..., 2^-8."""
    return [2.0 ** (-8.0 * (h + 1) / H) for h in range(H)]


def attention(q, k, v, scale, window=0, bias_slopes=None, sink=None):
    """q [T, H, D], k [T, G, D], v [T, G, Dv]; key j visible to query i when
    j <= i and (window == 0 or i - j < window); score = q . k scale - slope_h
    (i - j); with ``sink`` [H] the softmax denominator also holds exp(sink_h)."""
    T, H, _ = q.shape
    G = k.shape[1]
    out = torch.zeros(T, H, v.shape[2], dtype=F64)
    i = torch.arange(T)
    dist = i[:, None] - i[None, :]
    vis = dist >= 0
    if window:
        vis &= dist < window
    for h in range(H):
        g = h // (H // G)
        s = (q[:, h] @ k[:, g].T) * scale
        if bias_slopes is not None:
            s = s - bias_slopes[h] * dist.to(F64)
        s = s.masked_fill(~vis, -math.inf)
        m = s.max(-1, keepdim=True).values
        if sink is not None:
            m = torch.clamp(m, min=float(sink[h]))
        e = torch.exp(s - m)
        den = e.sum(-1, keepdim=True)
        if sink is not None:
            den = den + torch.exp(float(sink[h]) - m)
        out[:, h] = (e / den) @ v[:, g]
    return out


def mix_values(v, v_first, lam):
    """A layer's values blended with the first mixing layer's of the same token."""
    return v if v_first is None else (1.0 - lam) * v + lam * v_first


def mixer_biased_attention(sd, p, m, h, eps, v_first):
    """Returns (mixer output, this layer's values as projected)."""
    p = p + "mix."
    T = h.shape[0]
    H, G, D, Dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = norm_plain((h @ sd[p + "q"].T).view(T, H, D), sd[p + "q.norm"], eps)
    k = norm_plain((h @ sd[p + "k"].T).view(T, G, D), sd[p + "k.norm"], eps)
    v = h @ sd[p + "v"].T
    vm = mix_values(v, v_first, sd[p + "vmix"]) if m.get("v_mix") else v
    o = attention(q, k, vm.view(T, G, Dv), m["scale"], m["mask"]["size"], slopes(H), sd[p + "sink"])
    return o.reshape(T, H * Dv) @ sd[p + "o"].T, v


def mixer_latent(sd, p, m, h, eps):
    p = p + "mix."
    T = h.shape[0]
    H, D, Dr, Dv, R = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    r = m["rot"]
    cq = norm_plain(h @ sd[p + "dq"].T, sd[p + "dq.norm"], eps)
    q = (cq @ sd[p + "uq"].T).view(T, H, D + Dr)
    z = h @ sd[p + "dkv"].T
    c = norm_plain(z[:, :R], sd[p + "dkv.norm"], eps)
    kr = rotate_pairs(z[:, None, R:], r["dims"], r["base"])                # [T, 1, Dr]
    qr = rotate_pairs(q[..., D:], r["dims"], r["base"])
    kk = torch.cat([(c @ sd[p + "uk"].T).view(T, H, D), kr.expand(T, H, Dr)], -1)
    qq = torch.cat([q[..., :D], qr], -1)
    v = (c @ sd[p + "uv"].T).view(T, H, Dv)
    o = attention(qq, kk, v, m["scale"], m["mask"]["size"]).reshape(T, H * Dv)
    return (o * torch.sigmoid(h @ sd[p + "g"].T)) @ sd[p + "o"].T


def ff_dense(sd, p, h):
    """down(relu(up h)^2)."""
    return (torch.relu(h @ sd[p + "mlp.up"].T) ** 2) @ sd[p + "mlp.down"].T


# ------------------------------------------------------------------ model
def forward(cfg, sd, tokens, trail=None):
    """f64 logits [T, vocab] of one whole sequence; ``trail`` collects the
    residual stream after every layer."""
    sd = {k: v.to(F64) for k, v in sd.items()}
    eps = cfg["norm"]["eps"]

    def norm(name, x):
        return dynamic_tanh(x, sd[name], sd[name + ".b"], sd[name + ".alpha"])

    x = sd["embed"][torch.as_tensor(tokens, dtype=torch.long)] * cfg["embedding"]["scale"]
    v_first = None
    for i, L in enumerate(cfg["layers"]):
        p, m = f"l{i}.", L["mixer"]
        h = norm(p + "norm1", x)
        if L["type"] == "attention":
            y, v = mixer_biased_attention(sd, p, m, h, eps, v_first)
            if m.get("v_mix") and v_first is None:
                v_first = v
        else:
            y = mixer_latent(sd, p, m, h, eps)
        if L["mlp"] is not None:
            y = y + ff_dense(sd, p, h)
        x = x + y
        if trail is not None:
            trail.append(x.clone())
    return norm("final.norm", x) @ sd["head"].T
