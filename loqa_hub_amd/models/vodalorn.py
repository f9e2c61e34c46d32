"""Vodalorn: a pre-norm decoder-only language model whose config.json lists its
layers one by one. With m a constant of the model and layer norms (weight and
bias), a layer is

    x <- x + m mixer(norm1(x))      x <- x + m ff(norm2(x))
    x <- x + m rms_norm(W_proj (gelu(W_gate x) * e))

where e is the layer's part of a second, per-token embedding (the side input).
The embedding adds a row of a pair table, chosen by a hash of the previous and
the current token, so the previous token is state of a sequence. A stretch of
layers may run several times in a row with the same weights and a cache or state
of its own per pass; every pass is entered through x <- W_in [x ; embedding
output] + step[t]. Mixers:

* ``parallel``: two mixers on the same input, half the sum of their outputs, each
  RMS-normed over the width with a weight: sliding-window grouped-query softmax
  attention (biases on q, k and v, rotary positions on a part of each head) and
  retention, S <- decay_h S + k v^T, o = S^T q with rotary q and k, k D^(-1/2), a
  per-head RMS norm without weight and the gate silu(W_g h);
* ``channel_delta``: a gated delta rule whose decay is one number per head and
  key channel, g = exp(-exp(A_log_h) softplus(W_a2 W_a1 h + dt_bias)): short causal
  convolutions with SiLU on q, k, v, unit-length q and k, S <- g S; u = beta (v -
  S^T k); S <- S + k u^T; o = S^T q, a per-head RMS norm with a weight shared by the
  heads and the gate sigmoid(W_g2 W_g1 h).

Feed-forwards: down(relu(up h)^2), or a mixture of experts with a clamped gated
unit, chosen by softmax scores within the best groups of experts, the chosen
scores renormalised and scaled.

MI355X layout, in the manner of the other decoders: a flat [T, width] token
batch (prompt portions beside decode tokens), an f32 residual stream updated
inside one launch that also forms what comes next - the next sublayer's normed
input, the bf16 rows of a product over x, or the left half of a pass entry's
[x ; x0] rows. Everything that reads one normed row is one projection (both
mixers of a parallel layer; q | k | v | beta and the two low-rank inputs of the
delta rule). The rotate-half layout is folded into the interleaved one by
permuting projection rows and biases at load time. Plain GEMMs go to the vendor
library (with an f32 result where it is the residual stream or enters a
recurrence); everything around them is this repository's HIP (``ops/seqmix.py``).
"""
from __future__ import annotations

import torch

from .. import ops
from ..ops import seqmix
from ..ops.seqmix import LnParams
from .configs import VodalornConfig
from .gopopel import stack_rows
from .vilulix import _head_rows, _pairs_from_halves


class VodalornWeights:
    """Device weights in the fused layouts, from a state dict in checkpoint
    naming (``embed``, ``bigram``, ``side.embed``, ``loop.in|step``,
    ``l<i>.norm1|norm2[.b]``, ``l<i>.mix.*``, ``l<i>.mlp.*``, ``l<i>.side.*``,
    ``final.norm``, ``head``)."""

    def __init__(self, cfg: VodalornConfig, sd: dict, device, dtype=torch.bfloat16,
                 max_positions: int = 8192):
        self.cfg, self.dtype, self.device = cfg, dtype, torch.device(device)
        self.max_positions = max_positions
        dev, d = self.device, cfg.d_model

        def W(name, *shape):    # a projection matrix in the activation dtype
            w = sd[name]
            if tuple(w.shape) != shape:
                raise ValueError(f"{name}: shape {tuple(w.shape)}, the config gives {shape}")
            return w.to(dev, dtype).contiguous()

        def F(name, *shape):    # small vectors and gate rows the f32 paths read
            w = sd[name]
            if tuple(w.shape) != shape:
                raise ValueError(f"{name}: shape {tuple(w.shape)}, the config gives {shape}")
            return w.to(dev, torch.float32).contiguous()

        def table(name, *shape):    # rows picked by token: as stored (bf16 or f32)
            w = sd[name]
            if tuple(w.shape) != shape:
                raise ValueError(f"{name}: shape {tuple(w.shape)}, the config gives {shape}")
            return w.to(dev, torch.bfloat16 if w.dtype == torch.bfloat16 else torch.float32
                        ).contiguous()

        def norm(name):
            return LnParams(F(name, d), F(name + ".b", d))

        self._W, self._F = W, F
        self.embed = table("embed", cfg.vocab_size, d)
        self.bigram = None
        if cfg.bigram is not None:
            self.bigram = table("bigram", cfg.bigram.buckets + 1, d)
            if self.bigram.dtype != self.embed.dtype:
                self.embed, self.bigram = self.embed.float(), self.bigram.float()
        self.side_embed = table("side.embed", cfg.vocab_size, cfg.n_layers * cfg.side_dim) \
            if cfg.side_dim else None
        self.loop_in = self.loop_step = None
        if cfg.loop is not None:
            self.loop_in = W("loop.in", d, 2 * d)
            self.loop_step = F("loop.step", cfg.loop.times, d)
        self.head = F("head", cfg.vocab_size, d)
        self.final_norm = norm("final.norm")
        self._tables: dict[tuple, torch.Tensor] = {}
        self.layers: list[dict] = []
        for i, lc in enumerate(cfg.layers):
            p, f = f"l{i}.", lc.mlp
            L: dict = {"norm1": norm(p + "norm1")}
            if lc.kind == "channel_delta":
                self._channel_delta(L, p + "mix.", lc.mixer, sd)
            else:
                self._parallel(L, p + "mix.", lc.mixer)
            if f is not None:
                L["norm2"] = norm(p + "norm2")
                q = p + "mlp."
                if f.kind == "dense":
                    L["w_up"], L["w_down"] = W(q + "up", f.ff, d), W(q + "down", d, f.ff)
                else:
                    # f32 products of 16-bit values are exact: a router stored in
                    # 16 bits needs no f32 copy for f32 logits
                    L["router"] = (W if sd[q + "router"].dtype == torch.bfloat16 else F)(
                        q + "router", f.experts, d)
                    L["e_gate_up"] = torch.stack([
                        torch.cat([W(f"{q}e{e}.gate", f.ff, d), W(f"{q}e{e}.up", f.ff, d)])
                        for e in range(f.experts)]).contiguous()
                    L["e_down"] = torch.stack([W(f"{q}e{e}.down", d, f.ff)
                                               for e in range(f.experts)]).contiguous()
            if cfg.side_dim:
                L["side_gate"] = W(p + "side.gate", cfg.side_dim, d)
                L["side_proj"] = W(p + "side.proj", d, cfg.side_dim)
                L["side_norm"] = F(p + "side.norm", d)
            self.layers.append(L)
        del self._W, self._F

    def _channel_delta(self, L: dict, p: str, m, sd: dict) -> None:
        W, F, d, dev = self._W, self._F, self.cfg.d_model, self.device
        H, G, D, Dv = m.heads, m.kv_heads, m.dim, m.vdim
        Ra, Rg = sd[p + "a1"].shape[0], sd[p + "g1"].shape[0]
        qkv = torch.cat([W(p + "q", G * D, d), W(p + "k", G * D, d), W(p + "v", H * Dv, d)])
        L["w_in"], L["offs"] = stack_rows([qkv, W(p + "b", H, d), W(p + "a1", Ra, d),
                                           W(p + "g1", Rg, d)])
        L["ranks"] = Ra, Rg
        L["w_a2"], L["w_g2"] = W(p + "a2", H * D, Ra), W(p + "g2", H * Dv, Rg)
        L["conv"] = torch.cat([F(p + "q.conv", G * D, m.taps), F(p + "k.conv", G * D, m.taps),
                               F(p + "v.conv", H * Dv, m.taps)]).t().contiguous()  # tap-major
        L["a_neg"] = -torch.exp(F(p + "A_log", H))
        L["dt_bias"] = F(p + "dt_bias", H * D)
        L["norm"] = F(p + "norm", Dv).repeat(H).contiguous()         # shared by the heads
        L["wo"] = W(p + "o", d, H * Dv)

    def _parallel(self, L: dict, p: str, m) -> None:
        W, F, d, dev = self._W, self._F, self.cfg.d_model, self.device
        a, r = m.left, m.right
        q = p + "left."
        H, G, D, Dv = a.heads, a.kv_heads, a.dim, a.vdim
        per = _pairs_from_halves(a.rot.dims, D)[:a.rot.dims]
        iq, ik = _head_rows(H, D, 0, per).to(dev), _head_rows(G, D, 0, per).to(dev)
        left = torch.cat([W(q + "q", H * D, d)[iq], W(q + "k", G * D, d)[ik], W(q + "v", G * Dv, d)])
        bias = torch.cat([W(q + "q.b", H * D)[iq], W(q + "k.b", G * D)[ik], W(q + "v.b", G * Dv)])
        L["l_v_off"] = (H + G) * D
        L["l_wo"] = W(q + "o", d, H * Dv)
        L["l_cos_sin"] = self._table(a.rot)
        L["l_out"] = F(q + "out", d)
        q = p + "right."
        H, D, Dv = r.heads, r.dim, r.vdim
        per = _pairs_from_halves(r.rot.dims, D)[:r.rot.dims]
        ih = _head_rows(H, D, 0, per).to(dev)
        right = torch.cat([W(q + "q", H * D, d)[ih], W(q + "k", H * D, d)[ih], W(q + "v", H * Dv, d)])
        # left q | k | v, right q | k | v, right gate
        L["w_in"], L["offs"] = stack_rows([left, right, W(q + "g", H * Dv, d)])
        L["b_in"] = torch.zeros(L["w_in"].shape[0], dtype=self.dtype, device=dev)
        L["b_in"][:bias.numel()] = bias
        L["r_decay"] = torch.tensor(r.decay, dtype=torch.float32, device=dev)
        L["r_norm"] = torch.ones(H * Dv, dtype=torch.float32, device=dev)     # no weight
        L["r_cos_sin"] = self._table(r.rot)
        L["r_wo"] = W(q + "o", d, H * Dv)
        L["r_out"] = F(q + "out", d)

    def _table(self, rot) -> torch.Tensor | None:
        if not rot.dims:
            return None
        key = (rot.dims, rot.base)
        if key not in self._tables:
            self._tables[key] = seqmix.rope_table_pairs(rot.dims, self.max_positions, rot.base,
                                                        None, self.device)
        return self._tables[key]

    @classmethod
    def random(cls, cfg: VodalornConfig, device, seed: int = 0, dtype=torch.bfloat16,
               max_positions: int = 8192) -> "VodalornWeights":
        return cls(cfg, random_state_dict(cfg, seed), device, dtype, max_positions)


def random_state_dict(cfg: VodalornConfig, seed: int = 0, rank: int | None = None) -> dict:
    """Seeded random weights in checkpoint naming (bf16), scaled so that
    activations stay O(1) through the stack; used by tests, smoke and bench.
    ``rank``: of the delta rule's low-rank projections (a head's key size)."""
    g = torch.Generator().manual_seed(seed)
    d, S = cfg.d_model, cfg.side_dim
    sd: dict = {}

    def mat(name, rows, cols, gain=1.0):
        sd[name] = (torch.randn(rows, cols, generator=g) * gain / cols ** 0.5).to(torch.bfloat16)

    def vec(name, n, mean=0.0, std=0.1):
        sd[name] = (mean + torch.randn(n, generator=g) * std).to(torch.bfloat16)

    def norm(name):
        vec(name, d, 1.0)
        vec(name + ".b", d, 0.0, 0.05)

    def rows(name, n, w):
        sd[name] = torch.randn(n, w, generator=g).to(torch.bfloat16)

    rows("embed", cfg.vocab_size, d)
    if cfg.bigram is not None:
        rows("bigram", cfg.bigram.buckets + 1, d)
    if S:
        rows("side.embed", cfg.vocab_size, cfg.n_layers * S)
    if cfg.loop is not None:
        mat("loop.in", d, 2 * d, 1.4)
        rows("loop.step", cfg.loop.times, d)
    for i, lc in enumerate(cfg.layers):
        p, m, f = f"l{i}.", lc.mixer, lc.mlp
        norm(p + "norm1")
        q = p + "mix."
        if lc.kind == "channel_delta":
            H, GD, HV = m.heads, m.kv_heads * m.dim, m.heads * m.vdim
            R = rank or m.dim
            for n, c in (("q", GD), ("k", GD), ("v", HV)):
                mat(q + n, c, d, 2.0)
                sd[q + n + ".conv"] = (torch.randn(c, m.taps, generator=g) * 0.5).to(torch.bfloat16)
            mat(q + "b", H, d, 2.0)
            vec(q + "A_log", H, -0.5, 0.7); vec(q + "dt_bias", H * m.dim, -0.5, 0.5)
            mat(q + "a1", R, d); mat(q + "a2", H * m.dim, R)
            mat(q + "g1", R, d); mat(q + "g2", HV, R)
            vec(q + "norm", m.vdim, 1.0)
            mat(q + "o", d, HV, 2.0)
        else:
            a, r = m.left, m.right
            for n, c in (("q", a.heads * a.dim), ("k", a.kv_heads * a.dim),
                         ("v", a.kv_heads * a.vdim)):
                mat(q + "left." + n, c, d, 2.0)
                vec(q + "left." + n + ".b", c)
            mat(q + "left.o", d, a.heads * a.vdim, 2.0)
            for n, c in (("q", r.heads * r.dim), ("k", r.heads * r.dim), ("v", r.heads * r.vdim),
                         ("g", r.heads * r.vdim)):
                mat(q + "right." + n, c, d, 2.0)
            mat(q + "right.o", d, r.heads * r.vdim, 2.0)
            vec(q + "left.out", d, 1.0); vec(q + "right.out", d, 1.0)
        if f is not None:
            norm(p + "norm2")
            if f.kind == "dense":
                mat(p + "mlp.up", f.ff, d, 1.5); mat(p + "mlp.down", d, f.ff, 1.5)
            else:
                for e in range(f.experts):
                    mat(f"{p}mlp.e{e}.gate", f.ff, d, 2.0); mat(f"{p}mlp.e{e}.up", f.ff, d, 2.0)
                    mat(f"{p}mlp.e{e}.down", d, f.ff, 2.0)
                mat(p + "mlp.router", f.experts, d, 3.0)
        if S:
            mat(p + "side.gate", S, d, 1.5); mat(p + "side.proj", d, S)
            vec(p + "side.norm", d, 1.0)
    norm("final.norm")
    mat("head", cfg.vocab_size, d, 2.0)
    return sd


def config_to_json(cfg: VodalornConfig) -> dict:
    """The config.json of ``cfg`` (the inverse of ``vodalorn_config_from_json``)."""
    layers = []
    for lc in cfg.layers:
        m, f = lc.mixer, lc.mlp
        if lc.kind == "channel_delta":
            mx = {"heads": m.heads, "kv_heads": m.kv_heads, "dim": m.dim, "vdim": m.vdim,
                  "conv": m.taps}
        else:
            a, r = m.left, m.right
            mx = {"left": {"heads": a.heads, "kv_heads": a.kv_heads, "dim": a.dim, "vdim": a.vdim,
                           "scale": a.scale, "mask": {"size": a.window},
                           "rot": {"dims": a.rot.dims, "base": a.rot.base}},
                  "right": {"heads": r.heads, "dim": r.dim, "vdim": r.vdim, "decay": list(r.decay),
                            "rot": {"dims": r.rot.dims, "base": r.rot.base}}}
        if f is None:
            mlp = None
        elif f.kind == "dense":
            mlp = {"kind": "dense", "ff": f.ff}
        else:
            mlp = {"kind": "moe", "expert": {"ff": f.ff, "limit": f.limit},
                   "router": {"experts": f.experts, "top": f.top, "scale": f.weight_scale,
                              "groups": {"count": f.groups, "keep": f.keep}}}
        layers.append({"type": lc.kind, "mixer": mx, "mlp": mlp})
    out = {"architecture": "Vodalorn", "vocab": cfg.vocab_size, "width": cfg.d_model,
           "norm": {"eps": cfg.norm_eps}, "residual_mult": cfg.residual_mult, "layers": layers}
    if cfg.bigram is not None:
        b = cfg.bigram
        out["embedding"] = {"bigram": {"buckets": b.buckets, "mul_prev": b.mul_prev,
                                       "mul_cur": b.mul_cur}}
    if cfg.side_dim:
        out["token_side"] = {"dim": cfg.side_dim}
    if cfg.loop is not None:
        out["loop"] = {"start": cfg.loop.start, "stop": cfg.loop.stop, "times": cfg.loop.times}
    return out


class VodalornModel:
    """The step function: one pass of a flat token batch through all layer runs,
    reading and extending the paged K / V cache and the state slots."""

    hybrid = True
    # a step with at least this many tokens runs the attention side of a parallel
    # layer on a second HIP stream beside the retention scan, whose few long-running
    # waves leave most of the GPU idle; smaller steps are bound by launches
    overlap_min_tokens = 128

    def __init__(self, w: VodalornWeights):
        self.w, self.cfg = w, w.cfg
        self.runs = self.cfg.runs()
        self._side = None

    def _side_stream(self, T: int):
        """The second stream for a step of T tokens (default priority), or None."""
        if self.w.device.type != "cuda" or T < self.overlap_min_tokens:
            return None
        if self._side is None:
            from ..utils.streams import placed_stream
            self._side = placed_stream(self.w.device, "mixer")
        return self._side

    # the cache manager sizes its storage from this: one entry per layer RUN (a
    # layer of the repeated stretch holds a cache or state per pass)
    def cache_spec(self) -> dict:
        kv, state, rows = {}, {}, {}
        for r, (i, _) in enumerate(self.runs):
            m = self.cfg.layers[i].mixer
            if self.cfg.layers[i].kind == "channel_delta":
                state[r] = (m.heads, m.vdim, m.dim)        # a column's rows side by side
                if m.taps > 1:
                    rows[r] = {"tail": (m.taps - 1, m.conv_channels)}
            else:
                kv[r] = (m.left.kv_heads * m.left.dim, m.left.kv_heads * m.left.vdim)
                state[r] = (m.right.heads, m.right.dim, m.right.vdim)
        ints = {"embedding": {"prev": ()}} if self.cfg.bigram is not None else {}
        return {"latent": {}, "state": state, "kv_rows": kv, "rows": rows, "ints": ints}

    def embed(self, meta, cache, entry: torch.Tensor | None) -> torch.Tensor:
        """The embedding output, f32 [T, d]; ``entry`` [T, 2 d] receives two copies."""
        w, b = self.w, self.cfg.bigram
        if b is not None:
            return seqmix.bigram_embed(meta.tokens, w.embed, w.bigram, b.mul_prev, b.mul_cur,
                                       cache.ints["embedding"]["prev"], meta.state_slots, meta.cu_q,
                                       meta.positions, entry)
        x = torch.nn.functional.embedding(meta.tokens.long(), w.embed).float()
        if entry is not None:
            entry.copy_(x.repeat(1, 2))
        return x

    def forward(self, meta, cache, trail: list | None = None) -> torch.Tensor:
        """f32 logits [len(meta.logit_idx), vocab] of one step. ``meta``: the
        engine's StepMeta; ``cache``: a HybridCache. ``trail`` collects the
        residual stream after every layer run (tests)."""
        w, cfg, dt = self.w, self.cfg, self.w.dtype
        eps, mult, d, n = cfg.norm_eps, cfg.residual_mult, self.cfg.d_model, len(self.runs)
        T, dev = meta.tokens.numel(), w.device
        # rows [x ; x0] of the pass entries; every pass writes its own left half
        entry = torch.empty(T, 2 * d, dtype=dt, device=dev) if cfg.loop is not None else None
        x = self.embed(meta, cache, entry)

        def step(adds, scale, nxt):
            """x += scale * adds; the rows ``nxt`` asks for: a layer norm's, "rows"
            (x in the activation dtype), "entry" (the same, into the entry rows)."""
            if nxt is None:
                out = None
            elif isinstance(nxt, str) and nxt == "entry":
                out = entry[:, :d]
            elif isinstance(nxt, str) and dt == torch.float32:
                seqmix.residual_ln(x, adds, scale, None, eps, None)
                return x
            else:
                out = torch.empty(T, d, dtype=dt, device=dev)
            return seqmix.residual_ln(x, adds, scale, None if isinstance(nxt, str) else nxt, eps, out)

        h = None
        if n and self.runs[0][1] is None:
            h = step([], 1.0, w.layers[self.runs[0][0]]["norm1"])
        for r, (i, opens) in enumerate(self.runs):
            lc, L = cfg.layers[i], w.layers[i]
            if opens is not None:
                x = seqmix.linear_f32(entry, w.loop_in)
                h = seqmix.residual_ln(x, [], 1.0, L["norm1"], eps,
                                       torch.empty(T, d, dtype=dt, device=dev),
                                       vec=w.loop_step[opens])
            # what the next run starts from
            nxt = None
            if r + 1 < n:
                j, o = self.runs[r + 1]
                nxt = "entry" if o is not None else w.layers[j]["norm1"]
            tail = "rows" if cfg.side_dim else nxt          # what the feed-forward leaves behind
            if lc.kind == "channel_delta":
                adds, scale = self._channel_delta(r, lc.mixer, L, h, meta, cache), mult
            else:
                # both outputs carry the same constant
                adds = self._parallel(r, lc.mixer, L, h, meta, cache)
                scale = mult * lc.mixer.left_scale
            f = lc.mlp
            if f is not None:
                h = step(adds, scale, L["norm2"])
                adds, scale = [(self._dense(L, h) if f.kind == "dense" else self._moe(f, L, h), None)], mult
            h = step(adds, scale, tail)
            if cfg.side_dim:
                g = seqmix.token_gate(ops.linear(h, L["side_gate"]), w.side_embed, meta.tokens,
                                      i * cfg.side_dim)
                h = step([(ops.linear(g, L["side_proj"]), L["side_norm"])], mult, nxt)
            if trail is not None:
                trail.append(x.clone())
        rows = meta.logit_idx.numel()
        hf = seqmix.residual_ln(x, [], 1.0, w.final_norm, eps,
                                torch.empty(rows, d, dtype=torch.float32, device=dev),
                                row_idx=meta.logit_idx)
        return ops.linear(hf, w.head)

    def _channel_delta(self, r, m, L, h, meta, cache) -> list:
        H, G, D, Dv, C = m.heads, m.kv_heads, m.dim, m.vdim, m.conv_channels
        u = ops.linear(h, L["w_in"])                       # q | k | v, beta, decay and gate latents
        _, b_off, a_off, g_off = L["offs"]
        Ra, Rg = L["ranks"]
        za = seqmix.linear_f32(u[:, a_off:a_off + Ra], L["w_a2"])
        gate = ops.linear(u[:, g_off:g_off + Rg], L["w_g2"])
        tail = cache.rows[r]["tail"] if m.taps > 1 else \
            torch.zeros(1, 0, C, dtype=torch.float32, device=u.device)
        act, tok = seqmix.delta_prep(u, None, G, D, H, Dv, L["conv"], tail, L["a_neg"],
                                     L["dt_bias"], meta.state_slots, meta.cu_q, meta.positions,
                                     chan=(za, b_off))
        if m.taps > 1:
            # every reader of this step's tail is done: store the new rows
            seqmix.seq_state_save(None, u, None, tail, meta.state_slots, meta.cu_q, meta.positions)
        o = seqmix.delta_scan(act, H, D, Dv, 0, G * D, 2 * G * D, H // G, cache.state[r],
                              meta.state_slots, meta.cu_q, meta.positions, tok, g_off=C,
                              max_q=meta.max_q)
        y = seqmix.gated_rmsnorm(o, L["norm"], gate, self.cfg.norm_eps, self.w.dtype, groups=H)
        return [(ops.linear(y, L["wo"]), None)]

    def _parallel(self, r, m, L, h, meta, cache) -> list:
        u = ops.linear(h, L["w_in"], L["b_in"])            # left q | k | v, right q | k | v, gate
        side = self._side_stream(u.shape[0])
        if side is None:
            left = self._window(r, m.left, L, u, meta, cache)
            right = self._retention(r, m.right, L, u, meta, cache)
        else:
            main = torch.cuda.current_stream(u.device)
            side.wait_stream(main)
            with torch.cuda.stream(side):
                left = self._window(r, m.left, L, u, meta, cache)
            right = self._retention(r, m.right, L, u, meta, cache)
            # joined before anything either stream reads is given up here
            main.wait_stream(side)
        return [(left, L["l_out"]), (right, L["r_out"])]

    def _window(self, r, a, L, u, meta, cache) -> torch.Tensor:
        H, G, D, Dv = a.heads, a.kv_heads, a.dim, a.vdim
        kc, vc = cache.kv_rows[r]
        q = seqmix.qk_prep_append(u, H, G, D, Dv, L["l_v_off"], L["l_cos_sin"], a.rot.dims,
                                  self.cfg.norm_eps, None, meta.positions, kc, vc, meta.slots,
                                  self.w.dtype, norm=False)
        o = seqmix.window_attention(q, kc, vc, meta.cu_q, meta.ctx_lens, meta.block_tables,
                                    meta.positions, a.scale, 0.0, a.window, 0, None, H, G, D, Dv,
                                    meta.max_q, max_ctx=meta.max_ctx)
        return ops.linear(o, L["l_wo"])

    def _retention(self, r, m, L, u, meta, cache) -> torch.Tensor:
        H, D, Dv = m.heads, m.dim, m.vdim
        _, off, g_off = L["offs"]
        act = seqmix.retention_prep(u[:, off:off + 2 * H * D + H * Dv], H, D, Dv, L["r_cos_sin"],
                                    m.rot.dims, meta.positions)
        o = seqmix.state_scan(act, H, D, Dv, 0, H * D, 2 * H * D, 1, cache.state[r],
                              meta.state_slots, meta.cu_q, meta.positions, decay=L["r_decay"],
                              max_q=meta.max_q)
        y = seqmix.gated_rmsnorm(o, L["r_norm"], u[:, g_off:g_off + H * Dv], self.cfg.norm_eps,
                                 self.w.dtype, groups=H, gate_act="silu")
        return ops.linear(y, L["r_wo"])

    @staticmethod
    def _dense(L, h) -> torch.Tensor:
        return ops.linear(seqmix.relu2_(ops.linear(h, L["w_up"])), L["w_down"])

    @staticmethod
    def _moe(f, L, h) -> torch.Tensor:
        rw = L["router"]
        z = seqmix.linear_f32(h if rw.dtype == h.dtype else h.float(), rw)
        idx, wt = seqmix.moe_route(z, None, f.groups, f.keep, f.top, group_rank=f.group_rank,
                                   renorm=f.renorm, weight_scale=f.weight_scale)
        return seqmix.moe_experts(h, idx, wt, L["e_gate_up"], L["e_down"], limit=f.limit)
