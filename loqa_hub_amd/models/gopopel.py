"""Gopopel: a decoder-only language model of parallel layers whose config.json
lists its layers one by one:

    h = norm(x);   x <- x + mixer(h) + ff(h)

one Dynamic-Tanh norm (tanh(alpha x) * w + b, no statistics) per layer that both
sublayers read; the embedding is scaled by a constant. Mixers:

* ``attention``: sliding-window grouped-query softmax attention without rotary
  positions. q and k are RMS-normed per head (weights shared by the heads); a
  linear distance bias slope_h (i - j) comes off the scores, with the geometric
  slopes 2^(-8 (h + 1) / H); the softmax denominator holds a learned sink per
  head; layers marked ``v_mix`` blend their values with those of the first such
  layer, v <- (1 - lam) v + lam v_first, and cache the blend;
* ``latent_attention``: sliding-window attention over a cached latent row and
  one rotary key part (interleaved pairs) shared by all heads, the queries
  through an RMS-normed latent of their own, the heads' outputs times
  sigmoid(W_g h).

Feed-forwards are ungated, down(relu(up h)^2).

MI355X layout, in the manner of the other decoders: a flat [T, width] token
batch (prompt portions beside decode tokens), an f32 residual stream, K / V and
latent pages on the shared block pool. What a parallel layer with ONE norm
allows on top: every projection of h, the feed-forward's up projection
included, is one matrix product, and the output projections of both sublayers
are one product over the side-by-side row [heads | relu(up)^2]. The launch that
prepares the mixer's inputs (q / k norms and paged append, or the latent norms,
rotation and append) also squares the up columns into that row, attention
writes its heads beside them, and one launch adds the product to the residual
and norms for the next layer: five launches for an ``attention`` layer. Plain
GEMMs go to the vendor library; everything around them is this repository's
HIP (``ops/seqmix.py``).
"""
from __future__ import annotations

import torch

from .. import ops
from ..ops import seqmix
from ..ops.seqmix import DytParams, SideCols
from .configs import GopopelConfig
from .pipizen import latent_heads, latent_prompt_layout


def stack_rows(parts: list[torch.Tensor]) -> tuple[torch.Tensor, list[int]]:
    """Projections [n_i, d] of one input as ONE matrix, every part starting at a
    multiple of 8 rows (zero rows in between and at the end), so that each
    part's output columns are 16-byte aligned. Returns (matrix, first rows)."""
    rows, offs, at = [], [], 0
    for w in parts:
        offs.append(at)
        pad = -w.shape[0] % 8
        rows.append(w)
        if pad:
            rows.append(torch.zeros(pad, w.shape[1], dtype=w.dtype, device=w.device))
        at += w.shape[0] + pad
    return torch.cat(rows).contiguous(), offs


class GopopelWeights:
    """Device weights in the fused layouts, from a state dict in checkpoint
    naming (``embed``, ``l<i>.norm1[.b|.alpha]``, ``l<i>.mix.*``, ``l<i>.mlp.*``,
    ``final.norm``, ``head``)."""

    def __init__(self, cfg: GopopelConfig, sd: dict, device, dtype=torch.bfloat16,
                 max_positions: int = 8192):
        self.cfg, self.dtype, self.device = cfg, dtype, torch.device(device)
        self.max_positions = max_positions
        dev, d = self.device, cfg.d_model

        def W(name, *shape):    # a projection matrix in the activation dtype
            w = sd[name]
            if tuple(w.shape) != shape:
                raise ValueError(f"{name}: shape {tuple(w.shape)}, the config gives {shape}")
            return w.to(dev, dtype).contiguous()

        def F(name, n):         # small vectors the f32 paths read
            w = sd[name]
            if w.numel() != n:
                raise ValueError(f"{name}: {w.numel()} entries, the config gives {n}")
            return w.to(dev, torch.float32).reshape(n).contiguous()

        def norm(name):
            return DytParams(F(name, d), F(name + ".b", d), float(F(name + ".alpha", 1)))

        if tuple(sd["embed"].shape) != (cfg.vocab_size, d) or \
                tuple(sd["head"].shape) != (cfg.vocab_size, d):
            raise ValueError("embed or head does not match vocab x width")
        # the embedding's scale is folded into its f32 rows (the residual is f32)
        self.embed = sd["embed"].to(dev, torch.float32) * cfg.embed_scale
        self.head = sd["head"].to(dev, torch.float32).contiguous()
        self.final_norm = norm("final.norm")
        self._tables: dict[tuple, torch.Tensor] = {}
        self.layers: list[dict] = []
        for i, lc in enumerate(cfg.layers):
            p, m, f = f"l{i}.", lc.mixer, lc.mlp
            L: dict = {"norm1": norm(p + "norm1")}
            q, H, Dv = p + "mix.", m.heads, m.vdim
            if lc.kind == "attention":
                G, D = m.kv_heads, m.dim
                # q, k and v rows side by side (the append launch reads them so)
                parts = [torch.cat([W(q + "q", H * D, d), W(q + "k", G * D, d),
                                    W(q + "v", G * Dv, d)])]
                L["v_off"] = (H + G) * D
                L["q_norm"], L["k_norm"] = F(q + "q.norm", D), F(q + "k.norm", D)
                L["sink"] = F(q + "sink", H) if m.sink else None
                L["slopes"] = seqmix.alibi_slopes(H, dev) if m.alibi else None
                L["vmix"] = float(F(q + "vmix", 1)) if m.v_mix and i != cfg.first_v_mix else None
            else:
                D, Dr, R, Rq = m.dim, m.rot_dim, m.kv_rank, m.q_rank
                parts = [W(q + "dq", Rq, d), W(q + "dkv", R + Dr, d), W(q + "g", H * Dv, d)]
                L["dq_norm"], L["dkv_norm"] = F(q + "dq.norm", Rq), F(q + "dkv.norm", R)
                L["wq"], L["qw"] = W(q + "uq", H * (D + Dr), Rq), D + Dr
                L["wuk"] = W(q + "uk", H * D, R).view(H, D, R).contiguous()
                L["wuv_t"] = W(q + "uv", H * Dv, R).view(H, Dv, R).transpose(1, 2).contiguous()
                L["sink"] = None
                L["cos_sin"] = self._table(m.rot)
                latent_prompt_layout(L, m, dtype, dev)
            wo = W(q + "o", d, H * Dv)
            if f is not None:
                parts.append(W(p + "mlp.up", f.ff, d))
                wout, (_, L["act_off"]) = stack_rows([wo.t(), W(p + "mlp.down", d, f.ff).t()])
                wo = wout.t().contiguous()             # [d, heads | pad | ff | pad]
            L["w_out"] = wo
            L["w_in"], L["offs"] = stack_rows(parts)
            self.layers.append(L)

    def _table(self, rot) -> torch.Tensor:
        key = (rot.dims, rot.base)
        if key not in self._tables:
            self._tables[key] = seqmix.rope_table_pairs(rot.dims, self.max_positions, rot.base,
                                                        None, self.device)
        return self._tables[key]

    @classmethod
    def random(cls, cfg: GopopelConfig, device, seed: int = 0, dtype=torch.bfloat16,
               max_positions: int = 8192) -> "GopopelWeights":
        return cls(cfg, random_state_dict(cfg, seed), device, dtype, max_positions)


def random_state_dict(cfg: GopopelConfig, seed: int = 0) -> dict:
    """Seeded random weights in checkpoint naming (bf16), scaled so that
    activations stay O(1) through the stack; used by tests, smoke and bench."""
    g = torch.Generator().manual_seed(seed)
    d = cfg.d_model
    sd: dict = {}

    def mat(name, rows, cols, gain=1.0):
        sd[name] = (torch.randn(rows, cols, generator=g) * gain / cols ** 0.5).to(torch.bfloat16)

    def vec(name, n, mean=0.0, std=0.1):
        sd[name] = (mean + torch.randn(n, generator=g) * std).to(torch.bfloat16)

    def scalar(name, lo, hi):
        sd[name] = torch.tensor(lo + (hi - lo) * torch.rand((), generator=g).item(),
                                dtype=torch.bfloat16)

    def norm(name):
        vec(name, d, 1.0)
        vec(name + ".b", d, 0.0, 0.05)
        scalar(name + ".alpha", 0.3, 0.8)

    sd["embed"] = torch.randn(cfg.vocab_size, d, generator=g).to(torch.bfloat16)
    for i, lc in enumerate(cfg.layers):
        p, m, f = f"l{i}.", lc.mixer, lc.mlp
        norm(p + "norm1")
        q, H, D, Dv = p + "mix.", m.heads, m.dim, m.vdim
        if lc.kind == "attention":
            G = m.kv_heads
            mat(q + "q", H * D, d, 2.0); mat(q + "k", G * D, d, 2.0); mat(q + "v", G * Dv, d, 2.0)
            vec(q + "q.norm", D, 1.0); vec(q + "k.norm", D, 1.0)
            if m.v_mix:
                scalar(q + "vmix", 0.2, 0.8)
            if m.sink:
                vec(q + "sink", H, 0.0, 1.0)
        else:
            Dr, R, Rq = m.rot_dim, m.kv_rank, m.q_rank
            mat(q + "dq", Rq, d, 2.0); vec(q + "dq.norm", Rq, 1.0)
            mat(q + "uq", H * (D + Dr), Rq, 2.0)
            mat(q + "dkv", R + Dr, d, 2.0); vec(q + "dkv.norm", R, 1.0)
            mat(q + "uk", H * D, R, 2.0); mat(q + "uv", H * Dv, R, 2.0)
            mat(q + "g", H * Dv, d, 2.0)
        mat(q + "o", d, H * Dv, 2.0)
        if f is not None:
            mat(p + "mlp.up", f.ff, d, 1.5)
            mat(p + "mlp.down", d, f.ff, 1.5)
    norm("final.norm")
    mat("head", cfg.vocab_size, d, 2.0)
    return sd


def config_to_json(cfg: GopopelConfig) -> dict:
    """The config.json of ``cfg`` (the inverse of ``gopopel_config_from_json``)."""
    layers = []
    for lc in cfg.layers:
        m, f = lc.mixer, lc.mlp
        mx = {"heads": m.heads, "dim": m.dim, "vdim": m.vdim, "scale": m.scale}
        if m.window:
            mx["mask"] = {"size": m.window}
        if lc.kind == "attention":
            mx.update(kv_heads=m.kv_heads, v_mix=m.v_mix)
        else:
            mx.update(rot_dim=m.rot_dim, kv_rank=m.kv_rank, q_rank=m.q_rank,
                      rot={"dims": m.rot.dims, "base": m.rot.base})
        layers.append({"type": lc.kind, "mixer": mx,
                       "mlp": None if f is None else {"kind": "dense", "ff": f.ff}})
    return {"architecture": "Gopopel", "vocab": cfg.vocab_size, "width": cfg.d_model,
            "norm": {"eps": cfg.norm_eps}, "embedding": {"scale": cfg.embed_scale},
            "layers": layers}


class GopopelModel:
    """The step function: one pass of a flat token batch through all layers,
    reading and extending the paged caches."""

    hybrid = True
    # a step whose longest feed has at least this many tokens takes the
    # matrix-core prompt path of latent attention (bf16 on the GPU)
    prompt_min_q = 32

    def __init__(self, w: GopopelWeights):
        self.w, self.cfg = w, w.cfg
        # windows the prompt path of latent attention gathers keys for
        self.key_windows = sorted({lc.mixer.window for lc, L in zip(w.cfg.layers, w.layers)
                                   if "prompt_sizes" in L and lc.mixer.window > 0})

    # the cache manager sizes its storage from this
    def cache_spec(self) -> dict:
        latent, kv = {}, {}
        for i, lc in enumerate(self.cfg.layers):
            m = lc.mixer
            if lc.kind == "attention":
                kv[i] = (m.kv_heads * m.dim, m.kv_heads * m.vdim)
            else:
                latent[i] = m.kv_rank + m.rot_dim
        return {"latent": latent, "state": {}, "kv_rows": kv}

    def embed(self, tokens: torch.Tensor) -> torch.Tensor:
        return torch.nn.functional.embedding(tokens.long(), self.w.embed)

    def forward(self, meta, cache, trail: list | None = None) -> torch.Tensor:
        """f32 logits [len(meta.logit_idx), vocab] of one step. ``meta``: the
        engine's StepMeta; ``cache``: a HybridCache. ``trail`` collects the
        residual stream after every layer (tests)."""
        w, cfg, dt = self.w, self.cfg, self.w.dtype
        x = self.embed(meta.tokens).contiguous()
        n = len(w.layers)
        h = seqmix.dyt_norm(x, w.layers[0]["norm1"], dt) if n else None
        v_first = None
        for i, (lc, L) in enumerate(zip(cfg.layers, w.layers)):
            m, f = lc.mixer, lc.mlp
            u = ops.linear(h, L["w_in"])
            # the side-by-side input of the output projection
            row = torch.empty(u.shape[0], L["w_out"].shape[1], dtype=dt, device=u.device)
            heads, side = row[:, :m.heads * m.vdim], None
            if f is not None:
                up = L["offs"][-1]
                side = SideCols(u[:, up:up + f.ff], row, L["act_off"], m.heads * m.vdim)
            if lc.kind == "attention":
                v = u[:, L["v_off"]:L["v_off"] + m.kv_heads * m.vdim]
                if i == cfg.first_v_mix:
                    v_first = v
                self._attention(i, m, L, u, v_first, side, heads, meta, cache)
            else:
                self._latent(i, m, L, u, side, heads, meta, cache)
            y = ops.linear(row, L["w_out"])
            h = seqmix.residual_dyt(x, [y], w.layers[i + 1]["norm1"] if i + 1 < n else None, dt)
            if trail is not None:
                trail.append(x.clone())
        hf = seqmix.dyt_norm(x, w.final_norm, torch.float32, row_idx=meta.logit_idx)
        return ops.linear(hf, w.head)

    def _attention(self, i, m, L, u, v_first, side, out, meta, cache) -> None:
        H, G, D, Dv = m.heads, m.kv_heads, m.dim, m.vdim
        kc, vc = cache.kv_rows[i]
        q = seqmix.qk_prep_append(u, H, G, D, Dv, L["v_off"], None, 0, self.cfg.norm_eps, None,
                                  meta.positions, kc, vc, meta.slots, self.w.dtype, L["q_norm"],
                                  L["k_norm"],
                                  v_mix=None if L["vmix"] is None else (v_first, L["vmix"]),
                                  side=side)
        seqmix.window_attention(q, kc, vc, meta.cu_q, meta.ctx_lens, meta.block_tables,
                                meta.positions, m.scale, 0.0, m.window, 0, None, H, G, D, Dv,
                                meta.max_q, max_ctx=meta.max_ctx, sink=L["sink"],
                                slopes=L["slopes"], out=out)

    def _latent(self, i, m, L, u, side, out, meta, cache) -> None:
        H, Dv, R, Dr = m.heads, m.vdim, m.kv_rank, m.rot_dim
        dq, dkv, g = L["offs"][:3]
        cq = seqmix.latent_inputs(u[:, dkv:dkv + R + Dr], L["dkv_norm"], self.cfg.norm_eps,
                                  meta.positions, L["cos_sin"], cache.latent[i], meta.slots, R,
                                  m.rot.dims, u[:, dq:dq + m.q_rank], L["dq_norm"], side)
        latent_heads(L, m, ops.linear(cq, L["wq"]), cache.latent[i], meta, self.prompt_min_q,
                     u[:, g:g + H * Dv], out)
