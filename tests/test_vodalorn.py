"""The Vodalorn family through the framework (registry, weights, engine step,
hybrid cache, scheduler) against the plain float64 oracle in
``vodalorn_oracle.py``. Every test builds its own small configuration and
seeded weights. The same tests run on the CPU (reference ops) and, marked
``gpu``, on the HIP kernels.
"""
import json
import math
import os
import subprocess
import sys

import numpy as np
import pytest
import torch

import vodalorn_oracle as O
from loqa_hub_amd.engine.llm_engine import GenRequest, LLMEngine
from loqa_hub_amd.models.configs import vodalorn_config_from_json
from loqa_hub_amd.models.registry import family_of, lm_config_from_json
from loqa_hub_amd.models.vilulix import _head_rows, _pairs_from_halves
from loqa_hub_amd.models.vodalorn import VodalornWeights, config_to_json, random_state_dict
from loqa_hub_amd.ops import seqmix

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
DEVICES = ["cpu", pytest.param("cuda", marks=pytest.mark.gpu)]
DTYPES = [torch.float32, torch.bfloat16]
TOL = {torch.float32: 2e-4, torch.bfloat16: 6e-2}
F64 = torch.float64


def engine(cfg_json, sd, device, dtype=torch.float32, max_tokens=256, block=16, max_seqs=4):
    cfg = lm_config_from_json(O.public(cfg_json), "t")
    w = VodalornWeights(cfg, sd, device, dtype, max_positions=max_tokens)
    return LLMEngine(cfg, device, weights=w, max_seqs=max_seqs, max_seq_len=max_tokens,
                     block_size=block, num_blocks=max_tokens // block, use_graphs=False, dtype=dtype)


def rel_err(got: torch.Tensor, want: torch.Tensor, q: float = 1.0) -> float:
    """RMS difference (mean removed per row) over the RMS of the wanted logits:
    the worst row, or the ``q`` quantile of the rows."""
    d = got.double().cpu() - want.double()
    d = d - d.mean(-1, keepdim=True)
    w = want - want.mean(-1, keepdim=True)
    return float((d.pow(2).mean(-1).sqrt() / w.pow(2).mean().sqrt()).quantile(q))


def feed(eng, seq, toks, cuts):
    """Feed ``toks`` to one sequence in portions of ``cuts`` sizes (cycled);
    returns the logits of every position."""
    out, i, k = [], 0, 0
    while i < len(toks):
        n = min(cuts[k % len(cuts)], len(toks) - i)
        out.append(eng.step_logits([seq], [toks[i:i + n]], [list(range(n))]))
        i, k = i + n, k + 1
    return torch.cat(out)


def tokens(n, vocab, seed):
    g = torch.Generator().manual_seed(seed)
    return torch.randint(0, vocab, (n,), generator=g).tolist()


def close(got, want, tol):
    assert (got.double().cpu() - want).abs().max() < tol * max(1.0, float(want.abs().max()))


# both mixers, both kinds of feed-forward and a layer without one, a repeated
# stretch that holds both mixers (so every pass needs pages, states and tails of
# its own), grouped and ungrouped heads, partial and full rotation
FULL = [(O.delta(), O.dense_ff()),
        (O.parallel(), O.moe_ff()),
        (O.delta(heads=2, kv_heads=2, dim=6, vdim=10, conv=2, decay_rank=3, gate_rank=4), None),
        (O.parallel(O.window(heads=2, kv_heads=2, dim=8, vdim=8, size=20, rot_dims=8),
                    O.retention(heads=2, dim=6, vdim=5, rot_dims=2)),
         O.moe_ff(ff=12, experts=5, top=3, groups=None, scale=1.0, limit=0.7)),
        (O.parallel(), O.dense_ff(24))]


@pytest.fixture(scope="module")
def full_model():
    cfg = O.make_config(FULL, loop=(0, 3, 2))
    return cfg, O.make_weights(cfg, 1)


def test_registry_reads_config(full_model):
    cfg_json = O.public(full_model[0])
    cfg = lm_config_from_json(json.loads(json.dumps(cfg_json)))
    assert family_of(cfg).name == "vodalorn" and family_of(cfg_json).hybrid
    assert cfg.n_layers == len(FULL) and cfg.layers[2].mlp is None and cfg.side_dim == 6
    a, r = cfg.layers[1].mixer.left, cfg.layers[1].mixer.right
    assert a.window == 7 and a.bias and a.qk_norm == "none" and a.rot.half and a.rot.dims == 8
    assert r.decay == (0.75, 0.875, 0.9375) and r.rot.base == 300.0 and cfg.residual_mult == 0.6
    assert cfg.layers[0].mixer.channel_decay and cfg.layers[0].mixer.taps == 4
    f = cfg.layers[1].mlp
    assert (f.groups, f.keep, f.top, f.limit, f.weight_scale, f.renorm) == (3, 2, 2, 1.1, 1.7, True)
    assert cfg.layers[3].mlp.groups == 1 and cfg.layers[0].mlp.act == "relu2"
    assert cfg.bigram.buckets == 37 and (cfg.bigram.mul_prev, cfg.bigram.mul_cur) == (31, 7)
    assert cfg.runs() == [(0, 0), (1, None), (2, None), (0, 1), (1, None), (2, None), (3, None),
                          (4, None)]
    back = config_to_json(cfg)
    assert vodalorn_config_from_json(json.loads(json.dumps(back)), cfg.name) == cfg
    assert back["loop"] == cfg_json["loop"] and back["embedding"] == cfg_json["embedding"]
    for li, path, val in ((1, ("mixer", "left", "kv_heads"), 3), (0, ("mixer", "kv_heads"), 3),
                          (1, ("mixer", "left", "rot", "dims"), 5),
                          (1, ("mixer", "right", "rot", "dims"), 10),
                          (1, ("mixer", "right", "decay"), [0.5]), (1, ("mixer", "left", "mask", "size"), 0),
                          (1, ("mlp", "router", "top"), 5), (1, ("mlp", "router", "experts"), 7),
                          (0, ("type",), "other")):
        bad = json.loads(json.dumps(cfg_json))
        m = bad["layers"][li]
        for k in path[:-1]:
            m = m[k]
        m[path[-1]] = val
        with pytest.raises(ValueError):
            vodalorn_config_from_json(bad)
    bad = json.loads(json.dumps(cfg_json))
    bad["loop"]["stop"] = 9
    with pytest.raises(ValueError):
        vodalorn_config_from_json(bad)
    sd = random_state_dict(cfg, 0)
    assert sd["l0.mix.v.conv"].shape == (24, 4) and sd["bigram"].shape == (38, 32)
    assert sd["side.embed"].shape == (50, 30) and "l2.norm2" not in sd


def test_weights_check_shapes(full_model):
    cfg_json, sd = full_model
    cfg = lm_config_from_json(O.public(cfg_json))
    for name in ("bigram", "side.embed", "loop.step", "loop.in", "l0.mix.a2", "l0.mix.g2",
                 "l1.mix.left.k.b", "l1.mix.right.g", "l1.mlp.e3.down", "l1.norm1.b", "l3.side.proj",
                 "l0.mix.dt_bias", "l0.mix.q.conv", "head"):
        bad = dict(sd)
        bad[name] = sd[name][:-1]
        with pytest.raises(ValueError):
            VodalornWeights(cfg, bad, "cpu")


# ------------------------------------------------------ each mechanism alone
def _meta(lens, starts, device):
    cu = torch.tensor([0] + lens).cumsum(0).to(torch.int32)
    pos = torch.cat([s + torch.arange(n) for n, s in zip(lens, starts)]).to(torch.int32)
    return cu.to(device), pos.to(device)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("d", [37, 40, 256, 1028, 4100])
def test_residual_step(device, d):
    """Plain and normed addends, the added vector, the layer norm, the copy (also
    into a column slice of a wider row) and the gather."""
    g = torch.Generator().manual_seed(d)
    eps, T = 1e-3, 9
    x = torch.randn(T, d, generator=g) + 3.0          # a mean that is not small
    x[2] *= 0.01
    ys = [torch.randn(T, d, generator=g) * s for s in (5.0, 0.1)]
    ys[0][4] = 1e-3                                    # eps decides this row's norm
    ws = [torch.randn(d, generator=g) for _ in range(2)]
    nw, nb, vec = (torch.randn(d, generator=g) for _ in range(3))
    ln = seqmix.LnParams(nw.to(device), nb.to(device))
    for ydt in DTYPES:
        for n, normed, withvec in ((0, 0, True), (1, 0, False), (1, 1, False), (2, 2, False),
                                   (2, 0, True), (2, 1, True)):
            adds = [(ys[i].to(ydt), ws[i] if i < normed else None) for i in range(n)]
            want = x.double() + (vec.double() if withvec else 0.0)
            for y, w in adds:
                want = want + 0.7 * (y.double() if w is None else O.over_rms(y.double(), eps) * w.double())
            dev_adds = [(y.to(device), None if w is None else w.to(device)) for y, w in adds]
            for odt in DTYPES:
                tol = 2e-5 if odt == torch.float32 else 2e-2
                for nxt in (ln, None):
                    r = x.to(device).clone()
                    wide = torch.full((T, 2 * d), 7.0, dtype=odt, device=device)
                    got = seqmix.residual_ln(r, dev_adds, 0.7, nxt, eps, wide[:, :d],
                                             vec.to(device) if withvec else None)
                    close(r, want, 2e-5)
                    close(got, want if nxt is None else
                          O.layer_norm(want, nw.double(), nb.double(), eps), tol)
                    assert (wide[:, d:] == 7.0).all()
    r = x.to(device).clone()
    assert seqmix.residual_ln(r, [(ys[0].to(device), None)], 1.0, None, eps, None) is None
    close(r, x.double() + ys[0].double(), 2e-5)
    rows = torch.tensor([5, 0, 0, 8], device=device)
    got = seqmix.residual_ln(x.to(device), [], 1.0, ln, eps, torch.empty(4, d, device=device),
                             row_idx=rows)
    close(got, O.layer_norm(x.double(), nw.double(), nb.double(), eps)[rows.cpu()], 2e-5)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("d", [12, 33])
def test_pair_embedding(device, dtype, d):
    """Three sequences in portions of changing size, a padding sequence and
    padding rows behind them; slots that held other tokens before; the row of a
    first token, multipliers that exceed 32 bits together with the token."""
    g = torch.Generator().manual_seed(3)
    V, P, mp, mc = 60, 41, 10 ** 9 + 7, 998244353
    sd = {"embed": torch.randn(V, d, generator=g).to(torch.bfloat16).float(),
          "bigram": torch.randn(P + 1, d, generator=g).to(torch.bfloat16).float()}
    cfg = {"embedding": {"bigram": {"buckets": P, "mul_prev": mp, "mul_cur": mc}}}
    seqs = [tokens(n, V, 70 + n) for n in (17, 5, 9)]
    want = [O.embedding({k: v.double() for k, v in sd.items()}, cfg, t) for t in seqs]
    dev = torch.device(device)
    prev = torch.full((5,), 55, dtype=torch.int32, device=dev)
    slots = torch.tensor([3, 0, 2, 4], dtype=torch.int32, device=dev)
    emb, big = sd["embed"].to(dev, dtype), sd["bigram"].to(dev, dtype)
    at, k = [0, 0, 0], 0
    while any(a < len(t) for a, t in zip(at, seqs)):
        feeds = [min((1, 4, 2, 0, 3)[(k + b) % 5], len(t) - a)
                 for b, (a, t) in enumerate(zip(at, seqs))]
        k += 1
        n = sum(feeds)
        if not n:
            continue
        cu = torch.tensor([0] + feeds + [0]).cumsum(0).to(torch.int32).to(dev)
        pos = torch.cat([a + torch.arange(f) for a, f in zip(at, feeds)] + [torch.zeros(2)])
        tk = [x for t, a, f in zip(seqs, at, feeds) for x in t[a:a + f]] + [0, 0]
        out2 = torch.zeros(n + 2, 2 * d, dtype=torch.bfloat16, device=dev)
        x = seqmix.bigram_embed(torch.tensor(tk, dtype=torch.int32, device=dev), emb, big, mp, mc,
                                prev, slots, cu, pos.to(torch.int32).to(dev), out2)
        ref = torch.cat([w[a:a + f] for w, a, f in zip(want, at, feeds)])
        close(x[:n], ref, 1e-6)
        assert torch.equal(out2[:n, :d].cpu(), x[:n].to(torch.bfloat16).cpu())
        assert torch.equal(out2[:, :d], out2[:, d:])
        at = [a + f for a, f in zip(at, feeds)]
    assert prev.tolist() == [seqs[1][-1], 55, seqs[2][-1], seqs[0][-1], 55]


@pytest.mark.parametrize("device", DEVICES)
def test_token_gate_and_squared_relu(device):
    g = torch.Generator().manual_seed(4)
    z = torch.randn(7, 11, generator=g) * 3
    tab = torch.randn(20, 30, generator=g)
    tk = torch.tensor([0, 19, 3, 3, 7, 1, 18], dtype=torch.int32)
    for dt in DTYPES:
        for tdt in DTYPES:
            zz, tt = z.to(dt), tab.to(tdt)
            got = seqmix.token_gate(zz.to(device)[:, 2:9], tt.to(device), tk.to(device), 23)
            want = O.gelu_tanh(zz[:, 2:9].double()) * tt.double()[tk.long(), 23:]
            close(got, want, 1e-5 if dt == torch.float32 else 1e-2)
        for n in (44, 7):
            v = z.reshape(-1)[:n].reshape(1, n).to(dt)
            close(seqmix.relu2_(v.to(device).clone()), torch.relu(v.double()) ** 2,
                  1e-6 if dt == torch.float32 else 1e-2)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("H,G,D,Dv,dims", [(4, 2, 16, 24, 8), (3, 1, 24, 8, 0), (2, 2, 6, 6, 6),
                                           (5, 5, 64, 32, 16), (1, 1, 130, 9, 2), (2, 1, 7, 5, 4)])
def test_rotation_without_norm(device, H, G, D, Dv, dims):
    """q | k | v rows -> rotate-half rotation through the load-time row
    permutation, no norm, and the paged append."""
    g = torch.Generator().manual_seed(5)
    T, blk, base = 40, 4, 50.0
    u = torch.randn(T, (H + G) * D + G * Dv + 3, generator=g)
    pos = torch.arange(T, dtype=torch.int32)
    slots = torch.randperm(48, generator=g)[:T].to(torch.int32)
    slots[8] = -1
    wq = O.rotate_halves(u[:, :H * D].double().view(T, H, D), dims, base)
    wk = O.rotate_halves(u[:, H * D:(H + G) * D].double().reshape(T, G, D), dims, base)
    per = _pairs_from_halves(dims, D)
    iq, ik = _head_rows(H, D, 0, per), _head_rows(G, D, 0, per)
    up = torch.cat([u[:, :H * D][:, iq], u[:, H * D:(H + G) * D][:, ik], u[:, (H + G) * D:]], 1)
    cs = seqmix.rope_table_pairs(dims, 40, base, None, device) if dims else None
    kc = torch.zeros(12, blk, G * D, device=device)
    vc = torch.zeros(12, blk, G * Dv, device=device)
    q = seqmix.qk_prep_append(up.to(device), H, G, D, Dv, (H + G) * D, cs, dims, 1e-4, None,
                              pos.to(device), kc, vc, slots.to(device), torch.float32, norm=False)
    close(q.view(T, H, D), wq[:, :, per], 1e-5)
    ok = slots >= 0
    close(kc.view(-1, G, D)[slots[ok].long()], wk[ok][:, :, per], 1e-5)
    assert torch.equal(vc.view(-1, G * Dv)[slots[ok].long()].cpu(),
                       u[ok][:, (H + G) * D:(H + G) * D + G * Dv])


def _paged(k, v, lens, blk, device, seed=0):
    nb = sum(-(-n // blk) for n in lens) + 2
    perm = torch.randperm(nb, generator=torch.Generator().manual_seed(seed)).tolist()
    kc = torch.full((nb, blk, k[0].shape[1]), 7.0)
    vc = torch.full((nb, blk, v[0].shape[1]), 7.0)
    bt = torch.zeros(len(lens), max(-(-n // blk) for n in lens), dtype=torch.int32)
    for b, n in enumerate(lens):
        for j in range(-(-n // blk)):
            page = perm.pop()
            bt[b, j] = page
            m = min(blk, n - j * blk)
            kc[page, :m] = k[b][j * blk:j * blk + m]
            vc[page, :m] = v[b][j * blk:j * blk + m]
    return kc.to(device), vc.to(device), bt.to(device)


def _window_case(device, dtype, H, G, D, Dv, window, lens, feeds, mfma=None, spike=None, seed=2):
    """Sequences of ``lens`` keys whose last ``feeds`` positions are this step's
    queries. ``spike`` = (distance back, strength): the key that far behind each
    query gets a large score."""
    g = torch.Generator().manual_seed(seed)
    B = len(lens)
    ks = [torch.randn(n, G * D, generator=g).to(dtype).float() for n in lens]
    vs = [torch.randn(n, G * Dv, generator=g).to(dtype).float() for n in lens]
    qs = [torch.randn(n, H * D, generator=g) for n in lens]
    if spike is not None:
        back, strength = spike
        for b, n in enumerate(lens):
            for i in range(back, n):
                kk = ks[b][i - back].view(G, D)
                qs[b][i] = (kk.repeat_interleave(H // G, 0) * strength / D).reshape(-1)
    qs = [q.to(dtype).float() for q in qs]
    kc, vc, bt = _paged(ks, vs, lens, 16, device, seed)
    starts = [n - f for n, f in zip(lens, feeds)]
    cu, pos = _meta(feeds, starts, device)
    q = torch.cat([qs[b][starts[b]:] for b in range(B)])
    ctx = torch.tensor(lens, dtype=torch.int32, device=device)
    scale = 1.0 / math.sqrt(D)
    got = seqmix.window_attention(q.to(device, dtype), kc.to(dtype), vc.to(dtype), cu, ctx, bt, pos,
                                  scale, 0.0, window, 0, None, H, G, D, Dv, max(feeds),
                                  matrix_cores=mfma, max_ctx=max(lens))
    want = []
    for b, n in enumerate(lens):
        o = O.window_softmax(qs[b].double().view(n, H, D), ks[b].double().view(n, G, D),
                             vs[b].double().view(n, G, Dv), scale, window)
        want.append(o[starts[b]:].reshape(-1, H * Dv))
    return got.cpu().double(), torch.cat(want)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("H,G,D,Dv,window", [(4, 2, 16, 48, 5), (3, 3, 8, 24, 64), (6, 1, 64, 256, 37),
                                             (9, 1, 24, 8, 100), (2, 2, 6, 130, 1),
                                             (16, 1, 16, 512, 40)])
def test_window_attention(device, H, G, D, Dv, window):
    got, want = _window_case(device, torch.float32, H, G, D, Dv, window, [150, 1, 37, 90],
                             [150, 1, 1, 23])
    assert (got - want).abs().max() < 2e-5


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("back", [0, 1, 4, 5, 6, 63, 64, 65, 127, 128, 129])
def test_window_edges(device, back):
    """A key ``back`` positions behind every query carries almost all of the
    softmax weight if it is visible: windows of 5, 64 and 128 keys, in a prompt
    portion and in single tokens, with values wider than keys."""
    for size in (5, 64, 128):
        for feeds in ([300], [1]):
            got, want = _window_case(device, torch.float32, 2, 1, 16, 32, size, [300], feeds,
                                     spike=(back, 40.0))
            assert (got - want).abs().max() < 2e-5, (size, feeds)


@pytest.mark.gpu
@pytest.mark.parametrize("H,G,D,Dv,window", [(4, 2, 128, 256, 48), (6, 2, 64, 160, 200), (2, 1, 256, 256, 70),
                                             (3, 3, 200, 136, 33), (8, 1, 128, 256, 1000),
                                             (2, 1, 64, 512, 90), (2, 2, 40, 328, 64)])
def test_wide_values_on_matrix_cores(H, G, D, Dv, window):
    """The prompt-portion kernel with more than 128 value entries against the
    oracle and against the keys-parallel form."""
    lens, feeds = [700, 1, 333, 90, 450], [700, 1, 70, 17, 1]
    a, want = _window_case("cuda", torch.bfloat16, H, G, D, Dv, window, lens, feeds, mfma=True)
    b, _ = _window_case("cuda", torch.bfloat16, H, G, D, Dv, window, lens, feeds, mfma=False)
    scale = float(want.abs().max())
    assert (a - want).abs().max() < 0.03 * scale and (b - want).abs().max() < 0.03 * scale


@pytest.mark.gpu
@pytest.mark.parametrize("back", [0, 31, 63, 64, 65, 127, 128])
def test_wide_value_window_edges_on_matrix_cores(back):
    for size in (64, 128):
        a, want = _window_case("cuda", torch.bfloat16, 2, 1, 128, 256, size, [300], [300], mfma=True,
                               spike=(back, 60.0))
        assert (a - want).abs().max() < 0.03 * float(want.abs().max()), size


class Portions:
    """Unequal sequences fed together in portions of changing size, with slots
    that hold junk: yields (rows of each feed, cu_q, positions)."""

    def __init__(self, lens, cuts, device):
        self.lens, self.cuts, self.dev = list(lens), cuts, device
        self.slots = torch.tensor([2, 0, 1][:len(lens)], dtype=torch.int32, device=device)

    def __iter__(self):
        at, k = [0] * len(self.lens), 0
        while any(a < n for a, n in zip(at, self.lens)):
            feeds = [min(self.cuts[(k + b) % len(self.cuts)], n - a)
                     for b, (a, n) in enumerate(zip(at, self.lens))]
            cu, pos = _meta(feeds, at, self.dev)
            yield [(a, a + f) for a, f in zip(at, feeds)], cu, pos
            at = [a + f for a, f in zip(at, feeds)]
            k += 1


def _split(y, spans, got):
    o = 0
    for b, (a, e) in enumerate(spans):
        got[b].append(y[o:o + e - a])
        o += e - a


def _retention_case(device, m, cuts, dtype=torch.float32, seed=3, lens=(37, 1, 9)):
    """The retention mixer's ops in the model's order against the oracle's mixer
    on the whole sequences."""
    H, D, Dv, rot = m["heads"], m["dim"], m["vdim"], m["rot"]
    d = 24
    g = torch.Generator().manual_seed(seed)
    cfg = O.make_config([(O.parallel(O.window(), m), None)], width=d)
    sd = O.make_weights(cfg, seed)
    hs = [torch.randn(n, d, generator=g).to(dtype).float() for n in lens]
    p = "l0.mix.right."
    want = [O.mixer_retention({k: v.double() for k, v in sd.items()}, p, m, h.double(), 1e-5)
            for h in hs]
    dev = torch.device(device)
    ih = _head_rows(H, D, 0, _pairs_from_halves(rot["dims"], D))
    w_in = torch.cat([sd[p + "q"][ih], sd[p + "k"][ih], sd[p + "v"], sd[p + "g"]]).to(dev, dtype)
    n = 2 * H * D + H * Dv
    cs = seqmix.rope_table_pairs(rot["dims"], max(lens), rot["base"], None, dev) if rot["dims"] else None
    state = torch.full((len(lens) + 1, H, D, Dv), 9.0, device=dev)
    decay = torch.tensor(m["decay"], dtype=torch.float32, device=dev)
    por = Portions(lens, cuts, dev)
    got = [[] for _ in lens]
    for spans, cu, pos in por:
        h = torch.cat([hs[b][a:e] for b, (a, e) in enumerate(spans)]).to(dev, dtype)
        u = torch.nn.functional.linear(h, w_in)
        act = seqmix.retention_prep(u[:, :n], H, D, Dv, cs, rot["dims"], pos)
        o = seqmix.state_scan(act, H, D, Dv, 0, H * D, 2 * H * D, 1, state, por.slots, cu, pos,
                              decay=decay)
        y = seqmix.gated_rmsnorm(o, torch.ones(H * Dv, device=dev), u[:, n:], 1e-5, torch.float32,
                                 groups=H, gate_act="silu")
        _split(y.cpu().double() @ sd[p + "o"].double().T, spans, got)
    return [torch.cat(x) for x in got], want


CUTS = [[37], [1], [2, 1, 3, 17, 1, 13]]


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("cuts", CUTS, ids=lambda c: str(len(c)))
@pytest.mark.parametrize("m", [O.retention(), O.retention(1, 5, 3, 2, decay=[1.0]),
                               O.retention(2, 64, 128, 64),
                               O.retention(2, 72, 31, 0, decay=[0.0, 0.99]),
                               O.retention(4, 16, 8, 16)], ids=lambda m: f"{m['dim']}x{m['vdim']}")
def test_retention_mixer(device, m, cuts):
    got, want = _retention_case(device, m, cuts)
    for a, b in zip(got, want):
        close(a, b, 3e-4)


@pytest.mark.gpu
@pytest.mark.parametrize("H,hpg,D,Dv,decay", [
    (3, 1, 8, 10, [0.0, 0.9, 1.0]), (2, 2, 128, 64, [0.97, 0.9995]), (4, 2, 36, 130, [0.5, 0.99, 0.9, 1.0]),
    (1, 1, 5, 3, [0.93]), (2, 1, 256, 33, [0.99, 0.2]), (1, 1, 72, 256, [0.999])])
@pytest.mark.parametrize("starts", [(0, 0, 0, 0, 0), (77, 1, 0, 64, 300)])
def test_chunked_recurrence(H, hpg, D, Dv, decay, starts):
    """The chunked form on feeds that end on, before and after a chunk's edge (one
    of them empty, one a single token), from a fresh and from a carried state,
    against the oracle and the token-by-token kernel; then both go on one token."""
    lens = (200, 1, 0, 128, 65)
    B, T, G = len(lens), sum(lens), H // hpg
    g = torch.Generator().manual_seed(D)
    q, k = (torch.randn(T, G, D, generator=g) for _ in range(2))
    v = torch.randn(T, H, Dv, generator=g)
    act = torch.cat([q.reshape(T, -1), torch.zeros(T, 4), k.reshape(T, -1), v.reshape(T, -1)], 1).cuda()
    ko = G * D + 4
    vo = ko + G * D
    cu, pos = _meta(list(lens), list(starts), "cuda")
    slots = torch.tensor([4, 0, 5, 2, 1], dtype=torch.int32, device="cuda")
    state0 = torch.randn(7, H, D, Dv, generator=g)
    lam = torch.tensor(decay, device="cuda")
    one = torch.randn(B, act.shape[1], generator=g).cuda()
    outs = []
    for chunked in (True, False):
        st = state0.cuda()
        o = seqmix.state_scan(act, H, D, Dv, 0, ko, vo, hpg, st, slots, cu, pos, decay=lam,
                              chunked=chunked)
        cu1, pos1 = _meta([1] * B, [s + n for s, n in zip(starts, lens)], "cuda")
        o1 = seqmix.state_scan(one, H, D, Dv, 0, ko, vo, hpg, st, slots, cu1, pos1, decay=lam,
                               chunked=chunked)
        outs.append((o, o1, st))
    a, b = outs
    for x, y in zip(a, b):
        close(x, y.double().cpu(), 2e-5)
    o0 = 0
    for b_, n in enumerate(lens):
        S0 = torch.zeros(H, D, Dv, dtype=F64) if starts[b_] == 0 else \
            state0[int(slots[b_])].double()
        want = O.retention_scan(q[o0:o0 + n].repeat_interleave(hpg, 1).double(),
                                k[o0:o0 + n].repeat_interleave(hpg, 1).double(),
                                v[o0:o0 + n].double(), decay)
        for t in range(n):
            for h in range(H):
                want[t, h] += decay[h] ** (t + 1) * (S0[h].T @ q[o0 + t, h // hpg].double())
        close(a[0][o0:o0 + n].view(n, H, Dv), want, 2e-5) if n else None
        o0 += n


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", DTYPES)
def test_long_prompt_takes_the_chunked_form(dtype):
    """A model whose prompts are long enough for the chunked recurrences."""
    layers = [(O.delta(heads=4, kv_heads=2, dim=20, vdim=12), None),
              (O.parallel(O.window(size=30), O.retention(heads=2, dim=16, vdim=24, rot_dims=16,
                                                         decay=[0.97, 0.998])), O.dense_ff())]
    cfg = O.make_config(layers, loop=(0, 2, 2))
    sd = O.make_weights(cfg, 15)
    toks = tokens(330, cfg["vocab"], 22)
    want = O.forward(cfg, sd, toks)
    eng = engine(cfg, sd, "cuda", dtype, max_tokens=336)
    for cuts in ([330], [150, 1, 2, 140], [129, 1, 1, 200]):
        s = eng.open_sequence()
        got = feed(eng, s, toks, cuts)
        eng.close_sequence(s)
        assert rel_err(got, want, 1.0 if dtype == torch.float32 else 0.9) < 2 * TOL[dtype], cuts


@pytest.mark.parametrize("device", DEVICES)
def test_retention_remembers_one_far_key(device):
    """A single key written hundreds of tokens ago, every other key orthogonal to
    the query: the read-out is that value times the decay to the distance."""
    D, Dv, T = 8, 4, 400
    dev = torch.device(device)
    q, k, v = torch.zeros(T, D), torch.zeros(T, D), torch.randn(T, Dv)
    q[:, 2] = 1.0
    k[:, 5] = 1.0
    k[3] = 0.0
    k[3, 2] = 1.0
    lam = 0.998
    state = torch.full((2, 1, D, Dv), 5.0, device=dev)
    slot = torch.tensor([1], dtype=torch.int32, device=dev)
    got, at = [], 0
    for n in (130, 2, 1, 200, 67):
        cu, pos = _meta([n], [at], dev)
        act = torch.cat([q, k, v], 1)[at:at + n].to(dev).contiguous()
        got.append(seqmix.state_scan(act, 1, D, Dv, 0, D, 2 * D, 1, state, slot, cu, pos,
                                     decay=torch.tensor([lam], device=dev)))
        at += n
    want = torch.zeros(T, Dv, dtype=F64)
    for t in range(3, T):
        want[t] = v[3].double() * lam ** (t - 3)
    close(torch.cat(got), want, 1e-4)


def _delta_case(device, m, cuts, dtype=torch.float32, seed=4, lens=(37, 1, 9)):
    H, G, D, Dv, K = m["heads"], m["kv_heads"], m["dim"], m["vdim"], m["conv"]
    d = 24
    g = torch.Generator().manual_seed(seed)
    cfg = O.make_config([(("channel_delta", m), None)], width=d)
    sd = O.make_weights(cfg, seed)
    hs = [torch.randn(n, d, generator=g).to(dtype).float() for n in lens]
    p = "l0.mix."
    want = [O.mixer_channel_delta({k: v.double() for k, v in sd.items()}, "l0.", m, h.double(), 1e-5)
            for h in hs]
    dev = torch.device(device)
    C = 2 * G * D + H * Dv
    w_in = torch.cat([sd[p + n] for n in "qkvb"]).to(dev, dtype)
    conv = torch.cat([sd[p + n + ".conv"] for n in "qkv"]).t().contiguous().to(dev)
    state = torch.full((len(lens) + 1, H, Dv, D), 9.0, device=dev)
    tail = torch.full((len(lens) + 1, K - 1, C), -7.0, device=dev)
    a_neg = -torch.exp(sd[p + "A_log"]).to(dev)
    por = Portions(lens, cuts, dev)
    got = [[] for _ in lens]
    for spans, cu, pos in por:
        h = torch.cat([hs[b][a:e] for b, (a, e) in enumerate(spans)]).to(dev, dtype)
        u = torch.nn.functional.linear(h, w_in)
        hf = h.float()
        za = hf @ sd[p + "a1"].to(dev).T @ sd[p + "a2"].to(dev).T
        gate = hf @ sd[p + "g1"].to(dev).T @ sd[p + "g2"].to(dev).T
        act, tok = seqmix.delta_prep(u, None, G, D, H, Dv, conv, tail, a_neg,
                                     sd[p + "dt_bias"].to(dev), por.slots, cu, pos, chan=(za, C))
        if K > 1:
            seqmix.seq_state_save(None, u, None, tail, por.slots, cu, pos)
        o = seqmix.delta_scan(act, H, D, Dv, 0, G * D, 2 * G * D, H // G, state, por.slots, cu, pos,
                              tok, g_off=C)
        y = seqmix.gated_rmsnorm(o, sd[p + "norm"].repeat(H).to(dev), gate, 1e-5, torch.float32,
                                 groups=H)
        _split(y.cpu().double() @ sd[p + "o"].double().T, spans, got)
    return [torch.cat(x) for x in got], want


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("cuts", CUTS, ids=lambda c: str(len(c)))
@pytest.mark.parametrize("m", [O.delta()[1], O.delta(3, 1, 5, 3, 1)[1], O.delta(4, 2, 128, 64, 4)[1],
                               O.delta(2, 2, 72, 33, 2)[1], O.delta(1, 1, 200, 8, 3)[1],
                               O.delta(2, 1, 160, 24, 2)[1]], ids=lambda m: f"{m['dim']}x{m['vdim']}")
def test_channel_delta_mixer(device, m, cuts):
    got, want = _delta_case(device, m, cuts)
    for a, b in zip(got, want):
        close(a, b, 3e-4)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("G,D,H,Dv,K", [(2, 128, 4, 64, 4), (1, 16, 3, 8, 2), (3, 64, 3, 40, 3),
                                        (1, 512, 1, 8, 1), (2, 24, 2, 12, 3)])
def test_delta_inputs_with_channel_decays_bf16(device, G, D, H, Dv, K):
    """The input stage on 16-bit rows (the vectorised form where a head is a
    power-of-two number of 16-byte runs), whole and in portions with the tail."""
    dev = torch.device(device)
    g = torch.Generator().manual_seed(6)
    C, T = 2 * G * D + H * Dv, 21
    W = C + 8 + (-C) % 8
    u = torch.randn(T, W, generator=g).to(torch.bfloat16)
    za = torch.randn(T, H * D, generator=g) * 3
    conv = torch.randn(C, K, generator=g) * 0.6
    a_neg, dtb = -torch.rand(H, generator=g), torch.randn(H * D, generator=g)
    y = O.silu(O.short_conv(u[:, :C].double(), conv.double()))
    q = O.unit(y[:, :G * D].reshape(T, G, D)) / math.sqrt(D)
    k = O.unit(y[:, G * D:2 * G * D].reshape(T, G, D))
    dec = torch.exp(a_neg.double()[:, None] * O.softplus(za.double() + dtb.double()).view(T, H, D))
    want = torch.cat([q.reshape(T, -1), k.reshape(T, -1), y[:, 2 * G * D:], dec.reshape(T, -1)], 1)
    beta = torch.sigmoid(u[:, C:C + H].double())
    tail = torch.full((2, K - 1, C), 5.0, device=dev)
    slots = torch.tensor([1], dtype=torch.int32, device=dev)
    at = 0
    for n in (T,) if K == 1 else (9, 1, 2, 9):
        cu, pos = _meta([n], [at], dev)
        uu = u[at:at + n].to(dev)
        act, tok = seqmix.delta_prep(uu, None, G, D, H, Dv, conv.t().contiguous().to(dev), tail,
                                     a_neg.to(dev), dtb.to(dev), slots, cu, pos,
                                     chan=(za[at:at + n].to(dev), C))
        if K > 1:
            seqmix.seq_state_save(None, uu, None, tail, slots, cu, pos)
        assert (act.cpu().double() - want[at:at + n]).abs().max() < 2e-5
        assert (tok[:, :, 1].cpu().double() - beta[at:at + n]).abs().max() < 1e-5
        at += n


@pytest.mark.gpu
@pytest.mark.parametrize("chan", [True, False])
@pytest.mark.parametrize("H,hpg,D,Dv", [(3, 1, 8, 10), (4, 2, 128, 64), (2, 2, 36, 33), (1, 1, 5, 3),
                                        (2, 1, 200, 40), (1, 1, 256, 16), (2, 1, 64, 128)])
@pytest.mark.parametrize("starts", [(0, 0, 0, 0, 0), (77, 1, 0, 64, 300)])
def test_chunked_delta_rule(chan, H, hpg, D, Dv, starts):
    """The chunked form on feeds that end on, before and after a chunk's edge (one
    of them empty, one a single token), from a fresh and from a carried state,
    against the oracle; decays of 0, of almost 0 and of 1 among them, write
    strengths up to 1, one key repeated many times."""
    lens = (70, 1, 0, 32, 17)
    B, T, G = len(lens), sum(lens), H // hpg
    g = torch.Generator().manual_seed(D + chan)
    q, k = (torch.randn(T, G, D, generator=g) for _ in range(2))
    k[20:31] = k[20]
    q, k = q / q.norm(dim=-1, keepdim=True), k / k.norm(dim=-1, keepdim=True)
    v = torch.randn(T, H, Dv, generator=g)
    dec = torch.rand(T, H, D, generator=g) ** 0.1
    dec[:, :, 0], dec[::7, :, 1] = 1.0, 0.0
    dec[::3, :, 2] = 1e-30
    beta = torch.rand(T, H, generator=g)
    beta[20:31] = 1.0
    if not chan:
        dec = dec[:, :, 3:4].expand(T, H, D).contiguous()
        dec[40], dec[45] = 0.0, 1e-30
    act = torch.cat([q.reshape(T, -1), k.reshape(T, -1), torch.zeros(T, 3), v.reshape(T, -1)] +
                    ([dec.reshape(T, -1)] if chan else []), 1).cuda()
    vo = 2 * G * D + 3
    go = vo + H * Dv if chan else None
    tok = torch.stack([torch.full((T, H), 7.0) if chan else dec[:, :, 0], beta], -1).cuda()
    cu, pos = _meta(list(lens), list(starts), "cuda")
    slots = torch.tensor([4, 0, 5, 2, 1], dtype=torch.int32, device="cuda")
    state0 = torch.randn(7, H, Dv, D, generator=g) * 0.5
    outs = []
    for chunked in (True, False):
        st = state0.cuda()
        outs.append((seqmix.delta_scan(act, H, D, Dv, 0, G * D, vo, hpg, st, slots, cu, pos, tok,
                                       g_off=go, chunked=chunked), st))
    for x, y in zip(*outs):
        close(x, y.double().cpu(), 3e-5)
    o0 = 0
    rep = lambda x: x.repeat_interleave(hpg, 1)
    for b, n in enumerate(lens):
        if not n:
            continue
        sl = slice(o0, o0 + n)
        o0 += n
        S = torch.zeros(H, D, Dv, dtype=F64) if starts[b] == 0 else \
            state0[int(slots[b])].transpose(1, 2).double()
        want = torch.zeros(n, H, Dv, dtype=F64)
        for t in range(n):
            kt, qt = rep(k)[sl][t].double(), rep(q)[sl][t].double()
            S = S * dec[sl][t].double()[:, :, None]
            u = beta[sl][t].double()[:, None] * (v[sl][t].double() - torch.einsum("hde,hd->he", S, kt))
            S = S + kt[:, :, None] * u[:, None, :]
            want[t] = torch.einsum("hde,hd->he", S, qt)
        close(outs[0][0][sl].view(n, H, Dv), want, 3e-5)
        close(outs[0][1][int(slots[b])].transpose(1, 2), S, 3e-5)


@pytest.mark.parametrize("device", DEVICES)
def test_decay_acts_on_its_own_key_channel(device):
    """Two keys on different channels; one channel forgets at once, the other
    keeps everything. The decay comes before the write and the read-out sees the
    current token's write."""
    dev = torch.device(device)
    D, Dv, T = 8, 4, 3
    k, q, v = torch.zeros(T, D), torch.zeros(T, D), torch.randn(T, Dv)
    k[0, 1] = k[1, 5] = k[2, 6] = 1.0
    q[0, 1] = 1.0
    q[1, 1] = q[1, 5] = 1.0
    q[2, 1], q[2, 5], q[2, 6] = 1.0, 10.0, 100.0
    gd = torch.ones(T, D)
    gd[:, 5] = 0.0
    act = torch.cat([q, k, v, gd], 1).to(dev)
    tok = torch.ones(T, 1, 2, device=dev)
    state = torch.zeros(2, 1, Dv, D, device=dev)
    cu, pos = _meta([T], [0], dev)
    o = seqmix.delta_scan(act, 1, D, Dv, 0, D, 2 * D, 1, state,
                          torch.tensor([0], dtype=torch.int32, device=dev), cu, pos, tok,
                          g_off=2 * D + Dv)
    want = torch.stack([v[0], v[0] + v[1], v[0] + 100.0 * v[2]]).double()
    close(o, want, 1e-6)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("E,groups,keep,top,scale", [(12, 4, 2, 3, 2.0), (6, 1, 1, 2, 1.0), (8, 8, 3, 3, 0.5),
                                                     (5, 1, 1, 5, 1.3), (64, 4, 1, 1, 2.5)])
def test_router(device, E, groups, keep, top, scale):
    f = O.moe_ff(experts=E, top=top, groups=groups, keep=keep, scale=scale)
    z = torch.randn(30, E, generator=torch.Generator().manual_seed(E)) * 2
    z[3] -= 60.0
    z[4] = -80.0
    z[4, E // 2] = 40.0            # one score takes everything
    idx, wt = seqmix.moe_route(z.to(device), None, groups, keep, top, renorm=True, weight_scale=scale)
    for t in range(30):
        want = dict(O.route(z[t].double(), f))
        if t == 4:                 # the others underflow: their order is open
            assert int(idx[t, 0]) == E // 2 and abs(float(wt[t, 0]) - scale) < 1e-5
            continue
        got = dict(zip(idx[t].tolist(), wt[t].tolist()))
        assert set(got) == set(want) and all(abs(got[e] - want[e]) < 1e-5 for e in want)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("T,d,ff,E,top", [(37, 32, 40, 6, 2), (3, 24, 20, 5, 5), (2, 64, 8, 3, 1),
                                           (400, 64, 96, 4, 3)])
def test_clamped_experts(device, dtype, T, d, ff, E, top):
    """Gate and up products beyond the limit on both sides."""
    g = torch.Generator().manual_seed(T)
    f = O.moe_ff(ff=ff, experts=E, top=top, groups=None, limit=0.9)
    cfg = O.make_config([(O.delta(), f)], width=d)
    sd = O.make_weights(cfg, 5)
    h = torch.randn(T, d, generator=g).to(dtype)
    want = O.ff_moe({k: v.double() for k, v in sd.items()}, "l0.", f, h.double())
    gu = torch.stack([torch.cat([sd[f"l0.mlp.e{e}.gate"], sd[f"l0.mlp.e{e}.up"]]) for e in range(E)])
    dn = torch.stack([sd[f"l0.mlp.e{e}.down"] for e in range(E)])
    z = h.float() @ sd["l0.mlp.router"].T
    idx, wt = seqmix.moe_route(z.to(device), None, 1, 1, top, renorm=True,
                               weight_scale=f["router"]["scale"])
    got = seqmix.moe_experts(h.to(device), idx, wt, gu.to(device, dtype).contiguous(),
                             dn.to(device, dtype).contiguous(), limit=0.9)
    close(got, want, 2e-5 if dtype == torch.float32 else 2e-2)


# --------------------------------------------------------- the whole model
@pytest.mark.parametrize("device", DEVICES)
def test_residual_after_every_layer_run(device, full_model):
    cfg, sd = full_model
    toks = tokens(29, cfg["vocab"], 10)
    want = []
    O.forward(cfg, sd, toks, want)
    eng = engine(cfg, sd, device)
    max_q, max_ctx, host = eng._meta([eng.open_sequence()], [toks], decode=False)
    host["logit_idx"] = np.asarray([0], np.int64)
    meta = eng._build_meta(eng._to_device(host), max_q, max_ctx, False)
    got = []
    eng.model.forward(meta, eng.kv, got)
    assert len(got) == len(want) == 8
    for r, (a, b) in enumerate(zip(got, want)):
        assert (a.cpu().double() - b).abs().max() < 2e-4 * float(b.abs().max()), r


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
def test_whole_prompt(device, dtype, full_model):
    cfg, sd = full_model
    toks = tokens(70, cfg["vocab"], 11)
    want = O.forward(cfg, sd, toks)
    eng = engine(cfg, sd, device, dtype)
    got = eng.step_logits([eng.open_sequence()], [toks], [list(range(len(toks)))])
    if dtype == torch.float32:
        assert rel_err(got, want) < TOL[dtype]
    else:
        # a width this small averages little of the 16-bit rounding away, and a
        # close call of the router may go the other way: the typical row is pinned
        assert rel_err(got, want, 0.5) < TOL[dtype] and rel_err(got, want, 0.9) < 0.25


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("cuts", [[1], [2], [3, 2, 7], [16], [17, 1, 1, 30], [5, 64]],
                         ids=lambda c: "x".join(map(str, c)))
def test_portions_and_decode(device, cuts, full_model):
    """Token-by-token decoding and portions of any size (down to two tokens,
    shorter than the convolutions, across page borders at 16 and window edges
    at 7 and 20) give the whole prompt's logits."""
    cfg, sd = full_model
    toks = tokens(53, cfg["vocab"], 12)
    want = O.forward(cfg, sd, toks)
    eng = engine(cfg, sd, device)
    got = feed(eng, eng.open_sequence(), toks, cuts)
    assert rel_err(got, want) < TOL[torch.float32]


@pytest.mark.gpu
def test_two_streams_match_one(full_model):
    """A step long enough for the second stream gives the bits of one stream."""
    cfg, sd = full_model
    toks = tokens(180, cfg["vocab"], 19)
    for dtype in DTYPES:
        out = []
        for least in (1, 10 ** 9):
            eng = engine(cfg, sd, "cuda", dtype)
            eng.model.overlap_min_tokens = least
            s = eng.open_sequence()
            out.append(feed(eng, s, toks, [150, 1, 2]))
        assert torch.equal(out[0], out[1])


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
def test_unequal_batch_and_reuse(device, dtype, full_model):
    """Four unequal requests, portions beside single tokens in one step; requests
    end early and new ones take over their pages and state slots; one sits out
    some steps. Every request's logits equal the ones it gets alone (oracle)."""
    cfg, sd = full_model
    V = cfg["vocab"]
    reqs = {n: tokens(L, V, 20 + i) for i, (n, L) in
            enumerate([("a", 41), ("b", 1), ("c", 18), ("d", 33), ("e", 25), ("f", 47)])}
    want = {n: O.forward(cfg, sd, t) for n, t in reqs.items()}
    eng = engine(cfg, sd, device, dtype, max_tokens=192, max_seqs=4)
    plan = {"a": [7, 1, 0, 1, 16, 2, 1, 0, 0, 13], "b": [1], "c": [2, 0, 15, 1], "d": [16, 16, 1],
            "e": [3, 1, 21], "f": [30, 1, 16]}
    at = {n: 0 for n in reqs}
    live, waiting, got = {}, ["a", "b", "c", "d", "e", "f"], {n: [] for n in reqs}
    steps = 0
    while waiting or live:
        while waiting and len(live) < 4:
            n = waiting.pop(0)
            live[n] = eng.open_sequence()
        names, feeds, wants = [], [], []
        for n in live:
            k = plan[n].pop(0)
            if not k:
                continue
            names.append(n)
            feeds.append(reqs[n][at[n]:at[n] + k])
            wants.append(list(range(k)))
            at[n] += k
        steps += 1
        if not names:
            continue
        out = eng.step_logits([live[n] for n in names], feeds, wants)
        o = 0
        for n, f in zip(names, feeds):
            got[n].append(out[o:o + len(f)])
            o += len(f)
            if at[n] == len(reqs[n]):
                eng.close_sequence(live.pop(n))
    assert steps > 5
    for n in reqs:
        if dtype == torch.float32:
            assert rel_err(torch.cat(got[n]), want[n]) < TOL[dtype], n
        else:
            assert rel_err(torch.cat(got[n]), want[n], 0.5) < 2 * TOL[dtype], n
    assert eng.kv.pool.free_blocks() == 192 // 16 and eng.kv.slots.free_slots() == 4


@pytest.mark.parametrize("device", DEVICES)
def test_slot_and_pages_reused_clean(device, full_model):
    """A pool of exactly one request's size, every state tensor, previous token
    and page overwritten with junk between requests: the next must not see it."""
    cfg, sd = full_model
    eng = engine(cfg, sd, device, max_tokens=48, max_seqs=1)
    assert eng.kv.nbytes() > 0
    for i, n in enumerate([40, 48, 3, 33]):
        toks = tokens(n, cfg["vocab"], 30 + i)
        seq = eng.open_sequence()
        got = feed(eng, seq, toks, [9, 1, 2])
        eng.close_sequence(seq)
        assert rel_err(got, O.forward(cfg, sd, toks)) < TOL[torch.float32], i
        for t in eng.kv.state.values():
            t.fill_(1e3)
        for named in eng.kv.rows.values():
            for t in named.values():
                t.fill_(-1e3)
        for named in eng.kv.ints.values():
            for t in named.values():
                t.fill_(41 + i)
        for a, b in eng.kv.kv_rows.values():
            a.fill_(50.0), b.fill_(-50.0)
    assert eng.kv.pool.free_blocks() == 3 and eng.kv.slots.free_slots() == 1


LOOPS = {
    "none": (FULL, None), "whole": (FULL[:4], (0, 4, 3)), "once": (FULL, (2, 5, 1)),
    "one_layer": (FULL[:3], (2, 3, 4)), "empty": (FULL[:2], (1, 1, 5)), "tail": (FULL, (3, 5, 2)),
    "middle": (FULL, (1, 2, 2)),
}


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("name", list(LOOPS))
def test_repeated_stretch_variants(device, name):
    """No repetition, the whole stack repeated, a single pass (entered through the
    projection all the same), one layer repeated four times, an empty stretch,
    stretches in the middle and at the end of the stack."""
    layers, loop = LOOPS[name]
    cfg = O.make_config(layers, loop=loop)
    sd = O.make_weights(cfg, 7)
    toks = tokens(37, cfg["vocab"], 13)
    want = O.forward(cfg, sd, toks)
    eng = engine(cfg, sd, device)
    got = feed(eng, eng.open_sequence(), toks, [20, 1, 3])
    assert rel_err(got, want) < TOL[torch.float32]


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("size", [16, 17, 32, 33, 1])
def test_window_edges_in_prompts_and_decoding(device, size):
    """Windows that end on, just before and just after a page border; the keys
    just inside and just outside pass the edge in portions and in decoding."""
    layers = [(O.parallel(O.window(heads=2, kv_heads=1, dim=8, vdim=12, size=size, rot_dims=4,
                                   scale=2.0), O.retention(heads=1)), O.dense_ff(16))]
    cfg = O.make_config(layers, width=16)
    sd = O.make_weights(cfg, 8)
    sd["l0.mix.left.q"] *= 3.0          # peaked scores: one key more or less shows
    sd["l0.mix.left.out"] *= 4.0
    toks = tokens(70, cfg["vocab"], 14)
    want = O.forward(cfg, sd, toks)
    for cuts in ([70], [40] + [1] * 30, [15, 2, 16]):
        eng = engine(cfg, sd, device)
        got = feed(eng, eng.open_sequence(), toks, cuts)
        assert rel_err(got, want) < TOL[torch.float32], cuts


@pytest.mark.parametrize("device", DEVICES)
def test_far_tokens_in_the_states(device):
    """Decays close to one in both recurrences: what stood hundreds of tokens
    back still shows in the logits, whatever the cut."""
    layers = [(O.parallel(O.window(size=3), O.retention(heads=2, decay=[0.9995, 1.0])), None),
              (O.delta(heads=2, kv_heads=1), None)]
    cfg = O.make_config(layers, width=16, vocab=40, mult=1.0)
    sd = O.make_weights(cfg, 9)
    sd["l1.mix.A_log"] -= 4.0
    toks = tokens(300, 40, 15)
    want = O.forward(cfg, sd, toks)
    other = O.forward(cfg, sd, [(toks[0] + 1) % 40] + toks[1:])
    assert rel_err(other[-1:], want[-1:]) > 10 * TOL[torch.float32]      # the first token still counts
    for cuts in ([300], [290] + [1] * 10, [130, 2, 59]):
        eng = engine(cfg, sd, device, max_tokens=304)
        got = feed(eng, eng.open_sequence(), toks, cuts)
        assert rel_err(got, want) < TOL[torch.float32], cuts


@pytest.mark.parametrize("device", DEVICES)
def test_first_tokens(device, full_model):
    cfg, sd = full_model
    for n in (1, 2, 3):
        toks = tokens(n, cfg["vocab"], 16 + n)
        eng = engine(cfg, sd, device)
        got = feed(eng, eng.open_sequence(), toks, [1])
        assert rel_err(got, O.forward(cfg, sd, toks)) < TOL[torch.float32]


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
def test_other_sizes(device, dtype):
    """Sizes that are unequal where a usual model makes them equal, single heads,
    one tap, a window of one, no rotation, one expert of one, a side input of one
    entry, constants of 1, odd widths, no repeated stretch."""
    layers = [
        (O.parallel(O.window(heads=1, kv_heads=1, dim=10, vdim=3, size=1, rot_dims=2),
                    O.retention(heads=1, dim=5, vdim=9, rot_dims=4)), None),
        (O.delta(heads=1, kv_heads=1, dim=5, vdim=9, conv=1, decay_rank=1, gate_rank=2), O.dense_ff(9)),
        (O.parallel(O.window(heads=6, kv_heads=3, dim=4, vdim=6, size=100, rot_dims=0),
                    O.retention(heads=5, dim=3, vdim=2, rot_dims=0)),
         O.moe_ff(ff=7, experts=1, top=1, groups=None, scale=0.4, limit=100.0)),
        (O.delta(heads=6, kv_heads=1, dim=4, vdim=2, conv=6, decay_rank=9, gate_rank=3),
         O.moe_ff(ff=5, experts=9, top=4, groups=9, keep=5, limit=0.2))]
    cfg = O.make_config(layers, width=22, vocab=31, mult=1.0, side=1, bigram=(1, 5, 3))
    sd = O.make_weights(cfg, 10)
    toks = tokens(45, 31, 17)
    want = O.forward(cfg, sd, toks)
    eng = engine(cfg, sd, device, dtype)
    got = feed(eng, eng.open_sequence(), toks, [19, 1, 2])
    if dtype == torch.float32:
        assert rel_err(got, want) < TOL[dtype]
    else:
        assert rel_err(got, want, 0.5) < TOL[dtype] and rel_err(got, want, 0.9) < 0.25


@pytest.mark.parametrize("device", DEVICES)
def test_optional_parts(device):
    """Without the pair embedding, the side inputs and the residual constant (all
    absent from the config) the model is the rest of the design."""
    cfg = O.make_config(FULL[:2], mult=1.0)
    sd = O.make_weights(cfg, 14)
    toks = tokens(20, cfg["vocab"], 21)
    sd["bigram"] = torch.zeros_like(sd["bigram"])
    sd["side.embed"] = torch.zeros_like(sd["side.embed"])     # a gate on nothing adds nothing
    want = O.forward(cfg, sd, toks)
    bare = {k: v for k, v in cfg.items() if k not in ("embedding", "token_side", "residual_mult")}
    eng = engine(bare, sd, device)
    assert eng.cfg.bigram is None and not eng.cfg.side_dim and not eng.kv.ints
    got = feed(eng, eng.open_sequence(), toks, [11, 1, 4])
    assert rel_err(got, want) < TOL[torch.float32]


@pytest.mark.parametrize("device", DEVICES)
def test_long_decode(device):
    layers = [(O.delta(heads=2, kv_heads=1), None),
              (O.parallel(O.window(heads=2, kv_heads=1, dim=8, vdim=8, size=24, rot_dims=8)),
               O.moe_ff())]
    cfg = O.make_config(layers, width=16, vocab=40, loop=(0, 2, 2))
    sd = O.make_weights(cfg, 11)
    toks = tokens(150, 40, 18)
    want = O.forward(cfg, sd, toks)
    eng = engine(cfg, sd, device)
    got = feed(eng, eng.open_sequence(), toks, [10] + [1] * 140)
    assert rel_err(got, want) < TOL[torch.float32]


@pytest.mark.parametrize("device", DEVICES)
def test_greedy_generation_through_scheduler(device, full_model):
    """Schema-less requests through ``submit_batch`` (continuous batching:
    inline prompts, chunked prompts in mixed steps, decode steps) produce the
    oracle's greedy continuation."""
    cfg, sd = full_model
    V = cfg["vocab"]
    prompts = [tokens(n, V, 40 + i) for i, n in enumerate([5, 90, 23, 70])]
    n_new = 6

    def greedy(p):
        seq = list(p)
        for _ in range(n_new):
            seq.append(int(O.forward(cfg, sd, seq)[-1].argmax()))
        return seq[len(p):]
    want = [greedy(p) for p in prompts]
    eng = engine(cfg, sd, device, max_tokens=512, max_seqs=4)
    eng.chunk_prefill = 32          # prompts longer than inline_prefill go in 32-token chunks
    eng.inline_prefill = 8
    reqs = [GenRequest(p, None, max_new_tokens=n_new) for p in prompts]
    try:
        eng.submit_batch(reqs[:2]).result(timeout=300)
        f1 = eng.submit_batch(reqs[2:3])
        f2 = eng.submit_batch(reqs[3:])
        f1.result(timeout=300), f2.result(timeout=300)
    finally:
        eng.stop()
    for r, w in zip(reqs, want):
        assert r.done and r.grammar.emitted == w
    assert eng.kv.slots.free_slots() == 4


def test_generate_entry_point(full_model):
    cfg, sd = full_model
    p = tokens(12, cfg["vocab"], 50)
    eng = engine(cfg, sd, "cpu")
    r = eng.generate([GenRequest(p, None, max_new_tokens=3)])[0]
    seq = list(p)
    for _ in range(3):
        seq.append(int(O.forward(cfg, sd, seq)[-1].argmax()))
    assert r.grammar.emitted == seq[len(p):]


def test_checkpoint_round_trip(tmp_path, full_model):
    """save -> config.json + safetensors -> registry -> the same logits."""
    from loqa_hub_amd.models.loader import save_vodalorn
    from loqa_hub_amd.models.registry import lm_config_of_checkpoint, load_lm_weights
    cfg_json, sd = full_model
    cfg = lm_config_from_json(O.public(cfg_json), "t")
    save_vodalorn(cfg, {k: v.to(torch.bfloat16) for k, v in sd.items()}, str(tmp_path / "ck"))
    cfg2 = lm_config_of_checkpoint(str(tmp_path / "ck"), "t")
    assert cfg2 == cfg and family_of(cfg2).name == "vodalorn"
    w = load_lm_weights(cfg2, str(tmp_path / "ck"), "cpu", dtype=torch.float32, max_positions=64)
    eng = LLMEngine(cfg2, "cpu", weights=w, max_seqs=1, max_seq_len=64, block_size=16, num_blocks=4,
                    use_graphs=False, dtype=torch.float32)
    toks = tokens(30, cfg_json["vocab"], 51)
    got = eng.step_logits([eng.open_sequence()], [toks], [list(range(30))])
    assert rel_err(got, O.forward(cfg_json, sd, toks)) < TOL[torch.float32]


def test_trace_replay_program(tmp_path, full_model):
    """The replay command on a checkpoint folder: steps on stdin, logits files
    and ``done`` lines out; a request that sits out a step goes on later."""
    from loqa_hub_amd.models.loader import write_safetensors
    cfg, sd = full_model
    model = tmp_path / "m"
    model.mkdir()
    (model / "config.json").write_text(json.dumps(O.public(cfg)))
    write_safetensors({k: v.to(torch.bfloat16) for k, v in sd.items()},
                      str(model / "model.safetensors"))
    a, b = tokens(20, cfg["vocab"], 60), tokens(9, cfg["vocab"], 61)
    steps = [
        {"step": 0, "entries": [{"id": "a", "tokens": a[:11], "want": [0, 10]}], "end": []},
        {"step": 1, "entries": [{"id": "b", "tokens": b[:8], "want": []}], "end": []},
        {"step": 2, "entries": [{"id": "a", "tokens": a[11:], "want": [8]},
                                {"id": "b", "tokens": b[8:], "want": [0]}], "end": ["a", "b"]},
    ]
    out = tmp_path / "out"
    p = subprocess.run([sys.executable, "-m", "loqa_hub_amd.cli.trace_run", "--model", str(model),
                        "--dtype", "float32", "--out", str(out), "--max-tokens", "64",
                        "--device", "cpu"],
                       input="\n".join(json.dumps(s) for s in steps) + "\n", text=True,
                       capture_output=True, cwd=ROOT, timeout=300)
    assert p.returncode == 0, p.stderr
    assert [ln for ln in p.stdout.splitlines() if ln.startswith("done")] == \
        ["done 0", "done 1", "done 2"]
    V = cfg["vocab"]
    wa, wb = O.forward(cfg, sd, a), O.forward(cfg, sd, b)
    g0 = torch.from_numpy(np.fromfile(out / "0.f32", dtype="<f4").reshape(-1, V))
    g2 = torch.from_numpy(np.fromfile(out / "2.f32", dtype="<f4").reshape(-1, V))
    assert not (out / "1.f32").exists()
    assert rel_err(g0, wa[[0, 10]]) < TOL[torch.float32]
    assert rel_err(g2, torch.stack([wa[19], wb[8]])) < TOL[torch.float32]


@pytest.mark.gpu
def test_serving_sizes_bf16():
    """A model with matrix-core head sizes in bfloat16: whole prompt, portions
    and decoding agree with the oracle within 16-bit rounding."""
    layers = [(O.delta(heads=4, kv_heads=2, dim=64, vdim=64, conv=4, decay_rank=16, gate_rank=16),
               O.dense_ff(96)),
              (O.parallel(O.window(heads=4, kv_heads=2, dim=64, vdim=192, size=40, rot_dims=32),
                          O.retention(heads=2, dim=64, vdim=64, rot_dims=64)),
               O.moe_ff(ff=64, experts=8, top=2, groups=2, keep=1))]
    cfg = O.make_config(layers, width=128, vocab=90, loop=(0, 2, 2), side=32)
    sd = O.make_weights(cfg, 12)
    toks = tokens(200, 90, 14)
    want = O.forward(cfg, sd, toks)
    eng = engine(cfg, sd, "cuda", torch.bfloat16, max_tokens=208)
    for cuts in ([200], [150, 30] + [1] * 20, [33, 2, 70]):
        seq = eng.open_sequence()
        got = feed(eng, seq, toks, cuts)
        eng.close_sequence(seq)
        assert rel_err(got, want, 0.5) < TOL[torch.bfloat16] and rel_err(got, want, 0.9) < 0.25, cuts
