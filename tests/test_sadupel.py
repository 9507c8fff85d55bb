"""Sadupel (parallel sublayers on one norm, looped layers, pair embedding,
attention behind short convolutions with whole-row norms, soft cap, sinks and
per-head gates, routed squared-ReLU units with identity experts) against the
plain float64 oracle in sadupel_oracle.py: every mechanism alone, then whole
models through the engine's cache, state slots, batching, scheduler and
generation.

Each test runs on the CPU op path and, marked gpu, on the gfx950 kernels.
fp32 runs are held to rounding-level agreement; bf16 runs to bf16 rounding.
"""
import json
import subprocess
import sys
from pathlib import Path
from types import SimpleNamespace

import pytest
import torch

sys.path.insert(0, str(Path(__file__).resolve().parent))

import sadupel_oracle as orc  # noqa: E402
from agentfield_amd.engine import LLMEngine, SamplingParams  # noqa: E402
from agentfield_amd.models import load_model  # noqa: E402
from agentfield_amd.models.sadupel import (SadupelConfig,  # noqa: E402
                                           SadupelForCausalLM, save_sadupel)
from agentfield_amd.models.zudisun import RoutedExperts, RoutedSpec  # noqa: E402
from agentfield_amd.ops import seqmix as sm  # noqa: E402

REPO = Path(__file__).resolve().parent.parent
DEVICES = ["cpu", pytest.param("cuda", marks=pytest.mark.gpu)]
DTYPES = [torch.float32, torch.bfloat16]
F64 = torch.float64


# ------------------------------------------------------------ model zoo
def _attn(heads, kv_heads, dim, vdim, conv, scale=0.3, softcap=None,
          rot=None):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim,
         "conv": conv, "scale": scale}
    if softcap:
        m["softcap"] = softcap
    if rot:
        m["rot"] = rot
    return m


def _moe(experts, top, ff, shared=None, groups=None, identity=0):
    r = {"experts": experts, "top": top}
    if groups:
        r["groups"] = {"count": groups[0], "keep": groups[1]}
    if identity:
        r["identity"] = identity
    f = {"kind": "moe", "expert": {"ff": ff}, "router": r}
    if shared:
        f["shared"] = {"ff": shared}
    return f


def _layer(mixer, mlp):
    return {"type": "attention", "mixer": mixer, "mlp": mlp}


def cfg_mixed():
    """Unequal sizes everywhere: head, key and value sizes, taps, caps and
    rotations differ between layers; groups that straddle the border between
    experts and identity experts; a layer without feed-forward inside a loop
    of three passes that starts behind the first layer; a layer without shared
    unit, one without groups."""
    rot = {"dims": 8, "base": 300.0, "scaling": {"factor": 3.0}}
    return {"architecture": "Sadupel", "vocab": 96, "width": 48,
            "residual_mult": 0.45, "norm": {"eps": 1e-5},
            "embedding": {"bigram": {"buckets": 61, "mul_prev": 19,
                                     "mul_cur": 5}},
            "loop": {"start": 1, "stop": 3, "times": 3},
            "layers": [
                _layer(_attn(6, 3, 12, 20, 4, 0.31, 9.0, rot),
                       _moe(7, 2, 24, 40, (3, 2), 2)),
                _layer(_attn(4, 1, 16, 8, 2, 0.4, 5.0,
                             {"dims": 16, "base": 50.0}), None),
                _layer(_attn(9, 3, 8, 12, 3, 0.5, None, rot),
                       _moe(5, 3, 16, None, (2, 1), 1)),
                _layer(_attn(2, 2, 20, 4, 1, 0.2, 30.0),
                       _moe(6, 1, 32, 8))]}


def cfg_degenerate():
    """Values a model may happen to make equal or 1: one head, kv_heads ==
    heads, dim == vdim, one tap, one expert, one group, every expert chosen,
    one bucket, a loop of one pass over all layers, multiplier 1, scale 1."""
    return {"architecture": "Sadupel", "vocab": 40, "width": 32,
            "residual_mult": 1.0, "norm": {"eps": 1e-6},
            "embedding": {"bigram": {"buckets": 1, "mul_prev": 1,
                                     "mul_cur": 1}},
            "loop": {"start": 0, "stop": 2, "times": 1},
            "layers": [
                _layer(_attn(1, 1, 8, 8, 1, 1.0, 1.0,
                             {"dims": 8, "base": 10.0,
                              "scaling": {"factor": 1.0}}),
                       _moe(1, 1, 8, 8, (1, 1))),
                _layer(_attn(4, 4, 8, 8, 4, 1.0, 2.0),
                       _moe(3, 4, 8, 8, (4, 4), 1))]}


def cfg_odd():
    """Nothing divisible by 4 or 8 (scalar kernel paths), ten query heads on
    one K/V head, six taps, rotation of two dims, a first-layer loop, no pair
    table."""
    return {"architecture": "Sadupel", "vocab": 33, "width": 30,
            "residual_mult": 0.8, "norm": {"eps": 1e-4},
            "loop": {"start": 0, "stop": 1, "times": 2},
            "layers": [
                _layer(_attn(10, 1, 6, 10, 6, 0.41, 7.0,
                             {"dims": 2, "base": 50.0,
                              "scaling": {"factor": 2.5}}),
                       _moe(5, 2, 9, 7, (2, 1), 1)),
                _layer(_attn(3, 1, 5, 3, 3, 0.6, 4.0,
                             {"dims": 4, "base": 90.0}),
                       _moe(3, 2, 25, 11, None, 2))]}


def cfg_wide():
    """Many small experts: an output product long enough for the split-K
    kernel of decode steps, a router of 128 outputs in 16 groups."""
    return {"architecture": "Sadupel", "vocab": 64, "width": 64,
            "residual_mult": 0.6, "norm": {"eps": 1e-6},
            "embedding": {"bigram": {"buckets": 29, "mul_prev": 7,
                                     "mul_cur": 3}},
            "layers": [
                _layer(_attn(8, 1, 16, 32, 3, 0.3, 6.0,
                             {"dims": 16, "base": 1000.0}),
                       _moe(124, 4, 64, 64, (16, 5), 4))]}


ZOO = {"mixed": cfg_mixed, "degenerate": cfg_degenerate, "odd": cfg_odd,
       "wide": cfg_wide}


def build(cfg_json, device, dtype, seed=0, page=8, pages=64, live=4,
          paced=True, graphs=False):
    w = orc.random_weights(cfg_json, seed)
    cfg = SadupelConfig.from_json(cfg_json)
    cfg.max_position = 512
    model = SadupelForCausalLM(cfg, device=device, dtype=dtype)
    model.load_tensors(w.__getitem__)
    eng = LLMEngine(cfg, device=device, dtype=dtype, page_size=page,
                    num_pages=pages, max_num_seqs=live, model=model,
                    enable_graphs=graphs, caller_paced=paced, eos_id=-1)
    return eng, w


def tokens_for(cfg_json, n, seed):
    g = torch.Generator().manual_seed(1000 + seed)
    return torch.randint(0, cfg_json["vocab"], (n,), generator=g).tolist()


def rel_err(got, want):
    """Row-wise: rms of the mean-free difference over rms of the oracle."""
    d = got.to(F64).cpu() - want
    d = d - d.mean(-1, keepdim=True)
    scale = want.pow(2).mean().sqrt()
    return float((d.pow(2).mean(-1).sqrt() / scale).max())


def tol(dtype):
    return 2e-4 if dtype == torch.float32 else 8e-2


def model_close(got, want, dtype):
    """fp32: every row at rounding level.  bf16: every row within twice, the
    median row within half of the rounding of a few layers (a router's near
    tie may fall the other way in single rows)."""
    d = got.to(F64).cpu() - want
    d = d - d.mean(-1, keepdim=True)
    rows = d.pow(2).mean(-1).sqrt() / want.pow(2).mean().sqrt()
    if dtype == torch.float32:
        return float(rows.max()) < tol(dtype)
    return (float(rows.quantile(0.97)) < 2 * tol(dtype)
            and float(rows.median()) < tol(dtype) / 2)


def run_schedule(eng, requests, schedule):
    """requests: name -> tokens.  schedule: list of steps, each a list of
    (name, count).  Every fed position's logits are collected; a request is
    closed when its last token went in.  Returns name -> [T, V]."""
    at = {n: 0 for n in requests}
    seqs, out = {}, {n: [] for n in requests}
    for step in schedule:
        entries, names = [], []
        for name, count in step:
            if name not in seqs:
                seqs[name] = eng.open_request()
            lo = at[name]
            entries.append((seqs[name], requests[name][lo:lo + count],
                            list(range(count))))
            names.append((name, count))
            at[name] = lo + count
        logits = eng.feed_step(entries)
        r = 0
        for name, count in names:
            out[name].append(logits[r:r + count].cpu())
            r += count
            if at[name] == len(requests[name]):
                eng.close_request(seqs.pop(name))
    return {n: torch.cat(v) for n, v in out.items()}


def md_for(chunks, starts, slots, device, page=8, pages_per_seq=32):
    """Batch description for op-level tests: sequence i runs chunks[i] rows
    from position starts[i], owns pages 1 + i*pages_per_seq ..; all chunks of
    one row form a decode step."""
    cu, rowseq, pos, kvslots = [0], [], [], []
    bt = torch.zeros(len(chunks), pages_per_seq, dtype=torch.int32)
    for i, (n, s0) in enumerate(zip(chunks, starts)):
        cu.append(cu[-1] + n)
        rowseq += [i] * n
        bt[i] = torch.arange(pages_per_seq) + 1 + i * pages_per_seq
        for p in range(s0, s0 + n):
            pos.append(p)
            kvslots.append(int(bt[i, p // page]) * page + p % page)
    t = lambda v, d: torch.tensor(v, dtype=d, device=device)  # noqa: E731
    single = all(n == 1 for n in chunks)
    md = SimpleNamespace(cu_seqlens=t(cu, torch.int32),
                         q_start=t(starts, torch.int32),
                         state_slots=t(slots, torch.int32),
                         row_seq=t(rowseq, torch.int32),
                         block_table=bt.to(device),
                         slots=t(kvslots, torch.int64),
                         seq_lens=None if single else list(chunks),
                         is_prefill=not single)
    return md, t(pos, torch.int32)


PORTIONS = ((0, 11), (11, 13), (13, 14), (14, 15), (15, 31), (31, 33),
            (33, 90))


# ====================================================== mechanisms alone
@pytest.mark.parametrize("device", DEVICES)
def test_kernel_groups_present(device):
    if device == "cuda":
        from agentfield_amd.ops import _lib
        for group in ("glue", "seq", "conv", "rope", "skinny"):
            assert _lib.mixgroup(group) is not None  # no eager fallback


# --------------------------------------------------------------- embedding
@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("W,buckets,mul_prev,mul_cur", [
    (32, 61, 19, 5), (30, 7, 1, 1), (8, 1, 3, 2),
    (516, 1009, 3000000019, 70001)])
def test_pair_embedding(device, dtype, W, buckets, mul_prev, mul_cur):
    """Two interleaved sequences in portions and single rows through slots
    with leftovers: the pair row follows the previous token across steps, the
    last row opens a sequence; products beyond 32 bits."""
    torch.manual_seed(W)
    V = 5000
    cfg = {"embedding": {"bigram": {"buckets": buckets, "mul_prev": mul_prev,
                                    "mul_cur": mul_cur}}}
    P = {"embed": torch.randn(V, W).to(dtype),
         "bigram": torch.randn(buckets + 1, W).to(dtype)}
    toks = [torch.randint(0, V, (n,)).tolist() for n in (90, 61)]
    want = [orc.embed(t, P, cfg) for t in toks]
    prev = torch.full((4, 1), 17, dtype=torch.int32, device=device)
    tab, pairs = P["embed"].to(device), P["bigram"].to(device)
    got = [[], []]
    at = [0, 0]
    for a, b in ((3, 1), (1, 1), (1, 1), (2, 30), (40, 1), (1, 2), (42, 25)):
        starts, lens = list(at), [a, b]
        md, _p = md_for(lens, starts, [2, 3], device)
        ids = torch.tensor(toks[0][at[0]:at[0] + a] + toks[1][at[1]:at[1] + b],
                           dtype=torch.int32, device=device)
        x = sm.embed_pairs(ids, tab, pairs, mul_prev, mul_cur, prev, md).cpu()
        got[0].append(x[:a])
        got[1].append(x[a:])
        at = [at[0] + a, at[1] + b]
    for g, w in zip(got, want):
        g = torch.cat(g)
        assert torch.allclose(g.to(F64), w, atol=1e-6)
    assert prev[:, 0].tolist() == [17, 17, toks[0][89], toks[1][60]]


# --------------------------------------------------------- residual + norm
def _terms(T, W, dtype, seed, top=3, nid=2):
    g = torch.Generator().manual_seed(seed)
    rnd = lambda *s: torch.randn(*s, generator=g)  # noqa: E731
    n = T * top - 4                       # four choices without a row
    pos = torch.randperm(T * top, generator=g).to(torch.int32)
    pos[pos >= n] = -1
    ys, hin = rnd(n, W).to(dtype), rnd(T, W).to(dtype)
    wts, idw = rnd(T, top).abs(), rnd(T, nid + 3).abs()
    u = torch.zeros(T, W, dtype=F64)
    for t in range(T):
        for r in range(top):
            p = int(pos[t * top + r])
            if p >= 0:
                u[t] += wts[t, r].to(F64) * ys[p].to(F64)
        u[t] += idw[t, 3:].to(F64).sum() * hin[t].to(F64)
    return dict(ys=ys, pos=pos, weights=wts, hin=hin), idw, u


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("W", [30, 32, 1028, 2050, 8196, 17000])
def test_residual_norm(device, dtype, W):
    """Row term, expert terms with missing rows, identity weights in a strided
    view and the pass vector, each alone and together, with and without the
    norm; widths in and past the register-held range."""
    torch.manual_seed(W)
    T, eps, mult = 9, 1e-5, 0.37
    d = lambda t: t.to(device)  # noqa: E731
    x0 = torch.randn(T, W) * 3
    a = torch.randn(T, W + 8).to(dtype)[:, :W]           # a strided view
    vec, w = torch.randn(W), (1 + 0.2 * torch.randn(W)).to(dtype)
    terms, idw, u = _terms(T, W, dtype, W)
    dt_terms = {k: d(v) for k, v in terms.items()}
    t = 2e-6 if dtype == torch.float32 else 1e-2
    full = x0.to(F64) + mult * (a.to(F64) + u) + vec.to(F64)
    x = d(x0.clone())
    h = sm.residual_norm(x, d(a), mult, d(w), eps, dtype, vec=d(vec),
                         idw=d(idw)[:, 3:], **dt_terms)
    assert rel_err(x, full) < 1e-6 and h.dtype == dtype
    assert rel_err(h, orc.rms_norm(full, w, eps)) < t
    # the row term alone, no norm
    x = d(x0.clone())
    assert sm.residual_norm(x, d(a), mult, None, eps, dtype) is None
    assert rel_err(x, x0.to(F64) + mult * a.to(F64)) < 1e-6
    # the pass vector alone is not scaled
    x = d(x0.clone())
    h = sm.residual_norm(x, None, mult, d(w), eps, dtype, vec=d(vec))
    assert rel_err(x, x0.to(F64) + vec.to(F64)) < 1e-6
    # a norm in front of the first layer leaves the row as it is
    x = d(x0.clone())
    h = sm.residual_norm(x, None, mult, d(w), eps, dtype)
    assert torch.equal(x.cpu(), x0)
    assert rel_err(h, orc.rms_norm(x0.to(F64), w, eps)) < t


@pytest.mark.parametrize("device", DEVICES)
def test_residual_norm_many_rows(device):
    """More rows than the few-rows layout takes."""
    T, W = 700, 2048
    terms, idw, u = _terms(T, W, torch.float32, 1)
    torch.manual_seed(2)
    x0, a, w = torch.randn(T, W), torch.randn(T, W), 1 + 0.2 * torch.randn(W)
    full = x0.to(F64) + 0.6 * (a.to(F64) + u)
    x = x0.clone().to(device)
    h = sm.residual_norm(x, a.to(device), 0.6, w.to(device), 1e-6,
                         torch.float32, idw=idw.to(device)[:, 3:],
                         **{k: v.to(device) for k, v in terms.items()})
    assert rel_err(x, full) < 1e-6
    assert rel_err(h, orc.rms_norm(full, w, 1e-6)) < 2e-6


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("M", [1, 5, 64, 100, 128, 129])
@pytest.mark.parametrize("N,K", [(128, 8192), (64, 9024), (2048, 33216),
                                 (192, 8200)])
def test_split_products_into_the_residual(device, M, N, K):
    """Partial sums over pieces of a long inner dimension, added up by the
    residual step; None where the other product serves."""
    torch.manual_seed(K)
    x = (torch.randn(M, K) * 0.1).to(torch.bfloat16).to(device)
    w = (torch.randn(N, K) * 0.1).to(torch.bfloat16).to(device)
    parts = sm.split_k_parts(x, w)
    fits = device == "cuda" and M <= 128 and K % 64 == 0
    assert (parts is not None) == fits
    if not fits:        # any partition adds up
        parts = torch.stack([x[:, :K // 8 * 3].float() @
                             w[:, :K // 8 * 3].float().t(),
                             x[:, K // 8 * 3:].float() @
                             w[:, K // 8 * 3:].float().t()])
    want = x.cpu().to(F64) @ w.cpu().to(F64).t()
    x0 = torch.randn(M, N)
    xr = x0.clone().to(device)
    nw = 1 + 0.1 * torch.randn(N)
    h = sm.residual_norm(xr, parts, 0.25, nw.to(device), 1e-6, torch.float32)
    full = x0.to(F64) + 0.25 * want
    assert rel_err(xr, full) < 2e-5
    assert rel_err(h, orc.rms_norm(full, nw, 1e-6)) < 2e-5


# ------------------------------------------------------------ feed-forward
@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("lead,unit,n", [(8, 12, 3), (0, 5, 4), (7, 3, 2),
                                         (16, 4, 0), (4, 64, 9)])
def test_weighted_squared_relu(device, dtype, lead, unit, n):
    """Columns of a wider buffer in and out; the leading unit unweighted, a
    weight of zero silences a unit."""
    torch.manual_seed(unit)
    T, F = 19, lead + unit * n
    z = torch.randn(T, F + 13).to(dtype)
    rw = torch.rand(T, n + 2)
    rw[::2, 0] = 0.0
    want = torch.relu(z[:, 8:8 + F].to(F64)).pow(2)
    want[:, lead:] *= rw[:, :n].to(F64).repeat_interleave(unit, 1)
    buf = torch.full((T, F + 20), 7.0, dtype=dtype, device=device)
    sm.relu2(z.to(device)[:, 8:8 + F], out=buf[:, 8:8 + F],
             row_weight=rw.to(device), unit=unit, lead=lead)
    b = buf.cpu()
    err = (b[:, 8:8 + F].to(F64) - want).abs() / (want.abs() + 1e-3)
    assert float(err.max()) < (1e-6 if dtype == torch.float32 else 8e-3)
    assert bool((b[:, :8] == 7.0).all() and (b[:, 8 + F:] == 7.0).all())


ROUTERS = [dict(experts=7, top=2, groups={"count": 3, "keep": 2}, identity=2),
           dict(experts=5, top=3, groups={"count": 2, "keep": 1}, identity=1),
           dict(experts=6, top=6), dict(experts=1, top=1),
           dict(experts=12, top=4, groups={"count": 16, "keep": 5},
                identity=4),
           dict(experts=150, top=8, groups={"count": 10, "keep": 3},
                identity=10)]


def _spec(r, ff, shared=0):
    g = r.get("groups") or {"count": 0, "keep": 0}
    return RoutedSpec(experts=r["experts"], top=r["top"], ff=ff, act="relu2",
                      score="softmax", renorm=False, groups=g["count"],
                      keep=g["keep"], group_top=1,
                      identity=r.get("identity", 0), shared_ff=shared)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("shift", [0.0, -3.0])
@pytest.mark.parametrize("r", ROUTERS)
def test_router(device, shift, r):
    """Groups score their best choice score, choice scores may all be
    negative, weights are the plain softmax over all outputs."""
    n = r["experts"] + r.get("identity", 0)
    torch.manual_seed(n)
    T = 40
    z = torch.randn(T, n) * 2
    corr = torch.randn(n) * 0.3 + shift
    s = _spec(r, 8)
    idx, wts, wd = sm.moe_route(
        z.to(device), corr.to(device), s.top, s.groups, s.keep, dense=True,
        score="softmax", renorm=False, group_top=1)
    dense = torch.zeros(T, n, dtype=F64)
    for t in range(T):
        e, w = orc.choose(z[t].to(F64), corr, r)
        assert idx[t].tolist() == e
        assert torch.allclose(wts[t].cpu().to(F64), torch.tensor(w, dtype=F64),
                              rtol=2e-6)
        dense[t, e] = torch.tensor(w, dtype=F64)
    assert torch.allclose(wd.cpu().to(F64), dense, atol=1e-6)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("T", [1, 37])
@pytest.mark.parametrize("W", [24, 200, 1032, 30])
@pytest.mark.parametrize("r", ROUTERS[:5] + [
    dict(experts=40, top=3), dict(experts=96, top=5, identity=12)])
def test_router_from_rows(device, dtype, T, W, r):
    """Logits and routing in one step: fp32 products of rows in either dtype
    with router weights that use all their bits; strided rows."""
    n = r["experts"] + r.get("identity", 0)
    torch.manual_seed(n + W)
    h = torch.randn(T, W + 8).to(dtype)
    router = torch.randn(n, W) * 2 * W ** -0.5
    corr = torch.randn(n) * 0.1
    s = _spec(r, 8)
    idx, wts, wd = sm.moe_router(
        h.to(device)[:, :W], router.to(device), corr.to(device), s.top,
        s.groups, s.keep, dense=True, score="softmax", renorm=False,
        group_top=1)
    z = h[:, :W].to(F64) @ router.to(F64).t()
    full = torch.softmax(z, -1)
    for t in range(T):
        e, w = orc.choose(z[t], corr, r)
        got = idx[t].tolist()
        c = full[t] + corr.to(F64)
        assert all(abs(float(c[a] - c[b])) < 1e-5 for a, b in zip(got, e))
        assert torch.allclose(wts[t].cpu().to(F64), full[t, got], rtol=1e-5)
        row = torch.zeros(n)
        row[got] = wts[t].cpu()
        assert torch.equal(wd[t].cpu(), row)


def test_group_score_is_the_largest_not_a_sum():
    """One strong expert beats two middling ones of another group."""
    z = torch.log(torch.tensor([[0.40, 0.02, 0.28, 0.30]]))
    for top, first in ((1, 0), (2, 3)):
        idx, _w, _d = sm.moe_route(z, torch.zeros(4), 1, 2, 1,
                                   score="softmax", renorm=False,
                                   group_top=top)
        assert int(idx) == first


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("r", ROUTERS[:5])
@pytest.mark.parametrize("T", [1, 40])
def test_sorted_experts(device, dtype, T, r):
    """Each expert on the rows that chose it, identity experts without rows,
    summed by both combining kernels."""
    W, ff = 24, 20
    cfg = {"width": W, "vocab": 4, "norm": {"eps": 1e-5}, "layers": [
        _layer(_attn(1, 1, 4, 4, 1), _moe(r["experts"], r["top"], ff))]}
    cfg["layers"][0]["mlp"]["router"] = r
    P = orc.random_weights(cfg, 3)
    torch.manual_seed(T)
    h = torch.randn(T, W).to(dtype)
    want = orc.mixture(h.to(F64), P, "l0.mlp.", cfg["layers"][0]["mlp"])
    mod = RoutedExperts(_spec(r, ff), W, hosted=True)
    mod.router.copy_(P["l0.mlp.router"])
    mod.correction.copy_(P["l0.mlp.correction"])
    mod = mod.to(device)
    names = [f"l0.mlp.e{e}." for e in range(r["experts"])]
    up = torch.cat([P[n + "up"] for n in names]).to(device, dtype)
    down = torch.cat([P[n + "down"] for n in names], 1).to(device, dtype)
    hd = h.to(device)
    idx, wts, wd = mod.route(hd, True)
    ys, pos = mod.run_sorted(hd, mod.sort(idx), up, down)
    kw = {}
    if r.get("identity"):
        kw = dict(hin=hd, idw=wd[:, r["experts"]:])
        assert bool((pos.cpu() >= 0).eq(idx.cpu().flatten()
                                        < r["experts"]).all())
    zero = torch.zeros(T, W, dtype=dtype, device=device)
    got = sm.moe_combine(ys, pos if ys is not None else None,
                         wts if ys is not None else None, zero, **kw)
    assert rel_err(got, want) < tol(dtype) / 2
    x = torch.zeros(T, W, device=device)
    if ys is not None:
        kw.update(ys=ys, pos=pos, weights=wts)
    sm.residual_norm(x, None, 1.0, None, 1e-5, dtype, **kw)
    assert rel_err(x, want) < tol(dtype) / 2


@pytest.mark.parametrize("device", DEVICES)
def test_only_identity_experts_chosen(device):
    """A step in which no row takes a real expert."""
    W = 16
    mod = RoutedExperts(_spec(dict(experts=3, top=2, identity=2), 8), W,
                        hosted=True)
    mod.router.zero_()
    mod.correction.copy_(torch.tensor([0., 0., 0., 1., 2.]))
    mod = mod.to(device)
    h = torch.randn(20, W, device=device)
    idx, _w, wd = mod.route(h, True)
    assert idx.tolist() == [[4, 3]] * 20
    ys, pos = mod.run_sorted(h, mod.sort(idx),
                             torch.zeros(24, W, device=device),
                             torch.zeros(W, 24, device=device))
    assert ys is None and bool((pos == -1).all())
    x = torch.zeros(20, W, device=device)
    sm.residual_norm(x, None, 0.5, None, 1e-5, torch.float32, hin=h,
                     idw=wd[:, 3:])
    assert rel_err(x, 0.5 * 0.4 * h.cpu().to(F64)) < 1e-6


def test_plain_experts_need_a_host():
    with pytest.raises(ValueError):
        RoutedExperts(_spec(dict(experts=3, top=2), 8), 16)


# --------------------------------- convolution, norms, rotation, page append
def test_frequencies_are_divided():
    got = sm.scaled_inv_freq(16, 300.0, {"factor": 3.0})
    want = torch.tensor(orc.frequencies(
        {"dims": 16, "base": 300.0, "scaling": {"factor": 3.0}}), dtype=F64)
    assert torch.allclose(got, want, rtol=1e-14, atol=0)
    assert torch.allclose(got * 3, sm.scaled_inv_freq(16, 300.0), rtol=1e-14)


GEOMS = [  # heads, kv_heads, dim, vdim, taps, rotated dims
    (4, 2, 16, 8, 3, 8), (2, 2, 8, 8, 1, 8), (6, 3, 12, 20, 4, 8),
    (4, 4, 70, 24, 2, 6), (3, 1, 5, 3, 6, 4), (6, 2, 32, 16, 2, 0),
    (1, 1, 4, 4, 4, 0), (9, 3, 7, 9, 3, 2),
    # register tiles of 1, 2, 3 and 4 groups a thread
    (8, 2, 96, 64, 3, 96), (16, 8, 128, 128, 4, 64), (32, 8, 128, 128, 4, 128),
    (32, 12, 128, 128, 2, 128), (32, 12, 128, 128, 1, 8),
    # rows wider than the register tiles; rows that do not fit in LDS
    (40, 20, 128, 128, 3, 32), (128, 4, 128, 8, 2, 64)]


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("geom", GEOMS)
def test_conv_norm_rotation_and_page_append(device, dtype, geom):
    """Two sequences in portions shorter than the taps and single rows (the
    decode form), slots with leftovers; whole-row norms, partial rotation."""
    H, G, dk, dv, taps, rd = geom
    nq, nk, nv = H * dk, G * dk, G * dv
    C, page, eps = nq + nk + nv, 8, 1e-5
    torch.manual_seed(C + taps)
    big = C > 3000
    lens = (30, 27) if big else (90, 61)
    rot = {"dims": rd, "base": 700.0, "scaling": {"factor": 2.0}} if rd \
        else None
    w = torch.randn(C, taps).to(dtype) * 0.6
    wq, wk = ((1 + 0.2 * torch.randn(n)).to(dtype) for n in (nq, nk))
    us = [torch.randn(n, C).to(dtype) for n in lens]
    want = []
    for u in us:
        T = u.shape[0]
        y = orc.short_conv(u.to(F64), w)
        q = orc.rms_norm(y[:, :nq], wq, eps).view(T, H, dk)
        k = orc.rms_norm(y[:, nq:nq + nk], wk, eps).view(T, G, dk)
        want.append((orc.rotate(q, rot).reshape(T, -1),
                     orc.rotate(k, rot).reshape(T, -1), y[:, nq + nk:]))
    d = lambda t: t.to(device)  # noqa: E731
    kc = torch.zeros(70, G, page, dk, dtype=dtype, device=device)
    vc = torch.zeros(70, G, page, dv, dtype=dtype, device=device)
    st = torch.full((4, max(taps - 1, 1), C), 9.0, dtype=dtype, device=device)
    inv = sm.scaled_inv_freq(rd, 700.0, rot["scaling"]).to(device) if rd \
        else None
    cw, got, at = d(w.t().contiguous()), [[], []], [0, 0]
    cuts = ((3, 1), (1, 1), (1, 1), (2, 19), (20, 1), (1, 2), (2, 2)) if big \
        else ((3, 1), (1, 1), (1, 1), (2, 30), (40, 1), (1, 2), (42, 25))
    for a, b in cuts:
        md, pos = md_for([a, b], at, [2, 3], device)
        p = torch.zeros(a + b, C + (-C) % 8 + 8, dtype=dtype)
        p[:, :C] = torch.cat([us[0][at[0]:at[0] + a], us[1][at[1]:at[1] + b]])
        tab = sm.rotary_table(pos, inv) if rd else None
        q = sm.conv_qk_rope_cache(d(p)[:, :C], cw, st, md, H, G, eps, kc, vc,
                                  q_norm=d(wq), k_norm=d(wk),
                                  rot_tab=tab).cpu()
        got[0].append(q[:a])
        got[1].append(q[a:])
        at = [at[0] + a, at[1] + b]
    tl = 3e-6 if dtype == torch.float32 else 1.2e-2
    for i, (wq_, wk_, wv_) in enumerate(want):
        T = lens[i]
        assert rel_err(torch.cat(got[i]), wq_) < tl
        j = torch.arange(T)
        pg = 1 + i * 32 + j // page
        gk = kc.cpu()[pg, :, j % page].reshape(T, -1)
        gv = vc.cpu()[pg, :, j % page].reshape(T, -1)
        assert rel_err(gk, wk_) < tl and rel_err(gv, wv_) < tl
        if taps > 1:            # the slot holds the last inputs, oldest first
            assert torch.equal(st[i + 2].cpu(), us[i][T - taps + 1:T])
    assert bool((st[:2].cpu() == 9.0).all())


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("T", [600, 2100, 8300])
def test_conv_rows_over_workgroups(device, dtype, T):
    """Prompt portions long enough for every rows-per-workgroup choice, chunk
    borders inside and on the edge of a workgroup's rows, against the same
    rows one sequence at a time; no norm, far positions."""
    H, G, dk, dv, taps = 2, 1, 8, 4, 4
    C = H * dk + G * (dk + dv)
    torch.manual_seed(T)
    lens = [T - 300, 8, 3, 1, 288]
    starts = [70000, 0, 2, 40, 0]
    p = torch.randn(T, C).to(dtype).to(device)
    w = torch.randn(taps, C).to(dtype).to(device)
    st0 = torch.randn(6, taps - 1, C).to(dtype).to(device)
    inv = sm.scaled_inv_freq(8, 1e4).to(device)

    def run(sel, lens, starts, slots, st):
        cu, pos, rs = [0], [], []
        for i, (n, s0) in enumerate(zip(lens, starts)):
            cu.append(cu[-1] + n)
            pos += range(s0, s0 + n)
            rs += [i] * n
        t = lambda v, dt: torch.tensor(v, dtype=dt, device=device)  # noqa: E731
        md = SimpleNamespace(
            cu_seqlens=t(cu, torch.int32), q_start=t(starts, torch.int32),
            state_slots=t(slots, torch.int32), row_seq=t(rs, torch.int32),
            slots=t(list(range(len(pos))), torch.int64), seq_lens=lens,
            is_prefill=True)
        kc = torch.zeros(-(-T // 16), G, 16, dk, dtype=dtype, device=device)
        vc = torch.zeros(-(-T // 16), G, 16, dv, dtype=dtype, device=device)
        tab = sm.rotary_table(t(pos, torch.int32), inv)
        q = sm.conv_qk_rope_cache(p[sel], w, st, md, H, G, 1e-5, kc, vc,
                                  rot_tab=tab)
        n = len(pos)
        return (q.cpu(), kc.transpose(1, 2).reshape(-1, dk)[:n].cpu(),
                vc.transpose(1, 2).reshape(-1, dv)[:n].cpu())
    st = st0.clone()
    whole = run(slice(0, T), lens, starts, [1, 2, 3, 4, 5], st)
    lo, parts, st1 = 0, [], st0.clone()
    for i, n in enumerate(lens):
        parts.append(run(slice(lo, lo + n), [n], [starts[i]], [i + 1], st1))
        lo += n
    for j in range(3):
        assert torch.equal(whole[j], torch.cat([q[j] for q in parts]))
    assert torch.equal(st.cpu(), st1.cpu())
    y = orc.short_conv(p[:lens[0]].cpu().to(F64), w.cpu().t())
    pos = torch.arange(70000, 70000 + lens[0], dtype=F64)
    want = orc.rotate(y[:, :16].view(-1, 2, 8),
                      {"dims": 8, "base": 1e4}, pos).reshape(-1, 16)
    assert rel_err(whole[0][taps:lens[0]], want[taps:]) < \
        (3e-6 if dtype == torch.float32 else 1.2e-2)


# ---------------------------------------------------------------- attention
def _through_cache(device, dtype, q, k, v, scale, cap, sink, gate, schedule,
                   page=16):
    """q [T, H, dk], k [T, G, dk], v [T, G, dv] through pages and
    ops.masked_attention into columns of a wider buffer."""
    T, H, dk = q.shape
    G, dv = k.shape[1], v.shape[2]
    kc = torch.zeros(80, G, page, dk, dtype=dtype, device=device)
    vc = torch.zeros(80, G, page, dv, dtype=dtype, device=device)
    out, lo = [], 0
    for n in schedule:
        md, pos = md_for([n], [lo], [1], device, page=page, pages_per_seq=64)
        row = lambda t: t[lo:lo + n].reshape(n, -1).to(device, dtype)  # noqa
        sl = md.slots
        kc[sl // page, :, sl % page] = k[lo:lo + n].to(device, dtype)
        vc[sl // page, :, sl % page] = v[lo:lo + n].to(device, dtype)
        buf = torch.full((n, H * dv + 24), 3.0, dtype=dtype, device=device)
        gg = None
        if gate is not None:
            wide = torch.zeros(n, H + 5, dtype=dtype, device=device)
            wide[:, 2:2 + H] = row(gate)
            gg = wide[:, 2:2 + H]
        sm.masked_attention(row(q), kc, vc, md, pos, scale, H,
                            sink=sink.to(device) if sink is not None else None,
                            softcap=cap, gate=gg, out=buf[:, 8:8 + H * dv])
        b = buf.cpu()
        assert bool((b[:, :8] == 3.0).all() and (b[:, 8 + H * dv:] == 3.0).all())
        out.append(b[:, 8:8 + H * dv])
        lo += n
    return torch.cat(out)


SCHEDULES = {"whole": [150], "decoded": [40] + [1] * 110,
             "portions": [2, 3, 17, 2, 64, 30, 2, 29, 1]}


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("how", list(SCHEDULES))
@pytest.mark.parametrize("geom", [(4, 2, 16, 8), (3, 1, 10, 6), (2, 2, 64, 64),
                                  (16, 2, 8, 24), (2, 1, 72, 136),
                                  (8, 1, 128, 128), (5, 5, 7, 9),
                                  (2, 1, 520, 24), (1, 1, 20, 600)])
def test_gated_attention(device, dtype, how, geom):
    """Cap, sink and per-head gate in tile, row, many-heads, split and wide
    kernels, written into columns of a wider buffer; sinks from silent to
    ruling."""
    H, G, dk, dv = geom
    if how == "portions" and dk * dv > 2000:
        pytest.skip("covered by the other schedules")
    torch.manual_seed(H * dk)
    T = 150
    rnd = lambda *s: torch.randn(*s).to(dtype)  # noqa: E731
    q, k, v, gate = rnd(T, H, dk), rnd(T, G, dk), rnd(T, G, dv), rnd(T, H)
    sink = torch.linspace(-4.0, 7.0, H)
    scale, cap = 2.0 * dk ** -0.5, 3.0
    want = orc.attend(q.to(F64), k.to(F64), v.to(F64), scale, cap, sink)
    want = (want * torch.sigmoid(gate.to(F64))[:, :, None]).reshape(T, -1)
    got = _through_cache(device, dtype, q, k, v, scale, cap, sink, gate,
                         SCHEDULES[how])
    assert rel_err(got, want) < (5e-5 if dtype == torch.float32 else 3e-2)
    if how == "whole":
        plain = orc.attend(q.to(F64), k.to(F64), v.to(F64), scale)
        got = _through_cache(device, dtype, q, k, v, scale, 0.0, None, None,
                             SCHEDULES[how])
        assert rel_err(got, plain.reshape(T, -1)) < \
            (5e-5 if dtype == torch.float32 else 3e-2)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("how", ["whole", "decoded"])
@pytest.mark.parametrize("loud", [0, 15, 16, 63, 64, 255])
def test_one_loud_key_is_heard_for_ever(device, dtype, how, loud):
    """One key hundreds of positions back whose capped score towers over the
    rest, at page and tile borders and at position 0; a row in front of it
    does not hear it; a sink above the cap drowns it."""
    torch.manual_seed(loud)
    T, H, G, dk, dv, cap = 600, 4, 2, 32, 16, 12.0
    q, k = torch.randn(T, H, dk) * 0.2, torch.randn(T, G, dk) * 0.2
    v = torch.randn(T, G, dv)
    q[..., 0], k[..., 0] = 6.0, 0.0
    k[loud, :, 0] = 8.0                 # score 24, about 11.6 under the cap
    v[loud] = 0.0
    v[loud, :, 2] = 50.0
    q, k, v = (t.to(dtype) for t in (q, k, v))
    sink = torch.tensor([-5.0, 0.0, 5.0, 15.0])
    sched = [T] if how == "whole" else [540] + [1] * 60
    got = _through_cache(device, dtype, q, k, v, 0.5, cap, sink, None, sched)
    got = got.view(T, H, dv)[:, :, 2].float()
    m = float(torch.tensor(24.0 / cap).tanh() * cap)
    for i in (loud, loud + 1, 300, 541, 599):
        e = torch.exp(torch.tensor(m))
        share = 50.0 * e / (e + i + torch.exp(sink))
        assert torch.allclose(got[i], share, rtol=0.03, atol=0.05), i
    if loud:
        assert float(got[loud - 1].abs().max()) < 4.0
    assert float(got[599, 3]) < 3.0 < 45.0 < float(got[599, 0])


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("n", [1, 2, 40])
def test_first_tokens_share_with_the_sink(device, dtype, n):
    """Equal scores: row i gives its keys 1 / (i + 1 + e^sink) each, the sink
    neither scaled nor capped and counted once, in every kernel."""
    T, H, dv = 40, 2, 8
    q, k = torch.zeros(T, H, 16), torch.zeros(T, 1, 16)
    v = torch.ones(T, 1, dv)
    sink = torch.tensor([0.0, 2.5])
    sched = [T] if n == 40 else [n] * (T // n)
    got = _through_cache(device, dtype, q, k, v, 0.01, 1.5, sink, None, sched)
    i = torch.arange(1, T + 1, dtype=F64)[:, None]
    want = (i / (i + torch.exp(sink.to(F64)))).repeat_interleave(dv, 1)
    assert float((got.to(F64) - want).abs().max()) < \
        (1e-6 if dtype == torch.float32 else 4e-3)


# ============================================================ whole models
@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", list(ZOO))
def test_whole_prompt_and_layers(device, dtype, name):
    cj = ZOO[name]()
    eng, w = build(cj, device, dtype)
    toks = tokens_for(cj, 70, 1)
    layers = []
    want = orc.forward(toks, w, cj, layers)
    eng.model.record_runs = []
    got = run_schedule(eng, {"a": toks}, [[("a", len(toks))]])["a"]
    assert model_close(got, want, dtype)
    assert len(eng.model.record_runs) == len(layers)
    for g, r in zip(eng.model.record_runs, layers):
        assert model_close(g, r, dtype)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", list(ZOO))
def test_prefill_then_token_by_token(device, dtype, name):
    """The first tokens of a sequence one by one, a prompt portion, then long
    decoding: past every window and page border."""
    cj = ZOO[name]()
    eng, w = build(cj, device, dtype, pages=40)
    toks = tokens_for(cj, 170, 2)
    want = orc.forward(toks, w, cj)
    sched = [[("a", 1)]] * 6 + [[("a", 44)]] + [[("a", 1)]] * 120
    got = run_schedule(eng, {"a": toks}, sched)["a"]
    assert model_close(got, want, dtype)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
def test_portions_down_to_two_tokens(device, dtype):
    cj = cfg_mixed()
    eng, w = build(cj, device, dtype)
    toks = tokens_for(cj, 120, 3)
    want = orc.forward(toks, w, cj)
    cuts = [2, 2, 3, 2, 17, 2, 40, 5, 2, 16, 1, 2, 26]
    assert sum(cuts) == len(toks)
    got = run_schedule(eng, {"a": toks}, [[("a", c)] for c in cuts])["a"]
    assert model_close(got, want, dtype)
    whole = run_schedule(eng, {"a": toks}, [[("a", len(toks))]])["a"]
    # how a prompt is cut changes nothing beyond rounding
    assert model_close(got, whole.to(F64), dtype)
    if dtype == torch.float32:
        assert rel_err(got, whole.to(F64)) < 5e-5


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["mixed", "odd"])
def test_mixed_batches_reuse_pages_and_slots(device, dtype, name):
    """Eight unequal requests through two state slots and a pool of nine
    pages: portions beside single tokens, requests paused and resumed, pages
    and slots handed to the next request as soon as one ends; then every
    request alone, which must give the same."""
    cj = ZOO[name]()
    eng, w = build(cj, device, dtype, page=8, pages=10, live=2)
    lens = [30, 9, 33, 2, 17, 25, 1, 12]
    reqs = {f"r{i}": tokens_for(cj, n, 10 + i) for i, n in enumerate(lens)}
    sched = [
        [("r0", 5), ("r1", 2)], [("r0", 1), ("r1", 7)],          # r1 ends
        [("r2", 3)], [("r0", 20), ("r2", 1)], [("r0", 1), ("r2", 1)],
        [("r0", 3), ("r2", 1)], [("r2", 27)],                    # r0, r2 end
        [("r3", 2), ("r4", 16)], [("r4", 1), ("r5", 2)],         # r3, r4 end
        [("r5", 23), ("r6", 1)],                                 # both end
        [("r7", 2)], [("r7", 1)], [("r7", 9)]]
    got = run_schedule(eng, reqs, sched)
    want = {n: orc.forward(toks, w, cj) for n, toks in reqs.items()}
    assert model_close(torch.cat([got[n] for n in reqs]),
                       torch.cat([want[n] for n in reqs]), dtype)
    for n in reqs:
        alone = run_schedule(eng, {n: reqs[n]}, [[(n, len(reqs[n]))]])[n]
        if dtype == torch.float32:
            assert rel_err(got[n], alone.to(F64)) < 5e-5
    assert eng.sched.alloc.num_free == 9
    assert eng.state_slots.num_free == 2


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
def test_far_token_through_every_pass(device, dtype):
    """A token 300 positions back moves the logits, identically however the
    prompt in between was cut; every pass of the loop has pages of its own."""
    cj = cfg_mixed()
    eng, w = build(cj, device, dtype, pages=100)
    runs = orc.runs(cj)
    assert len(eng.kv.k) == len(runs) == 8
    a = tokens_for(cj, 310, 5)
    b = list(a)
    b[4] = (a[4] + 1) % cj["vocab"]
    wa, wb = orc.forward(a, w, cj), orc.forward(b, w, cj)
    assert rel_err(wa[-1:], wb[-1:]) > 1e-4          # the oracle hears it
    cuts = [3, 61, 2, 100, 1, 1, 77, 64, 1]
    got = run_schedule(eng, {"a": a, "b": b},
                       [[("a", c), ("b", c)] for c in cuts])
    assert model_close(got["a"], wa, dtype)
    assert model_close(got["b"], wb, dtype)
    if dtype == torch.float32:
        d = (got["a"] - got["b"])[-1].to(F64)
        assert rel_err(d[None], (wa - wb)[-1:]) < 0.05


@pytest.mark.parametrize("change", ["times", "start", "stop", "step"])
def test_oracle_tells_loops_apart(change):
    """What the loop's fields mean shows in the logits: a changed one in the
    oracle is noticed."""
    cj = cfg_mixed()
    eng, w = build(cj, "cpu", torch.float32)
    toks = tokens_for(cj, 12, 3)
    got = run_schedule(eng, {"a": toks}, [[("a", 12)]])["a"]
    assert model_close(got, orc.forward(toks, w, cj), torch.float32)
    other = cfg_mixed()
    if change == "step":
        w = dict(w)
        w["loop.step"] = w["loop.step"].roll(1, 0)
    else:
        other["loop"][change] += {"times": -1, "start": 1, "stop": -1}[change]
    assert not model_close(got, orc.forward(toks, w, other), torch.float32)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["mixed", "wide"])
def test_greedy_generation_through_scheduler(device, dtype, name):
    """engine.generate: the scheduler's batched prefill, (on GPU) the
    graph-captured decode step and the sampler reproduce the oracle's greedy
    continuation of unequal prompts; a second batch replays the same graphs
    over reused pages and slots."""
    cj = ZOO[name]()
    eng, w = build(cj, device, dtype, paced=False,
                   graphs=(device == "cuda"), pages=48)
    # the GPU sampler reads logits rounded to bf16, so near-ties may fall
    # either way: every emitted token must be (all but) the oracle's best
    # given the tokens emitted before it
    slack = 0.8 if dtype == torch.bfloat16 else \
        (0.1 if device == "cuda" else 1e-3)
    for lens in ((5, 23, 1, 14), (9, 2, 30, 4)):
        prompts = [tokens_for(cj, n, 20 + n) for n in lens]
        outs = eng.generate(prompts, SamplingParams(max_tokens=12,
                                                    temperature=0.0,
                                                    ignore_eos=True))
        for p, o in zip(prompts, outs):
            assert len(o) == 12
            want = orc.forward(p + o, w, cj)
            for i, tok in enumerate(o):
                row = want[len(p) + i - 1]
                assert row[tok] >= row.max() - slack, (len(p), i)
        assert eng.state_slots.num_free == 4   # all slots given back


def test_scheduler_preemption_restarts_state():
    """Running out of pages preempts a sequence; on re-admission it
    recomputes from position 0 in whatever slot is free and still produces
    the oracle's greedy tokens."""
    cj = cfg_degenerate()
    eng, w = build(cj, "cpu", torch.float32, seed=17, page=4, pages=9,
                   live=3, paced=False)
    prompts = [tokens_for(cj, 6, 40 + i) for i in range(3)]
    outs = eng.generate(prompts, SamplingParams(max_tokens=10,
                                                ignore_eos=True))
    assert eng.sched.n_preempted > 0
    for p, o in zip(prompts, outs):
        want = orc.forward(p + o, w, cj)
        for i, tok in enumerate(o):
            row = want[len(p) + i - 1]
            assert row[tok] >= row.max() - 1e-3


# ----------------------------------------------- config, registry, programs
def test_config_round_trip_and_registry(tmp_path):
    for make in ZOO.values():
        cfg = SadupelConfig.from_json(make())
        again = SadupelConfig.from_json(cfg.to_json())
        assert again.layers == cfg.layers and again.eps == cfg.eps
        assert again.residual_mult == cfg.residual_mult
        assert again.runs == cfg.runs and again.pairs == cfg.pairs
        assert [r[0] for r in cfg.runs] == [r[0] for r in orc.runs(make())]
    cj = cfg_mixed()
    w = orc.random_weights(cj, 4)
    cfg = SadupelConfig.from_json(cj)
    save_sadupel({k: v.to(torch.bfloat16) for k, v in w.items()}, cfg,
                 str(tmp_path / "ckpt"))
    model = load_model(str(tmp_path / "ckpt"), device="cpu",
                       dtype=torch.float32)
    assert isinstance(model, SadupelForCausalLM)
    assert model.cfg.layers == cfg.layers and model.cfg.runs == cfg.runs


@pytest.mark.parametrize("layer,field,value", [
    (0, "kv_heads", 4), (0, "conv", 0), (0, "rot", {"dims": 14, "base": 9.0}),
    (1, "rot", {"dims": 7, "base": 9.0})])
def test_bad_mixers_are_refused(layer, field, value):
    cj = cfg_mixed()
    cj["layers"][layer]["mixer"][field] = value
    with pytest.raises(ValueError):
        SadupelConfig.from_json(cj)


@pytest.mark.parametrize("router", [
    {"experts": 7, "top": 2, "groups": {"count": 2, "keep": 1}},
    {"experts": 6, "top": 4, "groups": {"count": 2, "keep": 1}},
    {"experts": 6, "top": 1, "groups": {"count": 2, "keep": 3}},
    {"experts": 3, "top": 5, "identity": 1}])
def test_bad_routers_are_refused(router):
    cj = cfg_mixed()
    cj["layers"][0]["mlp"]["router"] = router
    with pytest.raises(ValueError):
        SadupelConfig.from_json(cj)


def test_cache_layout_per_pass():
    """Every pass has pages and convolution inputs; the previous token sits
    once, as an integer, in the first run's entry."""
    cfg = SadupelConfig.from_json(cfg_mixed())
    lay = cfg.cache_layout()
    assert [r[0] for r in cfg.runs] == [0, 1, 2, 1, 2, 1, 2, 3]
    assert [n["kv"] for n in lay] == [
        (3, 12, 20)] + [(1, 16, 8), (3, 8, 12)] * 3 + [(2, 20, 4)]
    assert lay[0]["state"]["conv"][0] == (3, 6 * 12 + 3 * 32)
    assert "prev" in lay[0]["state"] and "prev" not in lay[1]["state"]
    m = SadupelForCausalLM(cfg, dtype=torch.float32)
    c = m.make_cache(3, 8, 2, "cpu", torch.float32)
    assert c.state["prev"][0].dtype == torch.int32
    assert c.k[6].shape == (3, 3, 8, 8) and c.v[6].shape == (3, 3, 8, 12)
    assert len(c.state["conv"]) == 8


def test_named_configs_build_and_step():
    from agentfield_amd.models import CONFIGS
    cfg = CONFIGS["sadupel-tiny"]
    eng = LLMEngine(cfg, device="cpu", dtype=torch.float32, page_size=8,
                    num_pages=32, max_num_seqs=2, enable_graphs=False,
                    eos_id=-1)
    out = eng.generate([[1, 2, 3, 4, 5]], SamplingParams(max_tokens=4,
                                                         ignore_eos=True))[0]
    assert len(out) == 4 and all(0 <= t < cfg.vocab_size for t in out)
    for name, n in (("sadupel-1b", 16), ("sadupel-8b", 32)):
        assert len(CONFIGS[name].runs) == n


def test_trace_runner_subprocess(tmp_path):
    """bin/trace_run on a checkpoint directory: a mixed schedule with reuse,
    logits compared with the oracle."""
    cj = cfg_degenerate()
    w = orc.random_weights(cj, 6)
    cfg = SadupelConfig.from_json(cj)
    save_sadupel({k: v.to(torch.bfloat16) for k, v in w.items()}, cfg,
                 str(tmp_path / "m"))
    a, b = tokens_for(cj, 70, 30), tokens_for(cj, 9, 31)
    steps = [
        {"step": 0, "entries": [{"id": "a", "tokens": a[:50], "want": [49]},
                                {"id": "b", "tokens": b[:2], "want": []}],
         "end": []},
        {"step": 1, "entries": [{"id": "a", "tokens": a[50:51], "want": [0]},
                                {"id": "b", "tokens": b[2:], "want": [0, 6]}],
         "end": ["b"]},
        {"step": 2, "entries": [{"id": "a", "tokens": a[51:], "want": [18]}],
         "end": ["a"]}]
    r = subprocess.run(
        [sys.executable, str(REPO / "bin" / "trace_run"), "--model",
         str(tmp_path / "m"), "--dtype", "float32", "--out",
         str(tmp_path / "o"), "--max-tokens", "128", "--device", "cpu"],
        input="\n".join(json.dumps(s) for s in steps) + "\n",
        capture_output=True, text=True, timeout=300)
    assert r.returncode == 0, r.stderr
    assert [ln for ln in r.stdout.split("\n") if ln.startswith("done")] == \
        ["done 0", "done 1", "done 2"]
    import numpy as np
    wa, wb = orc.forward(a, w, cj), orc.forward(b, w, cj)
    V = cj["vocab"]
    for step, rows in ((0, [wa[49]]), (1, [wa[50], wb[2], wb[8]]),
                       (2, [wa[69]])):
        got = torch.from_numpy(np.fromfile(str(tmp_path / "o" / f"{step}.f32"),
                                           dtype="<f4").reshape(-1, V))
        assert rel_err(got, torch.stack(rows)) < 2e-4
