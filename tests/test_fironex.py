"""Fironex (differential attention, shared latents with per-head gates,
real-gated linear recurrence, layer norms on both sides of every sublayer,
xIELU) against the plain float64 oracle in fironex_oracle.py: every mechanism
alone, then whole models through the engine's cache, state slots, batching,
scheduler and generation.

Each test runs on the CPU op path and, marked gpu, on the gfx950 kernels.
fp32 runs are held to rounding-level agreement; bf16 runs to bf16 rounding.
"""
import json
import math
import subprocess
import sys
from pathlib import Path
from types import SimpleNamespace

import pytest
import torch

sys.path.insert(0, str(Path(__file__).resolve().parent))

import fironex_oracle as orc  # noqa: E402
from agentfield_amd.engine import LLMEngine, SamplingParams  # noqa: E402
from agentfield_amd.models import load_model  # noqa: E402
from agentfield_amd.models.fironex import (DiffAttention,  # noqa: E402
                                           DiffAttnSpec, FironexConfig,
                                           FironexForCausalLM,
                                           GatedRecurrence, RglruSpec,
                                           save_fironex)
from agentfield_amd.models.fugevik import (LatentAttention,  # noqa: E402
                                           LatentAttnSpec)
from agentfield_amd.ops import seqmix as sm  # noqa: E402

REPO = Path(__file__).resolve().parent.parent
DEVICES = ["cpu", pytest.param("cuda", marks=pytest.mark.gpu)]
DTYPES = [torch.float32, torch.bfloat16]
F64 = torch.float64


# ------------------------------------------------------------ model zoo
def _dense(ff):
    return {"kind": "dense", "ff": ff}


def cfg_mixed():
    """Unequal sizes everywhere; a recurrent layer first; grouped K/V heads;
    two pairs of latent layers sharing latents, one pair apart from each
    other; a layer without feed-forward in the middle; windows shorter than
    the prompts; partial rotation, with and without frequency scaling."""
    rec = {"type": "rglru", "mlp": _dense(40),
           "mixer": {"width": 36, "blocks": 3, "conv": 4}}
    diff = {"type": "attention", "mlp": _dense(72), "mixer": {
        "heads": 6, "kv_heads": 3, "dim": 12, "vdim": 20, "scale": 0.31,
        "diff": 0.35, "mask": {"size": 23},
        "rot": {"dims": 8, "base": 300.0, "scaling": {
            "factor": 3.0, "low": 1.0, "high": 6.0, "original": 90}}}}
    lat = {"type": "latent_attention", "mlp": None, "mixer": {
        "heads": 5, "dim": 12, "rot_dim": 8, "vdim": 20, "kv_rank": 28,
        "scale": 0.27, "rot": {"dims": 8, "base": 500.0}}}
    shared = {"type": "latent_attention", "mlp": _dense(24), "mixer": {
        "heads": 3, "dim": 20, "rot_dim": 8, "vdim": 8, "kv_rank": 28,
        "scale": 0.21, "rot": {"dims": 8, "base": 500.0}, "kv_from": 2}}
    diff2 = {"type": "attention", "mlp": None, "mixer": dict(
        diff["mixer"], heads=4, kv_heads=1, vdim=8, diff=0.7,
        mask={"size": 40}, rot={"dims": 12, "base": 50.0})}
    far = {"type": "latent_attention", "mlp": _dense(16), "mixer": dict(
        shared["mixer"], heads=2, vdim=12)}
    rec2 = {"type": "rglru", "mlp": None,
            "mixer": {"width": 24, "blocks": 1, "conv": 2}}
    return {"architecture": "Fironex", "vocab": 96, "width": 48,
            "residual_mult": 0.45,
            "layers": [rec, diff, lat, shared, diff2, far, rec2],
            "norm": {"eps": 1e-5}}


def cfg_degenerate():
    """Values a model may happen to make equal or 1: one head, kv_heads ==
    heads, dim == vdim, one tap, blocks of one channel, multiplier 1, scale 1,
    no window, no rotation, full-width rotation."""
    d0 = {"type": "attention", "mlp": _dense(16), "mixer": {
        "heads": 1, "kv_heads": 1, "dim": 8, "vdim": 8, "scale": 1.0,
        "diff": 0.0}}
    l0 = {"type": "latent_attention", "mlp": _dense(8), "mixer": {
        "heads": 1, "dim": 8, "rot_dim": 8, "vdim": 8, "kv_rank": 8,
        "scale": 1.0, "rot": {"dims": 8, "base": 10000.0}}}
    r0 = {"type": "rglru", "mlp": _dense(32),
          "mixer": {"width": 8, "blocks": 8, "conv": 1}}
    d1 = {"type": "attention", "mlp": _dense(16), "mixer": {
        "heads": 2, "kv_heads": 2, "dim": 4, "vdim": 16, "scale": 0.5,
        "diff": 0.8, "mask": {"size": 1000},
        "rot": {"dims": 4, "base": 10.0}}}
    return {"architecture": "Fironex", "vocab": 40, "width": 32,
            "residual_mult": 1.0, "layers": [d0, l0, r0, d1],
            "norm": {"eps": 1e-6}}


def cfg_odd():
    """Nothing divisible by 4 or 8 (scalar kernel paths), nine query heads on
    three K/V heads, a window of one token, a latent wider than the heads,
    six taps."""
    d0 = {"type": "attention", "mlp": _dense(25), "mixer": {
        "heads": 9, "kv_heads": 3, "dim": 6, "vdim": 10, "scale": 0.41,
        "diff": 0.5, "mask": {"size": 1}, "rot": {"dims": 2, "base": 50.0}}}
    l0 = {"type": "latent_attention", "mlp": _dense(7), "mixer": {
        "heads": 3, "dim": 5, "rot_dim": 6, "vdim": 3, "kv_rank": 45,
        "scale": 0.3, "rot": {"dims": 6, "base": 90.0}}}
    r0 = {"type": "rglru", "mlp": None,
          "mixer": {"width": 35, "blocks": 5, "conv": 6}}
    l1 = {"type": "latent_attention", "mlp": None, "mixer": dict(
        l0["mixer"], heads=7, dim=9, kv_from=1)}
    d1 = {"type": "attention", "mlp": _dense(11), "mixer": dict(
        d0["mixer"], heads=3, kv_heads=1, dim=10, vdim=18,
        mask={"size": 17})}
    return {"architecture": "Fironex", "vocab": 33, "width": 30,
            "residual_mult": 0.8, "layers": [d0, l0, r0, l1, d1, r0],
            "norm": {"eps": 1e-4}}


ZOO = {"mixed": cfg_mixed, "degenerate": cfg_degenerate, "odd": cfg_odd}


def build(cfg_json, device, dtype, seed=0, page=8, pages=64, live=4,
          paced=True, graphs=False):
    w = orc.random_weights(cfg_json, seed)
    cfg = FironexConfig.from_json(cfg_json)
    cfg.max_position = 512
    model = FironexForCausalLM(cfg, device=device, dtype=dtype)
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
    median row within half of the rounding of a few layers (the unit-RMS norm
    of a difference of two nearly equal maps magnifies it in single rows)."""
    d = got.to(F64).cpu() - want
    d = d - d.mean(-1, keepdim=True)
    rows = d.pow(2).mean(-1).sqrt() / want.pow(2).mean().sqrt()
    if dtype == torch.float32:
        return float(rows.max()) < tol(dtype)
    return (float(rows.max()) < 2 * tol(dtype)
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


def fill(mod, P, pre, device, dtype):
    """A mixer module with checkpoint weights in `dtype` on `device`."""
    for p in mod.parameters():
        p.data = p.data.to(dtype)
        p.requires_grad_(False)
    mod.load(P.__getitem__, pre)
    return mod.to(device)


PORTIONS = ((0, 11), (11, 13), (13, 14), (14, 15), (15, 31), (31, 33),
            (33, 90))


# ====================================================== mechanisms alone
@pytest.mark.parametrize("device", DEVICES)
def test_kernel_groups_present(device):
    if device == "cuda":
        from agentfield_amd.ops import _lib
        for group in ("glue", "seq", "conv", "rope", "latent", "rglru"):
            assert _lib.mixgroup(group) is not None  # no eager fallback


# ------------------------------------------------------- norms, activation
@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("W", [30, 32, 1028, 2050, 8196, 17000])
def test_sandwich_norm(device, dtype, W):
    """Both halves alone and together, sublayer outputs in either dtype, a
    row mean far from zero (the variance is taken from the deviations)."""
    torch.manual_seed(W)
    T, eps, mult = 9, 1e-5, 0.37
    f = lambda t: t.to(F64)  # noqa: E731
    d = lambda t: t.to(device)  # noqa: E731
    x = torch.randn(T, W) + 40.0
    y = (torch.randn(T, W) * 3 + 7).to(dtype)
    wa, wb = ((1 + 0.2 * torch.randn(W)).to(dtype) for _ in range(2))
    want_x = f(x) + mult * orc.layer_norm(f(y), wa, eps)
    want_h = orc.layer_norm(want_x, wb, eps)
    t = 2e-5 if dtype == torch.float32 else 1e-2
    for yy in (y, y.float()):
        x1 = d(x.clone())
        h1 = sm.sandwich_norm(x1, d(yy), mult, d(wa), d(wb), eps, dtype)
        assert rel_err(x1, want_x) < 1e-6
        assert h1.dtype == dtype and rel_err(h1, want_h) < t
    x2 = d(x.clone())
    assert sm.sandwich_norm(x2, d(y), mult, d(wa), None, eps, dtype) is None
    assert rel_err(x2, want_x) < 1e-6
    h2 = sm.sandwich_norm(x2, None, mult, None, d(wb), eps, dtype)
    assert rel_err(h2, want_h) < t and rel_err(x2, want_x) < 1e-6
    rows = torch.tensor([3, 0, 8], dtype=torch.int32)
    h3 = sm.norm_rows(x2, d(wb), eps, d(rows), dtype, one_plus=False,
                      center=True)
    assert rel_err(h3, want_h[rows.long()]) < t


@pytest.mark.parametrize("device", DEVICES)
def test_sandwich_norm_many_rows(device):
    """More rows than the few-rows layout takes."""
    torch.manual_seed(1)
    T, W = 700, 2048
    x, y = torch.randn(T, W), torch.randn(T, W)
    wa, wb = 1 + 0.2 * torch.randn(W), 1 + 0.2 * torch.randn(W)
    want_x = x.to(F64) + 0.5 * orc.layer_norm(y.to(F64), wa, 1e-6)
    x1 = x.clone().to(device)
    h = sm.sandwich_norm(x1, y.to(device), 0.5, wa.to(device), wb.to(device),
                         1e-6, torch.float32)
    assert rel_err(x1, want_x) < 1e-6
    assert rel_err(h, orc.layer_norm(want_x, wb, 1e-6)) < 2e-5


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("F", [8, 13])
def test_xielu(device, dtype, F):
    z = torch.cat([torch.linspace(-30, 30, 60 * F - 2),
                   torch.tensor([0.0, -1e-3])]).view(60, F).to(dtype)
    act = torch.tensor([0.8, -1.3])
    coef = torch.tensor([float(orc.softplus(act.to(F64))[0]),
                         float(orc.softplus(act.to(F64))[1]) + 0.5])
    wide = torch.zeros(60, F + 4, dtype=dtype)
    wide[:, :F] = z                     # a strided view, as in a fused GEMM
    got = sm.xielu(wide.to(device)[:, :F], coef.to(device)).cpu().to(F64)
    want = orc.xielu(z.to(F64), act)
    err = (got - want).abs() / (want.abs() + 1e-4)
    assert float(err.max()) < (2e-5 if dtype == torch.float32 else 8e-3)


# ---------------------------------------------------------- the recurrence
def _rec_inputs(C, blocks, taps, T, dtype, seed):
    W = 20
    cfg = {"width": W, "vocab": 4, "norm": {"eps": 1e-5}, "residual_mult": 1,
           "layers": [{"type": "rglru", "mlp": None, "mixer": {
               "width": C, "blocks": blocks, "conv": taps}}]}
    P = orc.random_weights(cfg, seed)
    torch.manual_seed(seed)
    return W, cfg, P, torch.randn(T, W).to(dtype)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("shape", [(24, 3, 4), (8, 8, 1), (35, 5, 6),
                                   (130, 1, 2), (128, 2, 3), (96, 4, 4),
                                   (264, 3, 2)])
def test_recurrent_mixer_alone(device, dtype, shape):
    """State and convolution inputs carried through portions (some shorter
    than the convolution's history, single rows through the decode kernel) in
    a slot with leftovers; the other slots stay as they are."""
    C, blocks, taps = shape
    W, cfg, P, h = _rec_inputs(C, blocks, taps, 90, dtype, C)
    m = cfg["layers"][0]["mixer"]
    want = orc.rglru_mixer(h.to(F64), P, "l0.mix.", m, 1e-5)
    mod = fill(GatedRecurrence(RglruSpec(C, blocks, taps), W), P, "l0.mix.",
               device, dtype)
    cache = SimpleNamespace(
        rec={0: torch.full((3, C), 9.0, device=device)},
        state={"conv": {0: torch.full((3, max(taps - 1, 1), C), 9.0,
                                      device=device, dtype=dtype)}})
    got = []
    with torch.no_grad():
        for lo, hi in PORTIONS:
            md, pos = md_for([hi - lo], [lo], [2], device)
            got.append(mod(h[lo:hi].to(device), cache, 0, md, pos, {}).cpu())
    assert rel_err(torch.cat(got), want) < tol(dtype)
    assert float(cache.rec[0][1].min()) == 9.0
    assert float(cache.state["conv"][0][1].min()) == 9.0


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
def test_recurrence_from_the_first_token_by_decoding(device, dtype):
    """A sequence that starts with single rows: the state and the places
    before position 0 are zero whatever the slot holds; seventeen sequences
    at once, more than one workgroup's rows."""
    C, blocks, taps, B, T = 48, 2, 4, 17, 9
    W, cfg, P, _h = _rec_inputs(C, blocks, taps, 1, dtype, 3)
    m = cfg["layers"][0]["mixer"]
    torch.manual_seed(8)
    hs = torch.randn(B, T, W).to(dtype)
    mod = fill(GatedRecurrence(RglruSpec(C, blocks, taps), W), P, "l0.mix.",
               device, dtype)
    cache = SimpleNamespace(
        rec={0: torch.full((B + 1, C), -5.0, device=device)},
        state={"conv": {0: torch.full((B + 1, taps - 1, C), 5.0,
                                      device=device, dtype=dtype)}})
    got = []
    with torch.no_grad():
        for t in range(T):
            md, pos = md_for([1] * B, [t] * B, list(range(B, 0, -1)), device)
            got.append(mod(hs[:, t].to(device), cache, 0, md, pos, {}).cpu())
    got = torch.stack(got, 1)
    for b in range(B):
        want = orc.rglru_mixer(hs[b].to(F64), P, "l0.mix.", m, 1e-5)
        assert rel_err(got[b], want) < tol(dtype)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("lens", [(700, 3, 61, 257), (16, 1), (64, 63)])
def test_long_recurrence_remembers(device, dtype, lens):
    """Decays near one over unequal chunks of up to several passes of the
    scan: an early impulse is still in the state hundreds of tokens later."""
    C = 70
    torch.manual_seed(sum(lens))
    lam = torch.full((C,), -8.0) + torch.randn(C) * 0.1
    rate = (-8.0 * orc.softplus(lam.to(F64))).float()
    n = C
    wr, wi = torch.zeros(1, n, n), torch.zeros(1, n, n)
    br, bi = torch.randn(C), torch.randn(C)
    conv = torch.ones(1, C)
    xs = [(torch.randn(t, C) * 0.01).to(dtype) for t in lens]
    for x in xs:
        x[0] = 5.0
    ys = [torch.randn(t, C).to(dtype) for t in lens]
    dv = lambda t: t.to(device)  # noqa: E731
    st = torch.full((9, C), 3.0, device=device)
    cs = torch.zeros(9, 1, C, device=device, dtype=dtype)
    md, _pos = md_for(list(lens), [0] * len(lens),
                      list(range(1, len(lens) + 1)), device, page=64)
    got = sm.rglru(dv(torch.cat(xs)), None, dv(torch.cat(ys)), None,
                   dv(conv.to(dtype)), None, dv(wr.to(dtype)), dv(br),
                   dv(wi.to(dtype)), dv(bi), dv(rate), st, cs, md).cpu()
    lo = 0
    for i, (x, y) in enumerate(zip(xs, ys)):
        T = x.shape[0]
        r = torch.sigmoid(br.to(F64)).expand(T, C)
        g = torch.sigmoid(bi.to(F64)).expand(T, C)
        S = orc.gated_recurrence(x.to(F64), r, g, lam)
        want = S * orc.gelu_tanh(y.to(F64))
        assert rel_err(got[lo:lo + T], want) < tol(dtype) / 2
        assert rel_err(st[i + 1:i + 2].cpu(), S[-1:]) < \
            (1e-5 if dtype == torch.float32 else 1e-2)
        lo += T
    if lens[0] == 700:      # the impulse is most of the last state
        assert float(st[1].abs().mean()) > 0.03


# ---------------------------------------------------------------- rotation
def test_scaled_frequencies_three_regimes():
    rot = {"dims": 16, "base": 300.0,
           "scaling": {"factor": 3.0, "low": 1.0, "high": 6.0,
                       "original": 90}}
    got = sm.scaled_inv_freq(16, 300.0, rot["scaling"])
    assert torch.allclose(got, orc.frequencies(rot), rtol=1e-14, atol=0)
    ratio = (got / sm.scaled_inv_freq(16, 300.0, None)).tolist()
    assert ratio[0] == 1.0 and abs(ratio[-1] - 1 / 3) < 1e-12
    assert any(1 / 3 + 1e-6 < r < 1 - 1e-6 for r in ratio)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("geom", [(8, 4, 2, 16, 8, 6), (2, 2, 1, 8, 8, 8),
                                  (18, 6, 3, 6, 10, 2), (4, 4, 2, 70, 24, 0),
                                  (6, 2, 1, 130, 5, 64), (4, 2, 1, 200, 16, 100),
                                  (2, 2, 1, 9, 3, 4)])
def test_interleaved_rotation_and_page_append(device, dtype, geom):
    """Pairs (2i, 2i+1) on the leading dims at far positions; fewer value
    heads than key heads; K and V land in their pages."""
    H, G, Gv, dk, dv, rd = geom
    torch.manual_seed(5)
    T, page = 13, 8
    rot = {"dims": rd, "base": 700.0,
           "scaling": {"factor": 4.0, "low": 1.0, "high": 4.0,
                       "original": 64}} if rd else None
    q, k, v = (torch.randn(T, n).to(dtype)
               for n in (H * dk, G * dk, Gv * dv))
    md, pos = md_for([T], [3], [1], device)
    pos = pos + 100000                  # rotation takes the given positions
    kc = torch.zeros(40, G, page, dk, dtype=dtype, device=device)
    vc = torch.zeros(40, Gv, page, dv, dtype=dtype, device=device)
    inv = sm.scaled_inv_freq(rd, 700.0, rot["scaling"]).to(device) \
        if rd else None
    d = lambda t: t.to(device)  # noqa: E731
    got = sm.qk_rope_cache(d(q), d(k), d(v), H, G, 1e-5, kc, vc, md.slots,
                           pos, inv_freq=inv, pairs=True)
    p64 = pos.cpu().to(F64)
    wq = orc.rotate(q.to(F64).view(T, H, dk), rot, "pairs", p64)
    wk = orc.rotate(k.to(F64).view(T, G, dk), rot, "pairs", p64)
    sl = md.slots.cpu()
    gk = kc.cpu()[sl // page, :, sl % page]
    gv = vc.cpu()[sl // page, :, sl % page]
    t = 3e-6 if dtype == torch.float32 else 1e-2
    assert rel_err(got.view(T, -1), wq.reshape(T, -1)) < t
    assert rel_err(gk.reshape(T, -1), wk.reshape(T, -1)) < t
    assert torch.equal(gv.reshape(T, -1), v)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("pairs", [True, False])
@pytest.mark.parametrize("geom", [(4, 12, 8, 20, 8), (3, 5, 6, 45, 6),
                                  (2, 8, 16, 32, 8), (5, 7, 10, 9, 4),
                                  (16, 128, 64, 256, 64)])
def test_latent_rows(device, dtype, pairs, geom):
    """Latent norm, key part and query slices in both pair layouts (partial
    rotation included); without a down projection only queries are written."""
    H, du, dr, R, rd = geom
    torch.manual_seed(H)
    T, page, start = 13, 8, 3000
    rot = {"dims": rd, "base": 40.0}
    layout = "pairs" if pairs else "halves"
    q = torch.randn(T, H * (du + dr)).to(dtype)
    dkv = torch.randn(T, R + dr).to(dtype)
    w = (1 + 0.2 * torch.randn(R)).to(dtype)
    md, pos = md_for([T], [2], [1], device)
    pos = pos + start
    p64 = pos.cpu().to(F64)
    inv = sm.scaled_inv_freq(rd, 40.0).to(device)
    d = lambda t: t.to(device)  # noqa: E731
    wq = orc.rotate(q.to(F64).view(T, H, du + dr)[..., du:], rot, layout, p64)
    wc = torch.cat([orc.unit_rms(dkv.to(F64)[:, :R], 1e-5) * w.to(F64),
                    orc.rotate(dkv.to(F64)[:, None, R:], rot, layout,
                               p64)[:, 0]], 1)
    t = 3e-6 if dtype == torch.float32 else 1e-2
    for own in (True, False):
        kc = torch.full((40, 1, page, R + dr), 2.0, dtype=dtype,
                        device=device)
        qf = torch.full((T, H * (R + dr)), 6.0, dtype=dtype, device=device)
        sm.latent_prep(d(q), d(dkv) if own else None, qf,
                       d(w) if own else None, 1e-5, inv, pos, kc, md.slots,
                       H, du, pairs=pairs)
        g = qf.cpu().view(T, H, R + dr)
        assert rel_err(g[..., R:].reshape(T, -1), wq.reshape(T, -1)) < t
        assert bool((g[..., :R] == 6.0).all())      # the caller's part
        sl = md.slots.cpu()
        rows = kc.cpu()[sl // page, 0, sl % page]
        if own:
            assert rel_err(rows, wc) < t
        else:
            assert bool((kc == 2.0).all())


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,dv", [(3, 8), (5, 3), (1, 4), (4, 1)])
def test_gate_heads_per_head_and_per_element(device, dtype, H, dv):
    torch.manual_seed(H)
    T = 11
    o = torch.randn(H, T, dv).to(dtype)
    wide = torch.randn(T, H * dv + 8).to(dtype)
    want_o = o.to(F64).transpose(0, 1)
    t = 3e-6 if dtype == torch.float32 else 1e-2
    g = wide[:, :H]
    got = sm.gate_heads(o.to(device), wide.to(device)[:, :H])
    want = (want_o * torch.sigmoid(g.to(F64))[:, :, None]).reshape(T, -1)
    assert rel_err(got, want) < t
    g = wide[:, :H * dv]
    got = sm.gate_heads(o.to(device), wide.to(device)[:, :H * dv])
    want = want_o.reshape(T, -1) * torch.sigmoid(g.to(F64))
    assert rel_err(got, want) < t


# --------------------------------------------------- differential attention
def _maps_through_cache(device, dtype, q, k, v, scale, window, lam, diff,
                        schedule, gate=None, page=16, eps=1e-6):
    """q [T, H, 2, dk], k [T, G, 2, dk], v [T, G, dv] through the page append
    and ops.diff_attention, fed as the schedule's portions."""
    T, H, _, dk = q.shape
    G, dv = k.shape[1], v.shape[2]
    hpg = H // G
    ql = q.view(T, G, hpg, 2, dk).transpose(2, 3)       # [K/V head][map][head]
    kc = torch.zeros(80, 2 * G, page, dk, dtype=dtype, device=device)
    vc = torch.zeros(80, G, page, dv, dtype=dtype, device=device)
    out, lo = [], 0
    for n in schedule:
        md, pos = md_for([n], [lo], [1], device, page=page, pages_per_seq=64)
        sel = slice(lo, lo + n)
        row = lambda t: t[sel].reshape(n, -1).to(device, dtype)  # noqa: E731
        qq = sm.qk_rope_cache(row(ql), row(k), row(v), 2 * H, 2 * G, eps, kc,
                              vc, md.slots, pos)
        gg = row(gate) if gate is not None else None
        out.append(sm.diff_attention(qq, kc, vc, md, pos, scale, H, lam,
                                     diff, eps, gate=gg,
                                     window=window).cpu())
        lo += n
    return torch.cat(out).view(T, H, dv)


def _maps_oracle(q, k, v, scale, window, lam, diff, gate=None, eps=1e-6):
    a = [orc.attend(q[:, :, i].to(F64), k[:, :, i].to(F64), v.to(F64), scale,
                    window) for i in range(2)]
    o = orc.combine_maps(a[0], a[1], lam, diff, eps)
    return o if gate is None else o * torch.sigmoid(gate.to(F64))


SCHEDULES = {"whole": [150], "decoded": [40] + [1] * 110,
             "portions": [2, 3, 17, 2, 64, 30, 2, 29, 1]}


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("how", list(SCHEDULES))
@pytest.mark.parametrize("geom", [(4, 2, 16, 8, 37), (3, 1, 10, 6, 150),
                                  (2, 2, 64, 128, 0), (16, 2, 8, 24, 64),
                                  (2, 1, 72, 136, 50), (1, 1, 128, 256, 0),
                                  (1, 1, 20, 300, 0), (5, 5, 7, 9, 1)])
def test_differential_attention(device, dtype, how, geom):
    """Both maps over shared values, their combination, head norm and gate:
    tile, row and many-heads kernels, every head geometry class."""
    H, G, dk, dv, window = geom
    if how == "portions" and dk * dv > 2000:
        pytest.skip("covered by the other schedules")
    torch.manual_seed(H * dk)
    T = 150
    rnd = lambda *s: torch.randn(*s).to(dtype)  # noqa: E731
    q, k, v = rnd(T, H, 2, dk), rnd(T, G, 2, dk), rnd(T, G, dv)
    gate = rnd(T, H, dv)
    scale = 1.5 * dk ** -0.5
    want = _maps_oracle(q, k, v, scale, window, 0.6, 0.3, gate)
    got = _maps_through_cache(device, dtype, q, k, v, scale, window, 0.6, 0.3,
                              SCHEDULES[how], gate)
    assert rel_err(got.reshape(T, -1), want.reshape(T, -1)) < \
        (5e-5 if dtype == torch.float32 else 4e-2)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("how", list(SCHEDULES))
@pytest.mark.parametrize("which", [0, 1])
@pytest.mark.parametrize("loud", [0, 15, 16, 63, 64, 100])
def test_one_loud_key_at_the_window_edge(device, dtype, how, which, loud):
    """One key of one map whose score towers over the rest, and whose value
    points along one axis: heard exactly while i - j < window, with a plus
    sign through the first map and a minus sign through the second; at
    position 0 and on both sides of page borders."""
    torch.manual_seed(loud)
    T, H, G, dk, dv, window = 150, 4, 2, 16, 8, 37
    q = torch.randn(T, H, 2, dk) * 0.2
    k = torch.randn(T, G, 2, dk) * 0.2
    v = torch.randn(T, G, dv)
    q[..., 0] = 4.0
    k[..., 0] = 0.0
    k[loud, :, which, 0] = 4.0          # score 8 against about 0
    v[loud] = 0.0
    v[loud, :, 2] = 100.0
    q, k, v = (t.to(dtype) for t in (q, k, v))
    want = _maps_oracle(q, k, v, 0.5, window, 0.9, 0.25)
    got = _maps_through_cache(device, dtype, q, k, v, 0.5, window, 0.9, 0.25,
                              SCHEDULES[how])
    # around the loud key every row is ruled by it; rows that do not hear it
    # are a difference of two near-uniform averages, which magnifies rounding
    hear = [i for i in range(T) if loud <= i < loud + window]
    err = (got.to(F64) - want)[hear].abs().max()
    assert float(err) < (1e-4 if dtype == torch.float32 else 0.05)
    # unit-RMS rows: one loud axis is sqrt(dv) * (1 - diff)
    full = 0.75 * math.sqrt(dv) * (1 if which == 0 else -1)
    for i in range(loud + 2, T):
        near_full = abs(float(got[i, 0, 2]) / full - 1) < 0.1
        assert near_full == (i in hear or abs(float(want[i, 0, 2]) / full - 1)
                             < 0.1), i
    for i in (loud + window - 1, loud + window):       # last in, first out
        if i < T:
            assert (float(want[i, 0, 2] / full) > 0.9) == (i in hear)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("how", ["whole", "decoded"])
@pytest.mark.parametrize("loud,window", [(3, 0), (101, 300), (255, 300),
                                         (256, 300)])
def test_loud_key_far_back(device, dtype, how, loud, window):
    """Hundreds of keys back, single rows cutting their keys over several
    workgroups, the window's last and first row on either side."""
    torch.manual_seed(loud)
    T, H, G, dk, dv = 600, 2, 1, 32, 16
    q = torch.randn(T, H, 2, dk) * 0.2
    k = torch.randn(T, G, 2, dk) * 0.2
    v = torch.randn(T, G, dv)
    q[..., 0] = 5.0
    k[..., 0] = 0.0
    k[loud, :, 0, 0] = 5.0              # score 12.5
    v[loud] = 0.0
    v[loud, :, 1] = 50.0
    q, k, v = (t.to(dtype) for t in (q, k, v))
    sched = [T] if how == "whole" else [loud + 290] + [1] * 20 + \
        ([T - loud - 310] if T > loud + 310 else [])
    got = _maps_through_cache(device, dtype, q, k, v, 0.5, window, 0.8, 0.4,
                              sched)
    full = 0.6 * math.sqrt(dv)
    for i in range(loud + 280, min(T, loud + 320)):
        hears = window <= 0 or i - loud < window
        assert (float(got[i, 1, 1]) / full > 0.95) == hears, i


def test_map_weight_and_combination_constants():
    """lambda from the four vectors, and (1 - diff) on the unit-RMS heads."""
    cfg = cfg_mixed()
    P = orc.random_weights(cfg, 3)
    m = cfg["layers"][1]["mixer"]
    mod = DiffAttention(DiffAttnSpec(
        m["heads"], m["kv_heads"], m["dim"], m["vdim"], m["scale"],
        m["diff"]), cfg["width"], 1e-5)
    mod = fill(mod, P, "l1.mix.", "cpu", torch.float32)
    want = float(orc.map_weight(P, "l1.mix.", m["diff"]))
    assert abs(mod.lam - want) < 1e-9 and abs(mod.lam - m["diff"]) > 1e-3
    a = torch.randn(5, 2, 6, dtype=F64)
    o = orc.combine_maps(a, torch.zeros_like(a), want, 0.25, 0.0)
    assert torch.allclose(o.pow(2).mean(-1).sqrt(),
                          torch.full((5, 2), 0.75, dtype=F64))


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("heads,kv_heads", [(6, 3), (4, 4), (8, 1)])
def test_diff_mixer_alone(device, dtype, heads, kv_heads):
    """The module: projections with the query rows regrouped, rotation, gate
    and output, in portions and single rows, sequences of equal length in two
    slots of pages."""
    W, T = 24, 90
    mspec = {"heads": heads, "kv_heads": kv_heads, "dim": 12, "vdim": 8,
             "scale": 0.3, "diff": 0.4, "mask": {"size": 20},
             "rot": {"dims": 6, "base": 60.0}}
    cfg = {"width": W, "vocab": 4, "norm": {"eps": 1e-5}, "residual_mult": 1,
           "layers": [{"type": "attention", "mlp": None, "mixer": mspec}]}
    P = orc.random_weights(cfg, 5)
    torch.manual_seed(11)
    h = torch.randn(T, W).to(dtype)
    want = orc.diff_attention(h.to(F64), P, "l0.mix.", mspec, 1e-5)
    spec = FironexConfig.from_json(cfg).layers[0].mixer
    mod = fill(DiffAttention(spec, W, 1e-5), P, "l0.mix.", device, dtype)
    cache = SimpleNamespace(
        k={0: torch.zeros(40, 2 * kv_heads, 8, 12, dtype=dtype,
                          device=device)},
        v={0: torch.zeros(40, kv_heads, 8, 8, dtype=dtype, device=device)})
    got = []
    with torch.no_grad():
        for lo, hi in PORTIONS:
            md, pos = md_for([hi - lo], [lo], [1], device)
            got.append(mod(h[lo:hi].to(device), cache, 0, md, pos, {}).cpu())
    # a head's difference of two maps is normed to unit RMS, small or not:
    # in bf16 the rows where it is small carry a magnified rounding
    assert rel_err(torch.cat(got), want) < \
        (tol(dtype) if dtype == torch.float32 else 0.16)


# ---------------------------------------------------------- latent sharing
@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("heads", [1, 5, 16])
def test_shared_latents(device, dtype, heads):
    """A layer with latents of its own and one that reads its pages through
    other up-projections, head count and sizes, against per-head keys and
    values."""
    W, T, R, dr = 24, 90, 28, 8
    own = {"heads": heads, "dim": 12, "rot_dim": dr, "vdim": 20,
           "kv_rank": R, "scale": 0.3, "rot": {"dims": dr, "base": 60.0}}
    oth = dict(own, heads=heads + 2, dim=6, vdim=4, kv_from=0)
    cfg = {"width": W, "vocab": 4, "norm": {"eps": 1e-5}, "residual_mult": 1,
           "layers": [{"type": "latent_attention", "mlp": None, "mixer": m}
                      for m in (own, oth)]}
    P = orc.random_weights(cfg, 7)
    torch.manual_seed(12)
    h0, h1 = torch.randn(T, W).to(dtype), torch.randn(T, W).to(dtype)
    lat = orc.latents(h0.to(F64), P, "l0.mix.", own, 1e-5)
    want = [orc.latent_attention(h0.to(F64), P, "l0.mix.", own, 1e-5, lat),
            orc.latent_attention(h1.to(F64), P, "l1.mix.", oth, 1e-5, lat)]
    specs = [ls.mixer for ls in FironexConfig.from_json(cfg).layers]
    mods = [fill(LatentAttention(s, W, 1e-5), P, f"l{i}.mix.", device, dtype)
            for i, s in enumerate(specs)]
    cache = SimpleNamespace(k={0: torch.zeros(40, 1, 8, R + dr, dtype=dtype,
                                              device=device)}, v={})
    got = [[], []]
    with torch.no_grad():
        for lo, hi in PORTIONS:
            md, pos = md_for([hi - lo], [lo], [1], device)
            ctx = {}
            for i, (mod, h) in enumerate(zip(mods, (h0, h1))):
                got[i].append(mod(h[lo:hi].to(device), cache, i, md, pos,
                                  ctx).cpu())
            assert len(ctx) == 1        # one rotary table for both
    for i in range(2):
        assert rel_err(torch.cat(got[i]), want[i]) < tol(dtype)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("loud", [0, 7, 8, 63, 64])
def test_loud_latent_is_heard_forever(device, dtype, loud):
    """No window: one latent row that towers over 300 others is heard by every
    later row, in prompt tiles and in single rows, on page borders too."""
    torch.manual_seed(loud)
    T, H, R, dr, page = 300, 16, 24, 8, 8
    q = torch.randn(T, H * (R + dr)) * 0.1
    q.view(T, H, R + dr)[..., 0] = 4.0
    rows = torch.randn(T, R + dr) * 0.1
    rows[:, 0] = 0.0
    rows[loud, 0] = 6.0
    rows[loud, 3] = 9.0
    kc = torch.zeros(50, 1, page, R + dr, dtype=dtype, device=device)
    md, pos = md_for([T], [0], [1], device, page=page, pages_per_seq=40)
    sl = md.slots
    kc[sl // page, 0, sl % page] = rows.to(device, dtype)
    qd = q.to(device, dtype)
    whole = sm.masked_attention(qd, kc, None, md, pos, 0.6, H, v_width=R)
    for i in (loud, loud + 1, 200, 299):
        m1, p1 = md_for([1], [i], [1], device, page=page, pages_per_seq=40)
        one = sm.masked_attention(qd[i:i + 1], kc, None, m1, p1, 0.6, H,
                                  v_width=R)
        for o in (whole[i], one[0]):
            assert float(o.view(H, R)[:, 3].float().min()) > 8.0
    if loud:
        assert float(whole[loud - 1].view(H, R)[:, 3].float().max()) < 1.0


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
def test_far_token_through_latents_and_state(device, dtype):
    """A token 300 positions back, far outside every window, still moves the
    logits, and identically however the prompt in between was cut."""
    cj = cfg_mixed()
    eng, w = build(cj, device, dtype, pages=100)
    a = tokens_for(cj, 310, 5)
    b = list(a)
    b[4] = (a[4] + 1) % cj["vocab"]
    wa, wb = orc.forward(a, w, cj), orc.forward(b, w, cj)
    assert rel_err(wa[-1:], wb[-1:]) > 1e-3          # the oracle hears it
    cuts = [3, 61, 2, 100, 1, 1, 77, 64, 1]
    got = run_schedule(eng, {"a": a, "b": b},
                       [[("a", c), ("b", c)] for c in cuts])
    assert model_close(got["a"], wa, dtype)
    assert model_close(got["b"], wb, dtype)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
def test_greedy_generation_through_scheduler(device, dtype):
    """engine.generate: the scheduler's batched prefill, (on GPU) the
    graph-captured decode step and the sampler reproduce the oracle's greedy
    continuation of unequal prompts; a second batch replays the same graphs
    over reused pages and slots."""
    cj = cfg_mixed()
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
        cfg = FironexConfig.from_json(make())
        again = FironexConfig.from_json(cfg.to_json())
        assert again.layers == cfg.layers and again.eps == cfg.eps
        assert again.residual_mult == cfg.residual_mult
    cj = cfg_mixed()
    w = orc.random_weights(cj, 4)
    cfg = FironexConfig.from_json(cj)
    save_fironex({k: v.to(torch.bfloat16) for k, v in w.items()}, cfg,
                 str(tmp_path / "ckpt"))
    model = load_model(str(tmp_path / "ckpt"), device="cpu",
                       dtype=torch.float32)
    assert isinstance(model, FironexForCausalLM)
    assert model.cfg.layers == cfg.layers


@pytest.mark.parametrize("change", [
    {"kv_from": 1}, {"kv_from": 5}, {"kv_from": 3}, {"kv_rank": 24},
    {"rot_dim": 12}, {"rot": {"dims": 4, "base": 500.0}},
    {"rot": {"dims": 8, "base": 50.0}}])
def test_bad_sharing_is_refused(change):
    cj = cfg_mixed()
    cj["layers"][5]["mixer"].update(change)
    with pytest.raises(ValueError):
        FironexConfig.from_json(cj)


def test_pages_of_both_key_maps():
    """Layout bytes: two key heads per value head, one latent row, nothing for
    a sharing layer."""
    cfg = FironexConfig.from_json(cfg_mixed())
    lay = cfg.cache_layout()
    assert lay[1]["kv"] == ((6, 3), 12, 20)
    assert lay[2]["kv"] == (1, 36, 0) and lay[3]["kv"] is None
    m = FironexForCausalLM(cfg, dtype=torch.float32)
    assert m.cache_bytes_per_page(8) == 8 * 4 * (
        6 * 12 + 3 * 20 + 36 + 2 * 12 + 8)
    c = m.make_cache(3, 8, 2, "cpu", torch.float32)
    assert c.k[1].shape == (3, 6, 8, 12) and c.v[1].shape == (3, 3, 8, 20)


def test_named_configs_build_and_step():
    from agentfield_amd.models import CONFIGS
    cfg = CONFIGS["fironex-tiny"]
    eng = LLMEngine(cfg, device="cpu", dtype=torch.float32, page_size=8,
                    num_pages=32, max_num_seqs=2, enable_graphs=False,
                    eos_id=-1)
    out = eng.generate([[1, 2, 3, 4, 5]], SamplingParams(max_tokens=4,
                                                         ignore_eos=True))[0]
    assert len(out) == 4 and all(0 <= t < cfg.vocab_size for t in out)


def test_trace_runner_subprocess(tmp_path):
    """bin/trace_run on a checkpoint directory: a mixed schedule with reuse,
    logits compared with the oracle."""
    cj = cfg_degenerate()
    w = orc.random_weights(cj, 6)
    cfg = FironexConfig.from_json(cj)
    save_fironex({k: v.to(torch.bfloat16) for k, v in w.items()}, cfg,
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
