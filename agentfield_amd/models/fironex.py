"""Decoders with layer norms on both sides of every sublayer: the Fironex
design.

A Fironex model is a stack of layers `x <- x + m LN(mixer(LN(x)))`, `x <- x +
m LN(ff(LN(x)))` on an fp32 residual, LN a layer norm with a weight and no
bias, m a config constant.  config.json lists the layers; each names its mixer
and a feed-forward (or none):

  * ``attention`` — differential attention: every head has two query / key
    maps over the same values, each with its own softmax; the second map's
    output is taken off the first's with one learned weight per layer, the
    difference is RMS-normed per head; interleaved rotary positions on the
    leading dims (optionally wavelength-scaled), sliding window, element-wise
    sigmoid output gate
  * ``latent_attention`` — latent attention in absorbed form
    (models/fugevik.py: LatentAttention) with rotate-half positions and one
    output-gate logit per head; a layer with `kv_from` reads another layer's
    latents through up-projections of its own
  * ``rglru`` — gated recurrent block: a GELU branch times a real-gated linear
    recurrence behind a short causal convolution, one fp32 state value per
    channel
  * feed-forward — W_down xIELU(W_up h)

Logits reuse the embedding table.  Every mechanism is a module parameterised
by its spec on the sequence-mixer op set (ops/seqmix.py): gfx950 kernels on
GPU, vendor GEMMs for projections.  Pages, recurrent states and convolution
inputs live in `HybridCache`; the engine's scheduler hands out pages and state
slots.
"""
from __future__ import annotations

import json
import math
from dataclasses import dataclass, field
from pathlib import Path
from typing import Callable

import torch
from torch import nn

from ..ops import seqmix as sm
from .fugevik import LatentAttention, LatentAttnSpec, pad_rows
from .hybrid import HybridCache

# rate of the recurrence's log decay: log a = -RGLRU_RATE * r * softplus(lam)
RGLRU_RATE = 8.0


# ------------------------------------------------------------------ specs
@dataclass
class DiffAttnSpec:
    heads: int
    kv_heads: int
    dim: int                    # query/key size of one map
    vdim: int
    scale: float
    diff: float                 # constant part of the second map's weight
    window: int = 0             # 0: every earlier key
    rot_dims: int = 0
    rot_base: float = 10000.0
    rot_scaling: dict | None = None


@dataclass
class RglruSpec:
    width: int
    blocks: int                 # blocks of the recurrence's gate matrices
    conv: int                   # convolution taps


@dataclass
class FxLayerSpec:
    kind: str                   # "attention" | "latent_attention" | "rglru"
    mixer: DiffAttnSpec | LatentAttnSpec | RglruSpec
    ff: int | None = None       # None: no feed-forward


@dataclass
class FironexConfig:
    name: str = "fironex"
    vocab_size: int = 512
    width: int = 256
    layers: list = field(default_factory=list)
    eps: float = 1e-6
    residual_mult: float = 1.0
    max_position: int = 8192    # serving limit (block-table width)

    architecture = "Fironex"
    # engine-facing traits
    stateful = True
    num_kv_heads = 1
    num_experts = 1
    sliding_window = 0          # latent layers see every earlier key

    def __post_init__(self):
        for i, ls in enumerate(self.layers):
            m = ls.mixer
            if ls.kind == "rglru" and (m.blocks < 1 or m.width % m.blocks):
                raise ValueError(f"layer {i}: width must be a multiple of "
                                 "blocks")
            if ls.kind != "latent_attention" or m.kv_from is None:
                continue
            j = m.kv_from
            if not 0 <= j < i or self.layers[j].kind != "latent_attention" \
                    or self.layers[j].mixer.kv_from is not None:
                raise ValueError(f"layer {i}: kv_from must name an earlier "
                                 "latent_attention layer with latents of its "
                                 "own")
            o = self.layers[j].mixer
            if (o.kv_rank, o.rot_dim, o.rot_dims, o.rot_base,
                    o.rot_scaling) != (m.kv_rank, m.rot_dim, m.rot_dims,
                                       m.rot_base, m.rot_scaling):
                raise ValueError(f"layer {i}: latent geometry or rotation "
                                 f"differs from layer {j}'s")

    def build_model(self, device="cpu", dtype=torch.bfloat16):
        return FironexForCausalLM(self, device=device, dtype=dtype)

    def cache_layout(self) -> list:
        """What every layer keeps between steps (HybridCache): K pages with
        two key heads per value head, key pages of latents (values inside
        them), nothing for a layer that reads another's, or a recurrent state
        and its convolution's inputs."""
        out = []
        for ls in self.layers:
            m = ls.mixer
            need = {"kv": None, "state": {}}
            if ls.kind == "attention":
                need["kv"] = ((2 * m.kv_heads, m.kv_heads), m.dim, m.vdim)
            elif ls.kind == "latent_attention":
                if m.kv_from is None:
                    need["kv"] = (1, m.kv_rank + m.rot_dim, 0)
            else:
                need["state"] = {
                    "rec": ((m.width,), "f32"),
                    "conv": ((max(m.conv - 1, 1), m.width), "model")}
            out.append(need)
        return out

    @staticmethod
    def from_json(c: dict, name: str = "fironex") -> "FironexConfig":
        """Read a checkpoint's config.json."""
        layers = []
        for i, lc in enumerate(c["layers"]):
            m = lc["mixer"]
            window = int((m.get("mask") or {}).get("size", 0))
            rot = m.get("rot") or {}
            turn = dict(rot_base=float(rot.get("base", 10000.0)),
                        rot_scaling=dict(rot["scaling"])
                        if rot.get("scaling") else None)
            if lc["type"] == "attention":
                mixer = DiffAttnSpec(
                    heads=int(m["heads"]),
                    kv_heads=int(m.get("kv_heads", m["heads"])),
                    dim=int(m["dim"]), vdim=int(m.get("vdim", m["dim"])),
                    scale=float(m["scale"]), diff=float(m["diff"]),
                    window=window, rot_dims=int(rot.get("dims", 0)), **turn)
            elif lc["type"] == "latent_attention":
                src = m.get("kv_from")
                mixer = LatentAttnSpec(
                    heads=int(m["heads"]), dim=int(m["dim"]),
                    rot_dim=int(m.get("rot_dim", 0)),
                    vdim=int(m.get("vdim", m["dim"])),
                    kv_rank=int(m["kv_rank"]), scale=float(m["scale"]),
                    window=window,
                    rot_dims=int(rot.get("dims", m.get("rot_dim", 0)))
                    if rot else 0, **turn,
                    rot_pairs=False, gate="head", sink=False,
                    kv_from=int(src) if src is not None else None)
            elif lc["type"] == "rglru":
                mixer = RglruSpec(width=int(m["width"]),
                                  blocks=int(m["blocks"]),
                                  conv=int(m["conv"]))
            else:
                raise ValueError(f"layer {i}: unknown type {lc['type']}")
            mlp = lc.get("mlp")
            if mlp is not None and mlp.get("kind", "dense") != "dense":
                raise ValueError(f"layer {i}: unknown mlp kind {mlp['kind']}")
            layers.append(FxLayerSpec(
                kind=lc["type"], mixer=mixer,
                ff=int(mlp["ff"]) if mlp is not None else None))
        return FironexConfig(
            name=name, vocab_size=int(c["vocab"]), width=int(c["width"]),
            layers=layers, eps=float(c["norm"]["eps"]),
            residual_mult=float(c.get("residual_mult", 1.0)))

    def to_json(self) -> dict:
        layers = []
        for ls in self.layers:
            m = ls.mixer
            if ls.kind == "rglru":
                mixer = {"blocks": m.blocks, "conv": m.conv, "width": m.width}
            else:
                mixer = {"dim": m.dim, "heads": m.heads, "scale": m.scale,
                         "vdim": m.vdim}
                if ls.kind == "attention":
                    mixer.update(diff=m.diff, kv_heads=m.kv_heads)
                else:
                    mixer.update(kv_rank=m.kv_rank, rot_dim=m.rot_dim)
                    if m.kv_from is not None:
                        mixer["kv_from"] = m.kv_from
                if m.window > 0:
                    mixer["mask"] = {"size": m.window}
                if m.rot_dims > 0:
                    mixer["rot"] = {"base": m.rot_base, "dims": m.rot_dims}
                    if m.rot_scaling:
                        mixer["rot"]["scaling"] = dict(m.rot_scaling)
            layers.append({
                "mixer": mixer, "type": ls.kind,
                "mlp": ({"ff": ls.ff, "kind": "dense"}
                        if ls.ff is not None else None)})
        return {"architecture": self.architecture, "layers": layers,
                "norm": {"eps": self.eps},
                "residual_mult": self.residual_mult,
                "vocab": self.vocab_size, "width": self.width}


def _f32(*shape):
    return torch.zeros(*shape, dtype=torch.float32)


def _pad8(n: int) -> int:
    return n + (-n) % 8


# ----------------------------------------------------------------- mixers
class DiffAttention(nn.Module):
    """Differential attention: [q | k | v | gate logits] from one GEMM, the
    rotation and page append in ops.qk_rope_cache (2H query and 2G key heads
    over G value heads), both softmaxes, their combination, head norm and
    gate in ops.diff_attention.  The rows of W_q are stored [K/V head][map]
    [head of the group], so that the heads sharing a key map are neighbours;
    W_k's [K/V head][map] is the checkpoint's order."""

    def __init__(self, spec: DiffAttnSpec, width: int, eps: float):
        super().__init__()
        s = self.spec = spec
        self.eps = eps
        self.nq, self.nk = 2 * s.heads * s.dim, 2 * s.kv_heads * s.dim
        self.nv, self.ng = s.kv_heads * s.vdim, s.heads * s.vdim
        self.k0 = _pad8(self.nq)
        self.v0 = self.k0 + _pad8(self.nk)
        self.g0 = self.v0 + _pad8(self.nv)
        self.w_in = nn.Parameter(torch.empty(self.g0 + _pad8(self.ng), width))
        self.o = nn.Parameter(torch.empty(width, self.ng))
        self.register_buffer(
            "inv_freq", sm.scaled_inv_freq(s.rot_dims, s.rot_base,
                                           s.rot_scaling)
            if s.rot_dims > 0 else None)
        self.lam = s.diff       # weight of the second map

    def forward(self, h, cache: HybridCache, run: int, md, positions, ctx):
        s = self.spec
        p = sm.matmul(h, self.w_in)
        tab = None
        if self.inv_freq is not None:
            tab = sm.step_rotary(ctx, positions, self.inv_freq, s.rot_dims,
                                 s.rot_base, s.rot_scaling)
        q = sm.qk_rope_cache(
            p[:, :self.nq], p[:, self.k0:self.k0 + self.nk],
            p[:, self.v0:self.v0 + self.nv], 2 * s.heads, 2 * s.kv_heads,
            self.eps, cache.k[run], cache.v[run], md.slots, positions,
            rot_tab=tab, pairs=True)
        o = sm.diff_attention(q, cache.k[run], cache.v[run], md, positions,
                              s.scale, s.heads, self.lam, s.diff, self.eps,
                              gate=p[:, self.g0:self.g0 + self.ng],
                              window=s.window)
        return sm.matmul(o, self.o)

    def load(self, get: Callable[[str], torch.Tensor], pre: str):
        s = self.spec

        def put(dst, src):
            dst.copy_(src.to(dst.device, dst.dtype))
        wq = get(pre + "q")
        wq = wq.view(s.kv_heads, s.heads // s.kv_heads, 2, s.dim, -1) \
            .transpose(1, 2).reshape(self.nq, -1)
        put(self.w_in, pad_rows([wq, get(pre + "k"), get(pre + "v"),
                                 get(pre + "g")]))
        put(self.o, get(pre + "o"))

        def dot(a, b):
            return float((get(pre + a).double() * get(pre + b).double()).sum())
        self.lam = math.exp(dot("lq1", "lk1")) - math.exp(dot("lq2", "lk2")) \
            + s.diff


class GatedRecurrence(nn.Module):
    """Griffin's recurrent block: [y | x] from one GEMM, then convolution,
    gates, recurrence and the GELU branch in ops.rglru, W_o."""

    def __init__(self, spec: RglruSpec, width: int):
        super().__init__()
        s = self.spec = spec
        C, n = s.width, s.width // s.blocks
        self.x0 = _pad8(C)
        self.w_in = nn.Parameter(torch.empty(self.x0 + _pad8(C), width))
        self.y_b = nn.Parameter(torch.empty(C))
        self.x_b = nn.Parameter(torch.empty(C))
        self.conv = nn.Parameter(torch.empty(s.conv, C))    # tap-major
        self.conv_b = nn.Parameter(torch.empty(C))
        self.ra = nn.Parameter(torch.empty(s.blocks, n, n))
        self.ri = nn.Parameter(torch.empty(s.blocks, n, n))
        self.register_buffer("ra_b", _f32(C))
        self.register_buffer("ri_b", _f32(C))
        self.register_buffer("rate", _f32(C))
        self.o = nn.Parameter(torch.empty(width, C))

    def forward(self, h, cache: HybridCache, run: int, md, positions, ctx):
        C = self.spec.width
        p = sm.matmul(h, self.w_in)
        o = sm.rglru(p[:, self.x0:self.x0 + C], self.x_b, p[:, :C], self.y_b,
                     self.conv, self.conv_b, self.ra, self.ra_b, self.ri,
                     self.ri_b, self.rate, cache.rec[run],
                     cache.state["conv"][run], md)
        return sm.matmul(o, self.o)

    def set_lam(self, lam: torch.Tensor):
        sp = torch.nn.functional.softplus(lam.double().cpu(), threshold=40.0)
        self.rate.copy_((-RGLRU_RATE * sp).float())

    def load(self, get: Callable[[str], torch.Tensor], pre: str):
        def put(dst, src):
            dst.copy_(src.to(dst.device, dst.dtype))
        put(self.w_in, pad_rows([get(pre + "y"), get(pre + "x")]))
        put(self.y_b, get(pre + "y.b"))
        put(self.x_b, get(pre + "x.b"))
        put(self.conv, get(pre + "conv").t().contiguous())
        put(self.conv_b, get(pre + "conv.b"))
        for n in ("ra", "ri"):
            put(getattr(self, n), get(pre + n))
            put(getattr(self, n + "_b"), get(pre + n + ".b").reshape(-1))
        self.set_lam(get(pre + "lam"))
        put(self.o, get(pre + "o"))


class XieluMLP(nn.Module):
    """W_down xIELU(W_up h), the activation's two numbers learned."""

    def __init__(self, ff: int, width: int):
        super().__init__()
        self.up = nn.Parameter(torch.empty(ff, width))
        self.down = nn.Parameter(torch.empty(width, ff))
        self.register_buffer("coef", _f32(2))   # z^2 factor, exponential's

    def forward(self, h):
        return sm.matmul(sm.xielu(sm.matmul(h, self.up), self.coef),
                         self.down)

    def set_act(self, act: torch.Tensor):
        c = torch.nn.functional.softplus(act.double().cpu(), threshold=40.0)
        c[1] += 0.5
        self.coef.copy_(c.float())


# ------------------------------------------------------------------- layer
class FironexLayer(nn.Module):
    def __init__(self, cfg: FironexConfig, spec: FxLayerSpec):
        super().__init__()
        W = cfg.width
        self.spec = spec
        self.norm1 = nn.Parameter(torch.empty(W))       # in front of the mixer
        self.norm1b = nn.Parameter(torch.empty(W))      # behind it
        if spec.kind == "attention":
            self.mixer = DiffAttention(spec.mixer, W, cfg.eps)
        elif spec.kind == "latent_attention":
            self.mixer = LatentAttention(spec.mixer, W, cfg.eps)
        else:
            self.mixer = GatedRecurrence(spec.mixer, W)
        if spec.ff is None:
            self.norm2 = self.norm2b = self.mlp = None
        else:
            self.norm2 = nn.Parameter(torch.empty(W))
            self.norm2b = nn.Parameter(torch.empty(W))
            self.mlp = XieluMLP(spec.ff, W)


class FironexForCausalLM(nn.Module):
    # the engine asks these before wiring a model in
    needs_state_slots = True
    supports_speculation = False    # rejected drafts would need state rollback
    supports_prefix_cache = False   # recurrent state is not page-addressable

    def __init__(self, cfg: FironexConfig, device="cpu",
                 dtype=torch.bfloat16):
        super().__init__()
        self.cfg = cfg
        with torch.device(device):
            self.embed = nn.Parameter(torch.empty(cfg.vocab_size, cfg.width))
            self.layers = nn.ModuleList(
                [FironexLayer(cfg, ls) for ls in cfg.layers])
            self.final_norm = nn.Parameter(torch.empty(cfg.width))
        for p in self.parameters():
            p.data = p.data.to(dtype)
            p.requires_grad_(False)
        self.to(device)
        self.record_runs: list | None = None  # set to [] to keep x per layer

    # -- engine interface ---------------------------------------------------
    def make_cache(self, num_pages: int, page_size: int, num_slots: int,
                   device, dtype):
        return HybridCache(self.cfg.cache_layout(), num_pages, page_size,
                           num_slots, device, dtype)

    def cache_bytes_per_page(self, page_size: int) -> int:
        return HybridCache.bytes_per_page(self.cfg.cache_layout(), page_size,
                                          self.embed.element_size())

    def forward(self, ids, positions, cache: HybridCache, md,
                logit_rows: torch.Tensor | None = None):
        """ids/positions [T] i32 -> fp32 logits [T or len(logit_rows), V]."""
        cfg = self.cfg
        dt = self.embed.dtype
        eps, mult = cfg.eps, cfg.residual_mult
        x = sm.embed_rows(ids, self.embed)
        ctx: dict = {}          # what the layers of one step share
        # a sublayer's output enters the residual in the same kernel that
        # norms the next sublayer's input
        y = w_post = None
        for run, L in enumerate(self.layers):
            h = sm.sandwich_norm(x, y, mult, w_post, L.norm1, eps, dt)
            y = L.mixer(h, cache, run, md, positions, ctx)
            w_post = L.norm1b
            if L.mlp is not None:
                h = sm.sandwich_norm(x, y, mult, w_post, L.norm2, eps, dt)
                y = L.mlp(h)
                w_post = L.norm2b
            if self.record_runs is not None:
                sm.sandwich_norm(x, y, mult, w_post, None, eps, dt)
                y = w_post = None
                self.record_runs.append(x.clone())
        if logit_rows is None:
            hn = sm.sandwich_norm(x, y, mult, w_post, self.final_norm, eps, dt)
        else:
            if y is not None:
                sm.sandwich_norm(x, y, mult, w_post, None, eps, dt)
            hn = sm.norm_rows(x, self.final_norm, eps, logit_rows, dt,
                              one_plus=False, center=True)
        # vocabulary-sized N: the vendor GEMM wins there at every row count
        return sm.matmul(hn, self.embed, skinny=False).float()

    # -- weights ------------------------------------------------------------
    @torch.no_grad()
    def load_tensors(self, get: Callable[[str], torch.Tensor]):
        """Fill parameters from checkpoint tensors by name: 'embed',
        'final.norm', and per layer i 'l<i>.norm1|norm1b|norm2|norm2b',
        'l<i>.mix.<...>', 'l<i>.mlp.up|down|act'."""
        def put(dst, src):
            dst.copy_(src.to(dst.device, dst.dtype))
        put(self.embed, get("embed"))
        put(self.final_norm, get("final.norm"))
        for i, L in enumerate(self.layers):
            pre = f"l{i}."
            put(L.norm1, get(pre + "norm1"))
            put(L.norm1b, get(pre + "norm1b"))
            L.mixer.load(get, pre + "mix.")
            if L.mlp is not None:
                put(L.norm2, get(pre + "norm2"))
                put(L.norm2b, get(pre + "norm2b"))
                put(L.mlp.up, get(pre + "mlp.up"))
                put(L.mlp.down, get(pre + "mlp.down"))
                L.mlp.set_act(get(pre + "mlp.act"))
        return self

    @torch.no_grad()
    def init_random(self, seed: int = 0):
        """Random weights at scales that keep activations O(1) through depth
        (benchmarks and smoke runs; not a trained model)."""
        g = torch.Generator(device="cpu").manual_seed(seed)

        def rnd(t, std, mean=0.0):
            t.copy_((torch.randn(t.shape, generator=g) * std + mean)
                    .to(t.dtype))
        for name, p in self.named_parameters():
            leaf = name.rsplit(".", 1)[-1]
            if "norm" in leaf:
                rnd(p, 0.1, 1.0)
            elif p.dim() == 1:
                rnd(p, 0.1)
            elif leaf == "embed":
                rnd(p, 1.0)
            elif leaf == "conv":
                rnd(p, p.shape[0] ** -0.5)
            elif leaf in ("ra", "ri", "uk"):
                rnd(p, p.shape[2] ** -0.5)
            else:
                rnd(p, p.shape[1] ** -0.5)
        for L in self.layers:
            m = L.mixer
            if isinstance(m, GatedRecurrence):
                rnd(m.ra_b, 0.5)
                rnd(m.ri_b, 0.5)
                m.set_lam(torch.randn(m.spec.width, generator=g) - 4.0)
            elif isinstance(m, DiffAttention):
                m.lam = m.spec.diff + 0.1 * float(torch.randn(1, generator=g))
            if L.mlp is not None:
                L.mlp.set_act(torch.randn(2, generator=g) * 0.5)
        return self


# ------------------------------------------------------ checkpoint reading
def load_fironex(path: str, device="cpu", dtype=torch.bfloat16,
                 max_position: int | None = None) -> FironexForCausalLM:
    """config.json + *.safetensors -> model on `device` in `dtype`."""
    from safetensors import safe_open
    root = Path(path)
    c = json.loads((root / "config.json").read_text())
    files = sorted(root.glob("*.safetensors"))
    handles = [safe_open(str(f), framework="pt") for f in files]
    where = {k: h for h in handles for k in h.keys()}

    def get(name):
        return where[name].get_tensor(name)
    cfg = FironexConfig.from_json(c, name=root.name)
    if max_position is not None:
        cfg.max_position = max_position
    model = FironexForCausalLM(cfg, device=device, dtype=dtype)
    return model.load_tensors(get).eval()


def save_fironex(tensors: dict, cfg: FironexConfig, path: str) -> None:
    """Write checkpoint-named tensors + config.json (tests, tooling)."""
    from safetensors.torch import save_file
    root = Path(path)
    root.mkdir(parents=True, exist_ok=True)
    save_file({k: v.contiguous() for k, v in tensors.items()},
              str(root / "model.safetensors"))
    (root / "config.json").write_text(json.dumps(cfg.to_json(), indent=1))


def _bench_config(name, width, ff, n_layers, heads, kv_heads, dim,
                  vocab=32000, kv_rank=256, rot_dim=64, window=1024, blocks=16,
                  conv=4):
    """Blocks of four layers: differential attention (two maps of dim / 2 per
    head, values of dim), latent attention, latent attention on the same
    latents, gated recurrence."""
    layers = []
    for i in range(n_layers):
        k = i % 4
        if k == 0:
            kind, mixer = "attention", DiffAttnSpec(
                heads=heads, kv_heads=kv_heads, dim=dim // 2, vdim=dim,
                scale=(dim // 2) ** -0.5, diff=0.8 - 0.6 * math.exp(-0.3 * i),
                window=window, rot_dims=dim // 2, rot_base=500000.0,
                rot_scaling={"factor": 8.0, "low": 1.0, "high": 4.0,
                             "original": 8192})
        elif k == 3:
            kind, mixer = "rglru", RglruSpec(width=width, blocks=blocks,
                                             conv=conv)
        else:
            kind, mixer = "latent_attention", LatentAttnSpec(
                heads=heads, dim=dim, rot_dim=rot_dim, vdim=dim,
                kv_rank=kv_rank, scale=(dim + rot_dim) ** -0.5,
                rot_dims=rot_dim, rot_base=500000.0, rot_pairs=False,
                gate="head", sink=False, kv_from=i - 1 if k == 2 else None)
        layers.append(FxLayerSpec(kind=kind, mixer=mixer, ff=ff))
    return FironexConfig(name=name, vocab_size=vocab, width=width,
                         layers=layers, eps=1e-6, residual_mult=0.5)


FIRONEX_CONFIGS = {
    # a small model with every branch, for smoke runs and CPU tests
    "fironex-tiny": _bench_config("fironex-tiny", 128, 320, 4, 4, 2, 32,
                                  vocab=384, kv_rank=48, rot_dim=16,
                                  window=40, blocks=4, conv=3),
    # same width / ff / depth / heads as "fugevik-1b", "reperax-1b" and
    # "debug-1b"
    "fironex-1b": _bench_config("fironex-1b", 2048, 8192, 16, 16, 8, 128),
    # same width / ff / depth / heads / vocabulary as "fugevik-8b" and
    # "llama-3-8b"
    "fironex-8b": _bench_config("fironex-8b", 4096, 14336, 32, 32, 8, 128,
                                vocab=128256, kv_rank=512),
}
