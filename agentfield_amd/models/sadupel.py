"""Parallel decoders with looped layers: the Sadupel design.

A Sadupel model is a stack of layers `x <- x + m (mixer(h) + ff(h))`, h =
norm1(x), on an fp32 residual: both sublayers read one RMSNorm.  A span of
layers may run several times with the same weights, each pass with its own
cache and state and a learned vector added in front of it.  The embedding adds
a row of a second table that is looked up by the (previous token, token) pair.

  * mixer — grouped-query softmax attention whose q, k and v pass a short
    causal convolution, RMSNorm over the whole q and k rows, rotate-half
    rotary positions (frequencies optionally divided by a factor), soft-capped
    scores, a learned sink per head in the softmax denominator, one
    output-gate logit per head
  * ff — mixture of squared-ReLU units behind a softmax router with score
    correction and groups (models/zudisun.py: RoutedExperts), identity experts
    among the choices, an always-on shared unit

A layer's projections of h are one matrix and its output projections another:
`w_in` holds [q | k | v | gate | shared up | experts' up] as rows, `w_out` [o |
shared down | experts' down] as columns, so a decode step is one GEMM in, one
GEMM out, and a prompt portion runs the leading blocks of both for all rows
and the experts' blocks for the rows that chose them.

Every mechanism is parameterised by its spec on the sequence-mixer op set
(ops/seqmix.py): gfx950 kernels on GPU, vendor GEMMs for projections.  Pages,
convolution inputs and the previous token live in `HybridCache`; the engine's
scheduler hands out pages and state slots.
"""
from __future__ import annotations

import json
from dataclasses import dataclass, field
from pathlib import Path
from typing import Callable

import torch
from torch import nn

from ..ops import seqmix as sm
from .hybrid import HybridCache
from .zudisun import RoutedExperts, RoutedSpec


# ------------------------------------------------------------------ specs
@dataclass
class ConvAttnSpec:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    conv: int                   # taps of the q / k / v convolutions
    softcap: float = 0.0        # 0: none
    rot_dims: int = 0
    rot_base: float = 10000.0
    rot_scaling: dict | None = None


@dataclass
class SLayerSpec:
    mixer: ConvAttnSpec
    mlp: RoutedSpec | None = None


@dataclass
class PairTable:
    """A second embedding table, one row per hashed token pair and a last row
    for a sequence's first token."""
    buckets: int
    mul_prev: int
    mul_cur: int


@dataclass
class SadupelConfig:
    name: str = "sadupel"
    vocab_size: int = 512
    width: int = 256
    layers: list = field(default_factory=list)
    loop_start: int = 0
    loop_stop: int = 0
    loop_times: int = 1
    pairs: PairTable | None = None
    eps: float = 1e-6
    residual_mult: float = 1.0
    max_position: int = 8192    # serving limit (block-table width)

    architecture = "Sadupel"
    # engine-facing traits
    stateful = True
    num_kv_heads = 1
    sliding_window = 0          # every earlier key is seen

    def __post_init__(self):
        for i, ls in enumerate(self.layers):
            m, f = ls.mixer, ls.mlp
            if m.heads % m.kv_heads:
                raise ValueError(f"layer {i}: heads must be a multiple of "
                                 "kv_heads")
            if m.conv < 1:
                raise ValueError(f"layer {i}: a convolution needs a tap")
            if m.rot_dims % 2 or m.rot_dims > m.dim:
                raise ValueError(f"layer {i}: rotated dims must be even and "
                                 "inside the head")
            if f is None:
                continue
            n = f.experts + f.identity
            if f.groups and (n % f.groups or not 1 <= f.keep <= f.groups):
                raise ValueError(f"layer {i}: groups must divide the router's "
                                 "outputs")
            if not 1 <= f.top <= (n // f.groups * f.keep if f.groups else n):
                raise ValueError(f"layer {i}: more choices than experts")
        if self.loop_stop > len(self.layers) or self.loop_start < 0:
            raise ValueError("the loop reaches past the layers")

    @property
    def num_experts(self) -> int:
        return max([ls.mlp.experts for ls in self.layers
                    if ls.mlp is not None] or [1])

    @property
    def has_loop(self) -> bool:
        return self.loop_stop > self.loop_start and self.loop_times >= 1

    @property
    def runs(self) -> list[tuple[int, int | None]]:
        """Execution order as (layer index, pass index; None outside of the
        loop); a looped layer appears once per pass."""
        n = len(self.layers)
        if not self.has_loop:
            return [(i, None) for i in range(n)]
        a, b = self.loop_start, self.loop_stop
        return [(i, None) for i in range(a)] + \
            [(i, t) for t in range(self.loop_times) for i in range(a, b)] + \
            [(i, None) for i in range(b, n)]

    def build_model(self, device="cpu", dtype=torch.bfloat16):
        return SadupelForCausalLM(self, device=device, dtype=dtype)

    def cache_layout(self) -> list:
        """What every layer run keeps between steps (HybridCache); the first
        run's entry also holds the sequence's previous token."""
        out = []
        for run, (li, _t) in enumerate(self.runs):
            m = self.layers[li].mixer
            state = {"conv": ((max(m.conv - 1, 1), m.heads * m.dim
                               + m.kv_heads * (m.dim + m.vdim)), "model")}
            if run == 0 and self.pairs is not None:
                state["prev"] = ((1,), "i32")
            out.append({"kv": (m.kv_heads, m.dim, m.vdim), "state": state})
        return out

    @staticmethod
    def from_json(c: dict, name: str = "sadupel") -> "SadupelConfig":
        """Read a checkpoint's config.json."""
        layers = []
        for i, lc in enumerate(c["layers"]):
            if lc["type"] != "attention":
                raise ValueError(f"layer {i}: unknown type {lc['type']}")
            m = lc["mixer"]
            rot = m.get("rot") or {}
            mixer = ConvAttnSpec(
                heads=int(m["heads"]),
                kv_heads=int(m.get("kv_heads", m["heads"])),
                dim=int(m["dim"]), vdim=int(m.get("vdim", m["dim"])),
                scale=float(m["scale"]), conv=int(m["conv"]),
                softcap=float(m.get("softcap") or 0.0),
                rot_dims=int(rot.get("dims", 0)),
                rot_base=float(rot.get("base", 10000.0)),
                rot_scaling=dict(rot["scaling"])
                if rot.get("scaling") else None)
            mlp = lc.get("mlp")
            ff = None
            if mlp is not None:
                if mlp.get("kind", "moe") != "moe":
                    raise ValueError(
                        f"layer {i}: unknown mlp kind {mlp['kind']}")
                r = mlp["router"]
                g = r.get("groups") or {}
                ff = RoutedSpec(
                    experts=int(r["experts"]), top=int(r["top"]),
                    ff=int(mlp["expert"]["ff"]), act="relu2",
                    score="softmax", renorm=False,
                    groups=int(g.get("count", 0)), keep=int(g.get("keep", 0)),
                    group_top=1, identity=int(r.get("identity") or 0),
                    shared_ff=int((mlp.get("shared") or {}).get("ff", 0)))
            layers.append(SLayerSpec(mixer=mixer, mlp=ff))
        lp = c.get("loop") or {}
        b = (c.get("embedding") or {}).get("bigram")
        return SadupelConfig(
            name=name, vocab_size=int(c["vocab"]), width=int(c["width"]),
            layers=layers, loop_start=int(lp.get("start", 0)),
            loop_stop=int(lp.get("stop", 0)),
            loop_times=int(lp.get("times", 1)),
            pairs=PairTable(int(b["buckets"]), int(b["mul_prev"]),
                            int(b["mul_cur"])) if b else None,
            eps=float(c["norm"]["eps"]),
            residual_mult=float(c.get("residual_mult", 1.0)))

    def to_json(self) -> dict:
        layers = []
        for ls in self.layers:
            m, f = ls.mixer, ls.mlp
            mixer = {"conv": m.conv, "dim": m.dim, "heads": m.heads,
                     "kv_heads": m.kv_heads, "scale": m.scale,
                     "vdim": m.vdim}
            if m.softcap > 0:
                mixer["softcap"] = m.softcap
            if m.rot_dims > 0:
                mixer["rot"] = {"base": m.rot_base, "dims": m.rot_dims}
                if m.rot_scaling:
                    mixer["rot"]["scaling"] = dict(m.rot_scaling)
            mlp = None
            if f is not None:
                router = {"experts": f.experts, "top": f.top}
                if f.identity:
                    router["identity"] = f.identity
                if f.groups:
                    router["groups"] = {"count": f.groups, "keep": f.keep}
                mlp = {"expert": {"ff": f.ff}, "kind": "moe",
                       "router": router}
                if f.shared_ff:
                    mlp["shared"] = {"ff": f.shared_ff}
            layers.append({"mixer": mixer, "mlp": mlp, "type": "attention"})
        out = {"architecture": self.architecture, "layers": layers,
               "norm": {"eps": self.eps},
               "residual_mult": self.residual_mult,
               "vocab": self.vocab_size, "width": self.width}
        if self.has_loop:
            out["loop"] = {"start": self.loop_start, "stop": self.loop_stop,
                           "times": self.loop_times}
        if self.pairs is not None:
            p = self.pairs
            out["embedding"] = {"bigram": {
                "buckets": p.buckets, "mul_cur": p.mul_cur,
                "mul_prev": p.mul_prev}}
        return out


# ----------------------------------------------------------------- mixer
class ConvRopeAttention(nn.Module):
    """The attention mixer between its projections, which sit in the layer's
    matrices: convolution, whole-row norms, rotation and page append in
    ops.conv_qk_rope_cache; scores, cap, sink and the heads' gates in
    ops.masked_attention."""

    def __init__(self, spec: ConvAttnSpec, eps: float):
        super().__init__()
        s = self.spec = spec
        self.eps = eps
        self.nq, self.nk = s.heads * s.dim, s.kv_heads * s.dim
        self.nqkv = self.nq + self.nk + s.kv_heads * s.vdim
        self.nout = s.heads * s.vdim
        self.conv = nn.Parameter(torch.empty(s.conv, self.nqkv))  # tap-major
        self.q_norm = nn.Parameter(torch.empty(self.nq))
        self.k_norm = nn.Parameter(torch.empty(self.nk))
        self.register_buffer("sink", torch.zeros(s.heads,
                                                 dtype=torch.float32))
        self.register_buffer(
            "inv_freq", sm.scaled_inv_freq(s.rot_dims, s.rot_base,
                                           s.rot_scaling)
            if s.rot_dims > 0 else None)

    def in_rows(self) -> int:
        """Rows of [q | k | v | gate logits]."""
        return self.nqkv + self.spec.heads

    def forward(self, p, cache: HybridCache, run: int, md, positions, ctx,
                out):
        """p: the projections of the layer's input; writes the gated heads to
        out [T, heads * vdim]."""
        s = self.spec
        tab = None
        if self.inv_freq is not None:
            # layers that rotate alike share the step's cos / sin table
            tab = sm.step_rotary(ctx, positions, self.inv_freq, s.rot_dims,
                                 s.rot_base, s.rot_scaling)
        q = sm.conv_qk_rope_cache(
            p[:, :self.nqkv], self.conv, cache.state["conv"][run], md,
            s.heads, s.kv_heads, self.eps, cache.k[run], cache.v[run],
            q_norm=self.q_norm, k_norm=self.k_norm, rot_tab=tab)
        sm.masked_attention(
            q, cache.k[run], cache.v[run], md, positions, s.scale, s.heads,
            sink=self.sink, softcap=s.softcap,
            gate=p[:, self.nqkv:self.nqkv + s.heads], out=out)

    def load(self, get: Callable[[str], torch.Tensor], pre: str):
        def put(dst, src):
            dst.copy_(src.to(dst.device, dst.dtype))
        put(self.conv, torch.cat([get(pre + n + ".conv") for n in "qkv"], 0)
            .t().contiguous())
        put(self.q_norm, get(pre + "q.norm"))
        put(self.k_norm, get(pre + "k.norm"))
        put(self.sink, get(pre + "sink"))


# ------------------------------------------------------------------- layer
class SadupelLayer(nn.Module):
    def __init__(self, cfg: SadupelConfig, spec: SLayerSpec):
        super().__init__()
        W = cfg.width
        self.spec = spec
        self.norm1 = nn.Parameter(torch.empty(W))
        self.mixer = ConvRopeAttention(spec.mixer, cfg.eps)
        f = spec.mlp
        self.mlp = RoutedExperts(f, W, hosted=True) if f is not None else None
        rows = self.mixer.in_rows()
        # the units' block starts at a multiple of 8 rows
        self.u0 = rows + (-rows) % 8
        self.n_shared = f.shared_ff if f is not None else 0
        self.n_experts = f.experts * f.ff if f is not None else 0
        self.w_in = nn.Parameter(torch.empty(
            self.u0 + self.n_shared + self.n_experts, W))
        self.w_out = nn.Parameter(torch.empty(
            W, self.mixer.nout + self.n_shared + self.n_experts))

    def forward(self, h, cache: HybridCache, run: int, md, positions, ctx):
        """h: the normed input.  Returns what enters the residual: a row term
        and the experts' terms of ops.residual_norm."""
        f, T = self.spec.mlp, h.shape[0]
        no, ns = self.mixer.nout, self.n_shared
        terms: dict = {}
        static = f is not None and self.mlp.is_static(T, md)
        ff = ns + (self.n_experts if static else 0)     # units run on all rows
        wd = plan = None
        if f is not None:
            idx, wts, wd = self.mlp.route(h, static or f.identity > 0)
            if f.identity:
                terms.update(hin=h, idw=wd[:, f.experts:])
            if not static:
                plan = self.mlp.sort(idx)
        p = sm.matmul(h, self.w_in[:self.u0 + ff])
        act = torch.empty(T, no + ff, dtype=h.dtype, device=h.device)
        self.mixer(p, cache, run, md, positions, ctx, act[:, :no])
        if ff:
            sm.relu2(p[:, self.u0:self.u0 + ff], out=act[:, no:],
                     row_weight=wd if static else None, unit=f.ff, lead=ns)
        a = sm.split_k_parts(act, self.w_out) if not md.is_prefill else None
        if a is None:
            a = sm.matmul(act, self.w_out[:, :no + ff])
        if plan is not None:
            ys, pos = self.mlp.run_sorted(h, plan, self.w_in[self.u0 + ns:],
                                          self.w_out[:, no + ns:])
            if ys is not None:
                terms.update(ys=ys, pos=pos, weights=wts)
        return a, terms

    def load(self, get: Callable[[str], torch.Tensor], pre: str):
        def put(dst, src):
            dst.copy_(src.to(dst.device, dst.dtype))
        put(self.norm1, get(pre + "norm1"))
        mp, fp = pre + "mix.", pre + "mlp."
        self.mixer.load(get, mp)
        up, down = [get(mp + n) for n in ("q", "k", "v", "g")], [get(mp + "o")]
        pad = self.u0 - self.mixer.in_rows()
        if pad:
            up.append(up[0].new_zeros(pad, up[0].shape[1]))
        f = self.spec.mlp
        if f is not None:
            units = (["shared."] if f.shared_ff else []) + \
                [f"e{e}." for e in range(f.experts)]
            up += [get(fp + u + "up") for u in units]
            down += [get(fp + u + "down") for u in units]
            put(self.mlp.router, get(fp + "router"))
            put(self.mlp.correction, get(fp + "correction"))
        put(self.w_in, torch.cat(up, 0))
        put(self.w_out, torch.cat(down, 1))


class SadupelForCausalLM(nn.Module):
    # the engine asks these before wiring a model in
    needs_state_slots = True
    supports_speculation = False    # rejected drafts would need state rollback
    supports_prefix_cache = False   # convolution inputs are not in the pages

    def __init__(self, cfg: SadupelConfig, device="cpu",
                 dtype=torch.bfloat16):
        super().__init__()
        self.cfg = cfg
        W = cfg.width
        with torch.device(device):
            self.embed = nn.Parameter(torch.empty(cfg.vocab_size, W))
            self.pairs = nn.Parameter(torch.empty(cfg.pairs.buckets + 1, W)) \
                if cfg.pairs is not None else None
            self.layers = nn.ModuleList(
                [SadupelLayer(cfg, ls) for ls in cfg.layers])
            self.final_norm = nn.Parameter(torch.empty(W))
            self.head = nn.Parameter(torch.empty(cfg.vocab_size, W))
            self.register_buffer("loop_step", torch.zeros(
                max(cfg.loop_times, 1), W, dtype=torch.float32))
        for p in self.parameters():
            p.data = p.data.to(dtype)
            p.requires_grad_(False)
        self.to(device)
        self.record_runs: list | None = None  # set to [] to keep x per run

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
        dt, eps, mult = self.embed.dtype, cfg.eps, cfg.residual_mult
        if self.pairs is None:
            x = sm.embed_rows(ids, self.embed)
        else:
            x = sm.embed_pairs(ids, self.embed, self.pairs,
                               cfg.pairs.mul_prev, cfg.pairs.mul_cur,
                               cache.state["prev"][0], md)
        ctx: dict = {}          # what the layers of one step share
        # a layer's output enters the residual in the same kernel that adds
        # the next pass's vector and norms the next layer's input
        a, terms = None, {}
        for run, (li, t) in enumerate(cfg.runs):
            L = self.layers[li]
            vec = self.loop_step[t] \
                if t is not None and li == cfg.loop_start else None
            h = sm.residual_norm(x, a, mult, L.norm1, eps, dt, vec=vec,
                                 **terms)
            a, terms = L(h, cache, run, md, positions, ctx)
            if self.record_runs is not None:
                sm.residual_norm(x, a, mult, None, eps, dt, **terms)
                a, terms = None, {}
                self.record_runs.append(x.clone())
        if logit_rows is None:
            hn = sm.residual_norm(x, a, mult, self.final_norm, eps, dt,
                                  **terms)
        else:
            sm.residual_norm(x, a, mult, None, eps, dt, **terms)
            hn = sm.norm_rows(x, self.final_norm, eps, logit_rows, dt,
                              one_plus=False)
        # vocabulary-sized N: the vendor GEMM wins there at every row count
        return sm.matmul(hn, self.head, skinny=False).float()

    # -- weights ------------------------------------------------------------
    @torch.no_grad()
    def load_tensors(self, get: Callable[[str], torch.Tensor]):
        """Fill parameters from checkpoint tensors by name: 'embed', 'bigram',
        'loop.step', 'final.norm', 'head', and per layer i 'l<i>.norm1',
        'l<i>.mix.q|k|v|g|o', '.mix.q|k|v.conv', '.mix.q|k.norm', '.mix.sink',
        'l<i>.mlp.e<k>.up|down', '.mlp.shared.up|down',
        '.mlp.router|correction'."""
        def put(dst, src):
            dst.copy_(src.to(dst.device, dst.dtype))
        put(self.embed, get("embed"))
        put(self.head, get("head"))
        put(self.final_norm, get("final.norm"))
        if self.pairs is not None:
            put(self.pairs, get("bigram"))
        if self.cfg.has_loop:
            put(self.loop_step, get("loop.step"))
        for i, L in enumerate(self.layers):
            L.load(get, f"l{i}.")
        return self

    @torch.no_grad()
    def init_random(self, seed: int = 0):
        """Random weights at scales that keep activations O(1) through depth
        (benchmarks and smoke runs; not a trained model), drawn on the
        weights' own device."""
        g = torch.Generator(device=self.embed.device).manual_seed(seed)

        def rnd(t, std, mean=0.0):
            t.copy_(torch.randn(t.shape, generator=g, device=t.device,
                                dtype=t.dtype) * std + mean)
        for name, p in list(self.named_parameters()) + \
                list(self.named_buffers()):
            leaf = name.rsplit(".", 1)[-1]
            if leaf == "inv_freq":
                continue
            if leaf == "correction":
                rnd(p, 0.02)
            elif "norm" in leaf:
                rnd(p, 0.1, 1.0)
            elif leaf in ("embed", "sink"):
                rnd(p, 1.0)
            elif leaf in ("pairs", "loop_step"):
                rnd(p, 0.3)
            elif leaf == "conv":
                rnd(p, p.shape[0] ** -0.5)
            else:
                rnd(p, p.shape[1] ** -0.5)
        # the output matrix's columns are three sums side by side: o, the
        # shared unit and the experts
        for L in self.layers:
            no, f = L.mixer.nout, L.spec.mlp
            k = L.w_out.shape[1]
            L.w_out[:, :no] *= (k / no) ** 0.5
            if f is not None:
                if f.shared_ff:
                    L.w_out[:, no:no + f.shared_ff] *= \
                        (k / f.shared_ff) ** 0.5
                L.w_out[:, no + f.shared_ff:] *= (k / f.ff) ** 0.5
        return self


# ------------------------------------------------------ checkpoint reading
def load_sadupel(path: str, device="cpu", dtype=torch.bfloat16,
                 max_position: int | None = None) -> SadupelForCausalLM:
    """config.json + *.safetensors -> model on `device` in `dtype`."""
    from safetensors import safe_open
    root = Path(path)
    c = json.loads((root / "config.json").read_text())
    files = sorted(root.glob("*.safetensors"))
    handles = [safe_open(str(f), framework="pt") for f in files]
    where = {k: h for h in handles for k in h.keys()}

    def get(name):
        return where[name].get_tensor(name)
    cfg = SadupelConfig.from_json(c, name=root.name)
    if max_position is not None:
        cfg.max_position = max_position
    model = SadupelForCausalLM(cfg, device=device, dtype=dtype)
    return model.load_tensors(get).eval()


def save_sadupel(tensors: dict, cfg: SadupelConfig, path: str) -> None:
    """Write checkpoint-named tensors + config.json (tests, tooling)."""
    from safetensors.torch import save_file
    root = Path(path)
    root.mkdir(parents=True, exist_ok=True)
    save_file({k: v.contiguous() for k, v in tensors.items()},
              str(root / "model.safetensors"))
    (root / "config.json").write_text(json.dumps(cfg.to_json(), indent=1))


def _bench_config(name, width, n_layers, heads, kv_heads, dim, experts, top,
                  ff, identity, groups, keep, loop, vocab=32000, conv=4,
                  buckets=32003):
    """n_layers layers of which loop = (start, stop, times) repeat."""
    layer = SLayerSpec(
        mixer=ConvAttnSpec(
            heads=heads, kv_heads=kv_heads, dim=dim, vdim=dim,
            scale=dim ** -0.5, conv=conv, softcap=50.0, rot_dims=dim,
            rot_base=1e6, rot_scaling={"factor": 8.0}),
        mlp=RoutedSpec(
            experts=experts, top=top, ff=ff, act="relu2", score="softmax",
            renorm=False, groups=groups, keep=keep, group_top=1,
            identity=identity, shared_ff=ff))
    return SadupelConfig(
        name=name, vocab_size=vocab, width=width, layers=[layer] * n_layers,
        loop_start=loop[0], loop_stop=loop[1], loop_times=loop[2],
        pairs=PairTable(buckets, 613, 17), eps=1e-6, residual_mult=0.7)


SADUPEL_CONFIGS = {
    # a small model with every branch, for smoke runs and CPU tests
    "sadupel-tiny": _bench_config("sadupel-tiny", 128, 3, 4, 2, 32, 6, 2, 64,
                                  2, 4, 2, (1, 2, 2), vocab=384, conv=3,
                                  buckets=101),
    # same width / depth (16 layer runs) / heads as "vabedra-1b" and
    # "zudisun-1b-moe"; 16 experts of ff 2048 of which a row takes three,
    # beside the shared one and eight identity experts
    "sadupel-1b": _bench_config("sadupel-1b", 2048, 14, 16, 8, 128, 16, 3,
                                2048, 8, 4, 2, (6, 8, 2)),
    # same width / depth (32 layer runs) / heads / vocabulary as "vabedra-8b"
    "sadupel-8b": _bench_config("sadupel-8b", 4096, 30, 32, 8, 128, 16, 3,
                                3584, 8, 4, 2, (14, 16, 2), vocab=128256),
}
