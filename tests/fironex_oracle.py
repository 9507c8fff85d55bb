"""Plain float64 statement of the Fironex decoder, one function per mechanism.

Whole sequences only, no cache, no batching, no kernels: every function takes
the full [T, ...] input of one sequence and loops where the definition loops.
It shares no code with the package and is the yardstick of test_fironex.py.

Tensors are looked up by checkpoint name in a dict `P` (values are cast to
float64 on use); `cfg` is the parsed config.json.
"""
import math

import torch

F64 = torch.float64


def _f(t):
    return t.to(F64)


def lin(h, P, name, bias=False):
    y = h @ _f(P[name]).t()
    return y + _f(P[name + ".b"]) if bias else y


def layer_norm(x, w, eps):
    """(x - mean) / sqrt(mean of the squared deviations + eps) * w."""
    d = x - x.mean(-1, keepdim=True)
    return d / torch.sqrt(d.pow(2).mean(-1, keepdim=True) + eps) * _f(w)


def unit_rms(x, eps):
    return x / torch.sqrt(x.pow(2).mean(-1, keepdim=True) + eps)


def gelu_tanh(z):
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi)
                                       * (z + 0.044715 * z ** 3)))


def softplus(z):
    return torch.where(z > 30.0, z,
                       torch.log1p(torch.exp(torch.clamp(z, max=30.0))))


# --------------------------------------------------- real-gated linear unit
def short_conv(x, w, b):
    """out[t, c] = b[c] + sum_j w[c, j] x[t - (taps-1-j), c]: the last column
    weighs the current token, inputs before the start are zero."""
    T, C = x.shape
    taps = w.shape[1]
    out = _f(b).repeat(T, 1)
    for t in range(T):
        for j in range(taps):
            s = t - (taps - 1 - j)
            if s >= 0:
                out[t] += _f(w)[:, j] * x[s]
    return out


def recurrence_gates(u, P, pre):
    """sigmoid of the block-diagonal maps of u [T, C]: (r, i), each [T, C]."""
    blocks, n, _ = P[pre + "ra"].shape
    r, i = torch.empty_like(u), torch.empty_like(u)
    for b in range(blocks):
        sl = slice(b * n, (b + 1) * n)
        for out, name in ((r, "ra"), (i, "ri")):
            out[:, sl] = torch.sigmoid(
                u[:, sl] @ _f(P[pre + name][b]).t()
                + _f(P[pre + name + ".b"][b]))
    return r, i


def gated_recurrence(u, r, i, lam):
    """S_t = a_t S_(t-1) + sqrt(1 - a_t^2) i_t u_t from S = 0, with log a_t =
    -8 r_t softplus(lam); every S_t."""
    T, C = u.shape
    log_a = -8.0 * r * softplus(_f(lam))
    gain = torch.sqrt(-torch.expm1(2.0 * log_a))
    S = torch.zeros(C, dtype=F64)
    out = torch.empty(T, C, dtype=F64)
    for t in range(T):
        S = torch.exp(log_a[t]) * S + gain[t] * i[t] * u[t]
        out[t] = S
    return out


def rglru_mixer(h, P, pre, m, eps):
    y = gelu_tanh(lin(h, P, pre + "y", True))
    u = short_conv(lin(h, P, pre + "x", True), P[pre + "conv"],
                   P[pre + "conv.b"])
    r, i = recurrence_gates(u, P, pre)
    return lin(gated_recurrence(u, r, i, P[pre + "lam"]) * y, P, pre + "o")


# ------------------------------------------------------------------ rotary
def frequencies(rot):
    """f_i = base^(-2i/dims); with 'scaling' {factor, low, high, original}:
    wavelength l = 2 pi / f; l < original/high keeps f, l > original/low
    gives f / factor, in between a linear blend in s = (original / l - low)
    / (high - low)."""
    dims = rot["dims"]
    out = []
    for i in range(dims // 2):
        f = float(rot["base"]) ** (-2.0 * i / dims)
        sc = rot.get("scaling")
        if sc:
            orig, fac = float(sc["original"]), float(sc["factor"])
            lo, hi = float(sc["low"]), float(sc["high"])
            l = 2.0 * math.pi / f
            if l < orig / hi:
                pass
            elif l > orig / lo:
                f = f / fac
            else:
                s = (orig / l - lo) / (hi - lo)
                f = (1.0 - s) * f / fac + s * f
        out.append(f)
    return torch.tensor(out, dtype=F64)


def rotate(x, rot, layout, positions=None):
    """Rotary positions on the first rot.dims elements of the last axis of
    x [T, H, d].  layout 'pairs': element 2i turns with 2i + 1; 'halves':
    element i turns with i + dims/2.  Positions 0..T-1 unless given."""
    if not rot or rot["dims"] == 0:
        return x
    T, dims = x.shape[0], rot["dims"]
    pos = torch.arange(T, dtype=F64) if positions is None else \
        torch.as_tensor(positions, dtype=F64)
    f = frequencies(rot)
    out = x.clone()
    for i in range(dims // 2):
        a, b = (2 * i, 2 * i + 1) if layout == "pairs" else (i, i + dims // 2)
        c, s = (pos * f[i]).cos()[:, None], (pos * f[i]).sin()[:, None]
        out[..., a] = x[..., a] * c - x[..., b] * s
        out[..., b] = x[..., b] * c + x[..., a] * s
    return out


# --------------------------------------------------- differential attention
def attend(q, k, v, scale, window=0):
    """Softmax attention of q [T, H, d] over k [T, G, d], v [T, Gv, dv], query
    i seeing key j iff 0 <= i - j (< window when window > 0)."""
    T, H, _ = q.shape
    G, Gv = k.shape[1], v.shape[1]
    out = torch.zeros(T, H, v.shape[2], dtype=F64)
    for hh in range(H):
        for i in range(T):
            lo = max(0, i - window + 1) if window > 0 else 0
            s = (k[lo:i + 1, hh // (H // G)] @ q[i, hh]) * scale
            out[i, hh] = torch.softmax(s, 0) @ v[lo:i + 1, hh // (H // Gv)]
    return out


def map_weight(P, pre, diff):
    """The one number by which a layer's second map is taken off."""
    a = torch.exp((_f(P[pre + "lq1"]) * _f(P[pre + "lk1"])).sum())
    b = torch.exp((_f(P[pre + "lq2"]) * _f(P[pre + "lk2"])).sum())
    return a - b + diff


def combine_maps(a1, a2, lam, diff, eps):
    """a1, a2 [T, H, dv]: unit-RMS per head of a1 - lam a2, times 1 - diff."""
    return unit_rms(a1 - lam * a2, eps) * (1.0 - diff)


def diff_attention(h, P, pre, m, eps):
    T = h.shape[0]
    H, G, dk, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = lin(h, P, pre + "q").view(T, H, 2, dk)
    k = lin(h, P, pre + "k").view(T, G, 2, dk)
    v = lin(h, P, pre + "v").view(T, G, dv)
    size = (m.get("mask") or {}).get("size", 0)
    maps = [attend(rotate(q[:, :, i], m.get("rot"), "pairs"),
                   rotate(k[:, :, i], m.get("rot"), "pairs"), v, m["scale"],
                   size) for i in range(2)]
    o = combine_maps(maps[0], maps[1], map_weight(P, pre, m["diff"]),
                     m["diff"], eps)
    o = o.reshape(T, H * dv) * torch.sigmoid(lin(h, P, pre + "g"))
    return lin(o, P, pre + "o")


# --------------------------------------------------------- latent attention
def latents(h, P, pre, m, eps):
    """(normed latent [T, kv_rank], rotated key part [T, rot_dim])."""
    d = lin(h, P, pre + "dkv")
    R = m["kv_rank"]
    c = unit_rms(d[:, :R], eps) * _f(P[pre + "dkv.norm"])
    return c, rotate(d[:, None, R:], m.get("rot"), "halves")[:, 0]


def latent_attention(h, P, pre, m, eps, shared=None):
    """Unabsorbed: every head's keys and values are made from the latent.
    shared: another layer's (latent, rotated key part) to use."""
    T = h.shape[0]
    H, du, dr, dv = m["heads"], m["dim"], m["rot_dim"], m["vdim"]
    c, kr = shared if shared is not None else latents(h, P, pre, m, eps)
    q = lin(h, P, pre + "q").view(T, H, du + dr)
    qr = rotate(q[..., du:], m.get("rot"), "halves")
    ku = lin(c, P, pre + "uk").view(T, H, du)
    v = lin(c, P, pre + "uv").view(T, H, dv)
    o = attend(torch.cat([q[..., :du], qr], -1),
               torch.cat([ku, kr[:, None].expand(T, H, dr)], -1), v,
               m["scale"], (m.get("mask") or {}).get("size", 0))
    o = o * torch.sigmoid(lin(h, P, pre + "g"))[:, :, None]
    return lin(o.reshape(T, H * dv), P, pre + "o")


# ------------------------------------------------------------ feed-forward
def xielu(z, act):
    p, q = _f(act)[0], _f(act)[1]
    zn = torch.clamp(z, max=0.0)
    return torch.where(z > 0, softplus(p) * z * z + 0.5 * z,
                       (0.5 + softplus(q)) * (torch.exp(zn) - 1.0 - zn)
                       + 0.5 * z)


def feed_forward(h, P, pre):
    return lin(xielu(lin(h, P, pre + "up"), P[pre + "act"]), P, pre + "down")


# ------------------------------------------------------------------- model
def forward(tokens, P, cfg, layers_out=None):
    """tokens [T] -> logits [T, vocab] (float64).  layers_out: a list that
    receives the residual after every layer."""
    eps, mult = cfg["norm"]["eps"], cfg["residual_mult"]
    x = _f(P["embed"])[torch.as_tensor(tokens, dtype=torch.long)]
    kept = {}
    for i, lc in enumerate(cfg["layers"]):
        pre, m = f"l{i}.", lc["mixer"]
        h = layer_norm(x, P[pre + "norm1"], eps)
        if lc["type"] == "rglru":
            y = rglru_mixer(h, P, pre + "mix.", m, eps)
        elif lc["type"] == "attention":
            y = diff_attention(h, P, pre + "mix.", m, eps)
        else:
            src = m.get("kv_from")
            if src is None:
                kept[i] = latents(h, P, pre + "mix.", m, eps)
            y = latent_attention(h, P, pre + "mix.", m, eps,
                                 kept[i if src is None else src])
        x = x + mult * layer_norm(y, P[pre + "norm1b"], eps)
        if lc.get("mlp") is not None:
            y = feed_forward(layer_norm(x, P[pre + "norm2"], eps), P,
                             pre + "mlp.")
            x = x + mult * layer_norm(y, P[pre + "norm2b"], eps)
        if layers_out is not None:
            layers_out.append(x.clone())
    return lin(layer_norm(x, P["final.norm"], eps), P, "embed")


# ---------------------------------------------------------- random weights
def random_weights(cfg, seed=0):
    """Checkpoint-named random tensors (bf16-representable float32) for any
    config, at scales that keep every branch alive."""
    g = torch.Generator().manual_seed(seed)
    W, V = cfg["width"], cfg["vocab"]
    P = {}

    def rnd(name, *shape, std=None, mean=0.0):
        std = std if std is not None else shape[-1] ** -0.5
        t = torch.randn(*shape, generator=g) * std + mean
        P[name] = t.to(torch.bfloat16).float()

    rnd("embed", V, W, std=1.0)
    rnd("final.norm", W, std=0.1, mean=1.0)
    for i, lc in enumerate(cfg["layers"]):
        pre, m = f"l{i}.", lc["mixer"]
        mp = pre + "mix."
        rnd(pre + "norm1", W, std=0.1, mean=1.0)
        rnd(pre + "norm1b", W, std=0.1, mean=1.0)
        if lc["type"] == "rglru":
            C, nb = m["width"], m["blocks"]
            for n in ("y", "x"):
                rnd(mp + n, C, W)
                rnd(mp + n + ".b", C, std=0.3)
            rnd(mp + "conv", C, m["conv"], std=0.7)
            rnd(mp + "conv.b", C, std=0.3)
            for n in ("ra", "ri"):
                rnd(mp + n, nb, C // nb, C // nb)
                rnd(mp + n + ".b", nb, C // nb, std=1.0)
            rnd(mp + "lam", C, std=1.5, mean=-3.0)
            rnd(mp + "o", W, C)
        elif lc["type"] == "attention":
            H, G, dk, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
            rnd(mp + "q", H * 2 * dk, W)
            rnd(mp + "k", G * 2 * dk, W)
            rnd(mp + "v", G * dv, W)
            for n in ("lq1", "lk1", "lq2", "lk2"):
                rnd(mp + n, dk, std=0.6 * dk ** -0.25)
            rnd(mp + "g", H * dv, W)
            rnd(mp + "o", W, H * dv)
        else:
            H, du, dr, dv, R = (m["heads"], m["dim"], m["rot_dim"],
                                m["vdim"], m["kv_rank"])
            rnd(mp + "q", H * (du + dr), W)
            if m.get("kv_from") is None:
                rnd(mp + "dkv", R + dr, W)
                rnd(mp + "dkv.norm", R, std=0.1, mean=1.0)
            rnd(mp + "uk", H * du, R)
            rnd(mp + "uv", H * dv, R)
            rnd(mp + "g", H, W)
            rnd(mp + "o", W, H * dv)
        if lc.get("mlp") is not None:
            F = lc["mlp"]["ff"]
            rnd(pre + "norm2", W, std=0.1, mean=1.0)
            rnd(pre + "norm2b", W, std=0.1, mean=1.0)
            rnd(pre + "mlp.up", F, W)
            rnd(pre + "mlp.down", W, F)
            rnd(pre + "mlp.act", 2, std=1.0)
    return P
