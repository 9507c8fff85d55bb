"""Plain float64 statement of the Sadupel decoder, one function per mechanism.

Whole sequences only, no cache, no batching, no kernels: every function takes
the full [T, ...] input of one sequence and loops where the definition loops.
It shares no code with the package and is the yardstick of test_sadupel.py.

Tensors are looked up by checkpoint name in a dict `P` (values are cast to
float64 on use); `cfg` is the parsed config.json.
"""
import math

import torch

F64 = torch.float64


def _f(t):
    return t.to(F64)


def lin(h, P, name):
    return h @ _f(P[name]).t()


def rms_norm(x, w, eps):
    return x / torch.sqrt(x.pow(2).mean(-1, keepdim=True) + eps) * _f(w)


# --------------------------------------------------------------- embedding
def pair_row(prev, token, mul_prev, mul_cur, buckets):
    """Row of the pair table; prev None: the token opens its sequence."""
    if prev is None:
        return buckets
    return (prev * mul_prev + token * mul_cur) % buckets


def embed(tokens, P, cfg):
    x = _f(P["embed"])[torch.as_tensor(tokens, dtype=torch.long)]
    b = (cfg.get("embedding") or {}).get("bigram")
    if b is None:
        return x
    for t, tok in enumerate(tokens):
        x[t] += _f(P["bigram"])[pair_row(tokens[t - 1] if t else None, tok,
                                         b["mul_prev"], b["mul_cur"],
                                         b["buckets"])]
    return x


# --------------------------------------------------------------- attention
def short_conv(u, w):
    """y[t, c] = sum_j w[c, j] u[t - (taps-1-j), c]: the last column weighs
    the current token, inputs before the start are zero."""
    T = u.shape[0]
    taps = w.shape[1]
    y = torch.zeros_like(u)
    for t in range(T):
        for j in range(taps):
            s = t - (taps - 1 - j)
            if s >= 0:
                y[t] += _f(w)[:, j] * u[s]
    return y


def frequencies(rot):
    """base^(-2i/dims), all of them divided by the scaling factor."""
    fac = float((rot.get("scaling") or {}).get("factor", 1.0))
    return [float(rot["base"]) ** (-2.0 * i / rot["dims"]) / fac
            for i in range(rot["dims"] // 2)]


def rotate(x, rot, positions=None):
    """Element i of the last axis of x [T, H, d] turns with i + dims/2."""
    if not rot or rot["dims"] == 0:
        return x
    half = rot["dims"] // 2
    pos = torch.arange(x.shape[0], dtype=F64) if positions is None else \
        torch.as_tensor(positions, dtype=F64)
    out = x.clone()
    for i, f in enumerate(frequencies(rot)):
        c, s = (pos * f).cos()[:, None], (pos * f).sin()[:, None]
        out[..., i] = x[..., i] * c - x[..., i + half] * s
        out[..., i + half] = x[..., i + half] * c + x[..., i] * s
    return out


def attend(q, k, v, scale, cap=0.0, sink=None):
    """Causal softmax attention of q [T, H, d] over k [T, G, d], v [T, G, dv];
    scores bounded by cap, the sink only in the denominator."""
    T, H, _ = q.shape
    rep = H // k.shape[1]
    out = torch.zeros(T, H, v.shape[2], dtype=F64)
    for hh in range(H):
        for i in range(T):
            s = (k[:i + 1, hh // rep] @ q[i, hh]) * scale
            if cap:
                s = cap * torch.tanh(s / cap)
            # shifted by a common maximum, which changes nothing
            m = s.max() if sink is None else torch.maximum(s.max(),
                                                           _f(sink)[hh])
            e = torch.exp(s - m)
            den = e.sum()
            if sink is not None:
                den = den + torch.exp(_f(sink)[hh] - m)
            out[i, hh] = (e / den) @ v[:i + 1, hh // rep]
    return out


def attention(h, P, pre, m, eps):
    T = h.shape[0]
    H, G, dk, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q, k, v = (short_conv(lin(h, P, pre + n), P[pre + n + ".conv"])
               for n in "qkv")
    q = rms_norm(q, P[pre + "q.norm"], eps).view(T, H, dk)
    k = rms_norm(k, P[pre + "k.norm"], eps).view(T, G, dk)
    q, k = (rotate(t, m.get("rot")) for t in (q, k))
    o = attend(q, k, v.view(T, G, dv), m["scale"], m.get("softcap") or 0.0,
               P[pre + "sink"])
    o = o * torch.sigmoid(lin(h, P, pre + "g"))[:, :, None]
    return lin(o.reshape(T, H * dv), P, pre + "o")


# ------------------------------------------------------------ feed-forward
def unit(h, P, pre):
    return torch.relu(lin(h, P, pre + "up")).pow(2) @ _f(P[pre + "down"]).t()


def choose(z, correction, router):
    """One token's logits -> ([chosen indices], [weights])."""
    s = torch.exp(z - z.max())
    s = s / s.sum()
    c = s + _f(correction)
    n = z.numel()
    g = router.get("groups")
    allowed = set(range(n))
    if g:
        size = n // g["count"]
        best = sorted(range(g["count"]),
                      key=lambda a: -float(c[a * size:(a + 1) * size].max()))
        allowed = {e for a in best[:g["keep"]]
                   for e in range(a * size, (a + 1) * size)}
    order = sorted(allowed, key=lambda e: -float(c[e]))[:router["top"]]
    return order, [float(s[e]) for e in order]


def mixture(h, P, pre, mlp):
    r = mlp["router"]
    z = lin(h, P, pre + "router")
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e, w in zip(*choose(z[t], P[pre + "correction"], r)):
            y = h[t] if e >= r["experts"] else \
                unit(h[t:t + 1], P, f"{pre}e{e}.")[0]
            out[t] += w * y
    if mlp.get("shared"):
        out = out + unit(h, P, pre + "shared.")
    return out


# ------------------------------------------------------------------- model
def runs(cfg):
    """[(layer, pass or None outside of the loop)] in execution order."""
    n = len(cfg["layers"])
    lp = cfg.get("loop")
    if not lp:
        return [(i, None) for i in range(n)]
    a, b = lp["start"], lp["stop"]
    return [(i, None) for i in range(a)] + \
        [(i, t) for t in range(lp["times"]) for i in range(a, b)] + \
        [(i, None) for i in range(b, n)]


def forward(tokens, P, cfg, layers_out=None):
    """tokens [T] -> logits [T, vocab] (float64).  layers_out: a list that
    receives the residual after every layer run."""
    eps, mult = cfg["norm"]["eps"], cfg["residual_mult"]
    x = embed(list(tokens), P, cfg)
    for i, t in runs(cfg):
        lc, pre = cfg["layers"][i], f"l{i}."
        if t is not None and i == cfg["loop"]["start"]:
            x = x + _f(P["loop.step"])[t]
        h = rms_norm(x, P[pre + "norm1"], eps)
        y = attention(h, P, pre + "mix.", lc["mixer"], eps)
        if lc.get("mlp") is not None:
            y = y + mixture(h, P, pre + "mlp.", lc["mlp"])
        x = x + mult * y
        if layers_out is not None:
            layers_out.append(x.clone())
    return lin(rms_norm(x, P["final.norm"], eps), P, "head")


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
    b = (cfg.get("embedding") or {}).get("bigram")
    if b:
        rnd("bigram", b["buckets"] + 1, W, std=0.7)
    if cfg.get("loop"):
        rnd("loop.step", cfg["loop"]["times"], W, std=0.5)
    rnd("final.norm", W, std=0.1, mean=1.0)
    rnd("head", V, W)
    for i, lc in enumerate(cfg["layers"]):
        pre, m = f"l{i}.", lc["mixer"]
        mp = pre + "mix."
        H, G, dk, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
        rnd(pre + "norm1", W, std=0.1, mean=1.0)
        for n, rows in (("q", H * dk), ("k", G * dk), ("v", G * dv)):
            rnd(mp + n, rows, W)
            rnd(mp + n + ".conv", rows, m["conv"], std=0.6)
        rnd(mp + "q.norm", H * dk, std=0.2, mean=1.0)
        rnd(mp + "k.norm", G * dk, std=0.2, mean=1.0)
        rnd(mp + "sink", H, std=1.0)
        rnd(mp + "g", H, W)
        rnd(mp + "o", W, H * dv)
        f = lc.get("mlp")
        if f is None:
            continue
        r = f["router"]
        n_out = r["experts"] + r.get("identity", 0)
        fp = pre + "mlp."
        units = [(f"e{e}.", f["expert"]["ff"]) for e in range(r["experts"])]
        if f.get("shared"):
            units.append(("shared.", f["shared"]["ff"]))
        for u, ff in units:
            rnd(fp + u + "up", ff, W)
            rnd(fp + u + "down", W, ff)
        rnd(fp + "router", n_out, W)
        rnd(fp + "correction", n_out, std=0.1)
    return P
