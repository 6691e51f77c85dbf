"""A plain, slow implementation of Zudalorn in float64, one function per mechanism, written from
the design's equations.  It shares no code with the package: the tests compare the engine
against it.

Notation.  x: the residual stream [T, W].  rms(t) = t / sqrt(mean(t^2) + eps) over the last axis.
A layer is x <- x + g1b rms(mixer(g1 rms(x))); x <- x + g2b rms(ff(g2 rms(x))), every g one number
(the second line only with a feed-forward).  Mixers: attention out of a latent per position (no
latent of the queries, a rotated part of the keys that all heads share, a sliding window), and
retention, a linear attention with a fixed decay per head.  Feed-forward: one layer with the xIELU
activation, or a routed mixture of small gated ones with a shared one behind a gate.
"""
import math

import torch

F64 = torch.float64


def rms(t, eps):
    return t / torch.sqrt((t * t).mean(dim=-1, keepdim=True) + eps)


def scalar_norm(t, eps, g):
    return rms(t, eps) * g


# ---- positions --------------------------------------------------------------------------------------

def frequencies(rot):
    """Angles per position of the dims/2 pairs, and the factor on cosines and sines.  Without
    `scaling`: base^(-2i/dims) and 1.  With it, pairs that turn seldom within `original` positions
    are slowed down by `factor`, those that turn often are kept, a ramp between."""
    base, dims = float(rot["base"]), rot["dims"]
    f = [base ** (-2.0 * i / dims) for i in range(dims // 2)]
    sc = rot.get("scaling")
    if not sc:
        return torch.tensor(f, dtype=F64), 1.0

    def where(turns):
        return dims * math.log(sc["original"] / (2 * math.pi * turns)) / (2 * math.log(base))

    lo = max(math.floor(where(sc["fast"])), 0)
    hi = min(math.ceil(where(sc["slow"])), dims - 1)
    out = []
    for i, fi in enumerate(f):
        r = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        out.append(fi / sc["factor"] * r + fi * (1.0 - r))
    return torch.tensor(out, dtype=F64), 0.1 * math.log(sc["factor"]) + 1.0


def rotate(t, pos, rot, interleaved):
    """t [T, heads, d]: the first `dims` channels of every head turned by pos * f_i; pair i is
    (2i, 2i + 1) or (i, i + dims/2)."""
    if not rot or not rot["dims"]:
        return t
    dims = rot["dims"]
    f, mag = frequencies(rot)
    a = pos.to(F64)[:, None, None] * f
    c, s = (torch.cos(a) * mag).to(t.dtype), (torch.sin(a) * mag).to(t.dtype)
    out = t.clone()
    iu = torch.arange(dims // 2) * 2 if interleaved else torch.arange(dims // 2)
    iv = iu + 1 if interleaved else iu + dims // 2
    u, v = t[..., iu], t[..., iv]
    out[..., iu] = u * c - v * s
    out[..., iv] = v * c + u * s
    return out


def window_mask(pos, size):
    """[T, T] bool: row i sees column j iff 0 <= i - j < size (`size` None: 0 <= i - j)."""
    d = pos[:, None] - pos[None, :]
    ok = d >= 0
    return ok & (d < size) if size else ok


# ---- mixers -----------------------------------------------------------------------------------------

def latent_rows(h, w, p, m, pos, eps):
    """What a position leaves behind: the normed latent c [T, R] and the rotated key part [T, dr]."""
    R, dr = m["kv_rank"], m["rot_dim"]
    t = h @ w[p + "dkv"].T
    c = rms(t[:, :R], eps) * w[p + "dkv.norm"]
    return c, rotate(t[:, None, R:], pos, dict(m["rot"], dims=dr), True)[:, 0]


def latent_attention(h, w, p, m, pos, eps):
    T, H, dn, dr, dv = h.shape[0], m["heads"], m["dim"], m["rot_dim"], m["vdim"]
    q = (h @ w[p + "q"].T).view(T, H, dn + dr)
    qn, qr = q[..., :dn], rotate(q[..., dn:], pos, dict(m["rot"], dims=dr), True)
    c, kr = latent_rows(h, w, p, m, pos, eps)
    kn = (c @ w[p + "uk"].T).view(T, H, dn)
    v = (c @ w[p + "uv"].T).view(T, H, dv)
    s = (qn.transpose(0, 1) @ kn.permute(1, 2, 0) + qr.transpose(0, 1) @ kr.T[None]) * m["scale"]
    s = s.masked_fill(~window_mask(pos, (m.get("mask") or {}).get("size"))[None], -math.inf)
    o = torch.softmax(s, dim=-1) @ v.transpose(0, 1)
    return o.transpose(0, 1).reshape(T, H * dv) @ w[p + "o"].T


def retention_heads(q, k, v, decay, S=None):
    """q, k [T, H, d] (rotated, k scaled), v [T, H, dv]: S <- decay S + k v^T, o = S^T q, row by row."""
    T, H, d = q.shape
    S = torch.zeros(H, d, v.shape[-1], dtype=q.dtype) if S is None else S
    g = torch.as_tensor(decay, dtype=q.dtype)[:, None, None]
    out = []
    for t in range(T):
        S = g * S + k[t][:, :, None] * v[t][:, None, :]
        out.append((S * q[t][:, :, None]).sum(dim=1))
    return torch.stack(out), S


def retention(h, w, p, m, pos, eps):
    T, H, d, dv = h.shape[0], m["heads"], m["dim"], m["vdim"]
    q = rotate((h @ w[p + "q"].T).view(T, H, d), pos, m.get("rot"), False)
    k = rotate((h @ w[p + "k"].T).view(T, H, d), pos, m.get("rot"), False) * d ** -0.5
    v = (h @ w[p + "v"].T).view(T, H, dv)
    o, _ = retention_heads(q, k, v, m["decay"])
    g = h @ w[p + "g"].T
    return (rms(o, eps).reshape(T, H * dv) * (g * torch.sigmoid(g))) @ w[p + "o"].T


MIXERS = {"latent_attention": latent_attention, "retention": retention}


# ---- feed-forwards ----------------------------------------------------------------------------------

def softplus(t):
    return torch.log1p(torch.exp(-t.abs())) + torch.clamp(t, min=0)


def xielu(z, pq):
    a, b = softplus(pq[0]), 0.5 + softplus(pq[1])
    return torch.where(z > 0, a * z * z + 0.5 * z, b * (torch.expm1(torch.clamp(z, max=0)) - z) + 0.5 * z)


def dense_ff(h, w, p):
    return xielu(h @ w[p + "up"].T, w[p + "act"]) @ w[p + "down"].T


def gated_expert(h, w, p):
    g = h @ w[p + "gate"].T
    return (g * torch.sigmoid(g) * (h @ w[p + "up"].T)) @ w[p + "down"].T


def route(h, w, p, r, margins=None):
    """[T, E] weights: s / (sum of the chosen s + 1e-20) where chosen, 0 elsewhere, s = logistic(W_r h).
    The choice goes by s + correction: the `keep` groups whose two largest add up to most, in them
    the `top` largest (of equal ones the smaller index).  `margins`: a list that receives, per row,
    the smallest gap of choice scores by which an expert or a group was preferred."""
    s = torch.sigmoid(h @ w[p + "router"].T)
    choice = s + w[p + "correction"]
    T, E = s.shape
    gap = torch.full((T,), math.inf, dtype=s.dtype)
    groups = r.get("groups")
    if groups:
        n, keep = groups["count"], groups["keep"]
        by = choice.view(T, n, E // n)
        score = by.topk(min(2, E // n), dim=-1).values.sum(dim=-1)
        order = torch.sort(score, dim=-1, descending=True, stable=True)
        ok = torch.zeros(T, n, dtype=torch.bool).scatter_(1, order.indices[:, :keep], True)
        if keep < n:
            gap = torch.minimum(gap, order.values[:, keep - 1] - order.values[:, keep])
        choice = choice.masked_fill(~ok.repeat_interleave(E // n, dim=1), -math.inf)
    order = torch.sort(choice, dim=-1, descending=True, stable=True)
    top = r["top"]
    if top < E:
        gap = torch.minimum(gap, order.values[:, top - 1] - order.values[:, top])
    chosen = torch.zeros(T, E, dtype=torch.bool).scatter_(1, order.indices[:, :top], True)
    if margins is not None:
        margins.append(gap)
    s = torch.where(chosen, s, torch.zeros_like(s))
    return s / (s.sum(dim=-1, keepdim=True) + 1e-20)


def routed_ff(h, w, p, mlp, margins=None):
    wt = route(h, w, p, mlp["router"], margins)
    y = torch.zeros(h.shape[0], w[p + "e0.down"].shape[0], dtype=h.dtype)
    for e in range(mlp["router"]["experts"]):
        rows = (wt[:, e] != 0).nonzero().flatten()
        if len(rows):
            y[rows] += wt[rows, e:e + 1] * gated_expert(h[rows], w, f"{p}e{e}.")
    if mlp.get("shared"):
        y = y + torch.sigmoid(h @ w[p + "shared.sg"].T) * gated_expert(h, w, p + "shared.")
    return y


# ---- the model --------------------------------------------------------------------------------------

def forward(w, cfg, ids, dtype=F64, streams=None, margins=None):
    """Logits [T, vocab] of one sequence.  `streams`: a list that receives the stream after every
    layer; `margins`: see `route`."""
    w = {k: (v.to(dtype) if v.is_floating_point() else v) for k, v in w.items()}
    eps = cfg["norm"]["eps"]
    ids = torch.as_tensor(ids, dtype=torch.long)
    pos = torch.arange(len(ids))
    x = w["embed"][ids]
    for i, layer in enumerate(cfg["layers"]):
        p = f"l{i}."
        h = scalar_norm(x, eps, w[p + "norm1"])
        y = MIXERS[layer["type"]](h, w, p + "mix.", layer["mixer"], pos, eps)
        x = x + scalar_norm(y, eps, w[p + "norm1b"])
        f = layer.get("mlp")
        if f:
            h = scalar_norm(x, eps, w[p + "norm2"])
            y = dense_ff(h, w, p + "mlp.") if f["kind"] == "dense" else routed_ff(h, w, p + "mlp.", f, margins)
            x = x + scalar_norm(y, eps, w[p + "norm2b"])
        if streams is not None:
            streams.append(x)
    return scalar_norm(x, eps, w["final.norm"]) @ w["head"].T


def generate_greedy(w, cfg, ids, n, dtype=F64):
    ids = list(ids)
    out = []
    for _ in range(n):
        t = int(torch.argmax(forward(w, cfg, ids, dtype)[-1]))
        out.append(t)
        ids.append(t)
    return out


def tensor_shapes(cfg):
    W, V = cfg["width"], cfg["vocab"]
    s = {"embed": (V, W), "head": (V, W), "final.norm": ()}
    for i, layer in enumerate(cfg["layers"]):
        p, m, f = f"l{i}.", layer["mixer"], layer.get("mlp")
        for n in ("norm1", "norm1b") + (("norm2", "norm2b") if f else ()):
            s[p + n] = ()
        H, d, dv = m["heads"], m["dim"], m["vdim"]
        if layer["type"] == "latent_attention":
            R, dr = m["kv_rank"], m["rot_dim"]
            s.update({p + "mix.q": (H * (d + dr), W), p + "mix.dkv": (R + dr, W), p + "mix.dkv.norm": (R,),
                      p + "mix.uk": (H * d, R), p + "mix.uv": (H * dv, R), p + "mix.o": (W, H * dv)})
        else:
            s.update({p + "mix.q": (H * d, W), p + "mix.k": (H * d, W), p + "mix.v": (H * dv, W),
                      p + "mix.g": (H * dv, W), p + "mix.o": (W, H * dv)})
        if f and f["kind"] == "dense":
            s.update({p + "mlp.up": (f["ff"], W), p + "mlp.down": (W, f["ff"]), p + "mlp.act": (2,)})
        elif f:
            E = f["router"]["experts"]
            parts = [(f"e{e}", f["expert"]["ff"]) for e in range(E)]
            if f.get("shared"):
                parts.append(("shared", f["shared"]["ff"]))
                s[p + "mlp.shared.sg"] = (1, W)
            for n, ff in parts:
                s.update({f"{p}mlp.{n}.gate": (ff, W), f"{p}mlp.{n}.up": (ff, W), f"{p}mlp.{n}.down": (W, ff)})
            s[p + "mlp.router"] = (E, W)
            s[p + "mlp.correction"] = (E,)
    return s


def random_weights(cfg, seed, gain=1.0, dtype=torch.bfloat16):
    """Weights of the tests' own making: products N(0, gain / sqrt(fan in)), norms near 1, corrections
    large enough to turn choices and of both signs, activation numbers of both signs."""
    g = torch.Generator().manual_seed(seed)
    out = {}
    for name, shape in tensor_shapes(cfg).items():
        leaf = name.split(".")[-1]
        if "norm" in leaf:
            t = 1.0 + 0.3 * torch.randn(shape, generator=g)
        elif leaf == "correction":
            t = 0.4 * torch.randn(shape, generator=g) - 0.3
        elif leaf == "act":
            t = torch.randn(shape, generator=g)
        elif name == "embed":
            t = torch.randn(shape, generator=g)
        elif leaf in ("router", "sg"):
            t = 2.0 * torch.randn(shape, generator=g) / math.sqrt(shape[1])
        else:
            t = gain * torch.randn(shape, generator=g) / math.sqrt(shape[-1])
        out[name] = t.to(dtype)
    return out
