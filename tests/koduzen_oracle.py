"""A plain, slow Koduzen: every mechanism written from its equations as one function over a whole
sequence in float64. It shares no code with llmd_amd; the tests compare the framework with it.

``cfg`` is the configuration as a dict (the layout of a config.json), ``W`` maps tensor names
to tensors.
"""
from __future__ import annotations

import math

import torch

F64 = torch.float64


def rms_norm(x, eps, w=None):
    """x / sqrt(mean(x^2) + eps) over the last axis, times w."""
    y = x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)
    return y if w is None else y * w.to(F64)


def linear(x, W, name):
    return x @ W[name].to(F64).T


def silu(z):
    return z / (1.0 + torch.exp(-z))


def frequencies(dims, base, scaling=None):
    """base^(-2i/dims); the ramp form divides the slow ones by ``factor``. Returns (frequencies, magnitude of cos and sin)."""
    f = [base ** (-2.0 * i / dims) for i in range(dims // 2)]
    if not scaling:
        return f, 1.0
    factor, original = scaling["factor"], scaling["original"]

    def index_of(turns):  # the pair that turns so many times over the original length
        return dims * math.log(original / (2.0 * math.pi * turns)) / (2.0 * math.log(base))

    lo = max(math.floor(index_of(scaling["fast"])), 0)
    hi = min(math.ceil(index_of(scaling["slow"])), dims - 1)
    out = []
    for i, fi in enumerate(f):
        r = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        out.append(fi / factor * r + fi * (1.0 - r))
    return out, 0.1 * math.log(factor) + 1.0


def rotate(x, dims, base, scaling=None):
    """x [T, heads, n] at positions 0 .. T - 1: the pair (i, i + dims/2) turns by p f_i."""
    half = dims // 2
    f, mag = frequencies(dims, base, scaling)
    y = x.clone()
    for p in range(x.shape[0]):
        for i in range(half):
            c, s = mag * math.cos(p * f[i]), mag * math.sin(p * f[i])
            u, v = x[p, :, i], x[p, :, i + half]
            y[p, :, i] = u * c - v * s
            y[p, :, i + half] = v * c + u * s
    return y


def visible(i, j, size=None):
    """Does position i see position j: itself and the size - 1 before it."""
    return 0 <= i - j and (size is None or i - j < size)


def temperature(p, q_temp):
    """What a query at position p is multiplied with."""
    return 1.0 + q_temp["coef"] * math.log(math.floor((p + 1) / q_temp["every"]) + 1.0)


def slope(h, heads):
    return 2.0 ** (-8.0 * (h + 1) / heads)


def softmax_rows(q, k, v, scale, size=None, sink=None, slope=0.0):
    """One head: q [T, d], k [T, d], v [T, dv]. ``slope`` times the distance comes off a score; ``sink``: a number
    whose exponential joins the denominator."""
    T = q.shape[0]
    out = torch.zeros(T, v.shape[-1], dtype=F64)
    for i in range(T):
        lo = 0 if size is None else max(0, i - size + 1)
        js = torch.arange(lo, i + 1)
        s = (k[lo:i + 1] @ q[i]) * scale - slope * (i - js).to(F64)
        top = s.max() if sink is None else torch.maximum(s.max(), sink.to(F64))
        e = torch.exp(s - top)
        den = e.sum() if sink is None else e.sum() + torch.exp(sink.to(F64) - top)
        out[i] = (e / den) @ v[lo:i + 1]
    return out


def attention(h, W, pre, m, eps, kv=None):
    """Grouped attention: norms over whole projections, partial rotation, a window; ``kv`` the (rotated) keys and the
    values of another layer. Returns (result, (k, v))."""
    T = h.shape[0]
    H, G, d, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = rms_norm(linear(h, W, pre + "q"), eps, W[pre + "q.norm"]).view(T, H, d)
    rot = m["rot"]
    q = rotate(q, rot["dims"], rot["base"], rot.get("scaling"))
    if kv is None:
        k = rms_norm(linear(h, W, pre + "k"), eps, W[pre + "k.norm"]).view(T, G, d)
        kv = rotate(k, rot["dims"], rot["base"], rot.get("scaling")), linear(h, W, pre + "v").view(T, G, dv)
    k, v = kv
    size = m["mask"]["size"]
    o = [softmax_rows(q[:, n], k[:, n // (H // G)], v[:, n // (H // G)], m["scale"], size) for n in range(H)]
    return linear(torch.cat(o, -1), W, pre + "o"), kv


def attention_2(h, W, pre, m, kv=None):
    """Grouped attention without rotation: query temperature, distance bias, a window, sinks; ``kv`` the keys and
    values of another layer. Returns (result, (k, v))."""
    T = h.shape[0]
    H, G, d, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = linear(h, W, pre + "q").view(T, H, d)
    if m.get("q_temp"):
        q = q * torch.tensor([temperature(p, m["q_temp"]) for p in range(T)], dtype=F64)[:, None, None]
    if kv is None:
        kv = linear(h, W, pre + "k").view(T, G, d), linear(h, W, pre + "v").view(T, G, dv)
    k, v = kv
    size = m["mask"]["size"]
    o = [softmax_rows(q[:, n], k[:, n // (H // G)], v[:, n // (H // G)], m["scale"], size, W[pre + "sink"][n], slope(n, H))
         for n in range(H)]
    return linear(torch.cat(o, -1), W, pre + "o"), kv


def retention_rows(q, k, v, decay):
    """One head: S <- decay S + k v^T; o = S^T q."""
    S = torch.zeros(k.shape[1], v.shape[1], dtype=F64)
    out = torch.zeros(v.shape, dtype=F64)
    for t in range(q.shape[0]):
        S = decay * S + torch.outer(k[t], v[t])
        out[t] = S.T @ q[t]
    return out


def retention(h, W, pre, m, eps):
    T = h.shape[0]
    H, d, dv = m["heads"], m["dim"], m["vdim"]
    rot = m["rot"]
    q, k = (rotate(linear(h, W, pre + n).view(T, H, d), rot["dims"], rot["base"]) for n in "qk")
    k = k / math.sqrt(d)
    v = linear(h, W, pre + "v").view(T, H, dv)
    o = [rms_norm(retention_rows(q[:, n], k[:, n], v[:, n], m["decay"][n]), eps) for n in range(H)]
    return linear(torch.cat(o, -1) * silu(linear(h, W, pre + "g")), W, pre + "o")


def gated_ff(h, W, pre, limit):
    """W_down (g sigmoid(1.702 g) (u + 1)), g cut off above ``limit``, u on both sides."""
    g = torch.clamp(linear(h, W, pre + "gate"), max=limit)
    u = torch.clamp(linear(h, W, pre + "up"), min=-limit, max=limit)
    return linear(g / (1.0 + torch.exp(-1.702 * g)) * (u + 1.0), W, pre + "down")


def route(z, correction, router):
    """One token's router outputs -> [(index, weight)]: only members of the best groups can be chosen, by score +
    correction; the weights are the scores alone."""
    n = z.shape[0]
    s = torch.softmax(z, 0)
    c = [float(s[i] + correction[i]) for i in range(n)]
    groups, keep = router["groups"]["count"], router["groups"]["keep"]
    per = n // groups
    best = [max(c[g * per:(g + 1) * per]) for g in range(groups)]
    kept = sorted(range(groups), key=lambda g: (-best[g], g))[:keep]
    chosen = sorted((i for i in range(n) if i // per in kept), key=lambda i: (-c[i], i))[:router["top"]]
    total = sum(float(s[i]) for i in chosen) + 1e-20
    return [(i, float(s[i]) / total * router["scale"]) for i in chosen]


def experts(h, W, pre, m):
    """Gated experts, identity experts (the last router outputs) and one shared expert for every token."""
    r, limit = m["router"], m["expert"]["limit"]
    z = linear(h, W, pre + "router")
    y = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for n, w in route(z[t], W[pre + "correction"].to(F64), r):
            y[t] += w * (h[t] if n >= r["experts"] else gated_ff(h[t:t + 1], W, f"{pre}e{n}.", limit)[0])
    if m.get("shared"):
        y = y + gated_ff(h, W, pre + "shared.", m["shared"]["limit"])
    return y


def hyper(X, W, pre, sublayer):
    """The streams X after one sublayer: it reads a sum of them, they are remixed and each gets a share of its result."""
    w_in, w_out, mix = W[pre + "in"].to(F64), W[pre + "out"].to(F64), W[pre + "mix"].to(F64)
    n = len(X)
    y = sublayer(sum(w_in[s] * X[s] for s in range(n)))
    return [sum(mix[s, t] * X[s] for s in range(n)) + w_out[t] * y for t in range(n)]


def forward(cfg, W, tokens, layers_out=None):
    """Logits [T, vocab] of one sequence; ``layers_out`` receives the sum of the streams after every layer."""
    eps = cfg["norm"]["eps"]
    x = W["embed"].to(F64)[torch.as_tensor(tokens)]
    X = [x.clone() for _ in range(cfg["streams"])]
    kvs = {}
    for i, spec in enumerate(cfg["layers"]):
        pre, m, f = f"l{i}.", spec["mixer"], spec.get("mlp")

        def mixer(u):
            h = rms_norm(u, eps, W[pre + "norm1"])
            if spec["type"] == "retention":
                return retention(h, W, pre + "mix.", m, eps)
            kv = kvs[m["kv_from"]] if "kv_from" in m else None
            if spec["type"] == "attention":
                y, kvs[i] = attention(h, W, pre + "mix.", m, eps, kv)
            elif spec["type"] == "attention_2":
                y, kvs[i] = attention_2(h, W, pre + "mix.", m, kv)
            else:
                raise ValueError(spec["type"])
            return y

        def ff(u):
            h = rms_norm(u, eps, W[pre + "norm2"])
            return gated_ff(h, W, pre + "mlp.", f["limit"]) if f["kind"] == "dense" else experts(h, W, pre + "mlp.", f)

        X = hyper(X, W, pre + "hc1.", mixer)
        if f:
            X = hyper(X, W, pre + "hc2.", ff)
        if layers_out is not None:
            layers_out.append(sum(X))
    return linear(rms_norm(sum(X), eps, W["final.norm"]), W, "embed")


def random_weights(cfg, seed=0, dtype=torch.float32):
    """Random tensors with the design's names and shapes (std chosen so that nothing saturates)."""
    g = torch.Generator().manual_seed(seed)
    d, V, S = cfg["width"], cfg["vocab"], cfg["streams"]
    W = {}

    def mat(name, *shape, std=None):
        std = std if std is not None else 1.0 / math.sqrt(shape[-1])
        W[name] = (torch.randn(*shape, generator=g) * std).to(dtype)

    def vec(name, n, mean=1.0, std=0.1):
        W[name] = (mean + torch.randn(n, generator=g) * std).to(dtype)

    def ffn(pre, n):
        mat(pre + "gate", n, d, std=1.5 / math.sqrt(d))     # wide enough for both limits to act
        mat(pre + "up", n, d, std=1.5 / math.sqrt(d))
        mat(pre + "down", d, n)

    mat("embed", V, d, std=1.0)
    for i, spec in enumerate(cfg["layers"]):
        pre, m, f = f"l{i}.", spec["mixer"], spec.get("mlp")
        for q in ("1", "2") if f else ("1",):
            vec(pre + "norm" + q, d)
            vec(f"{pre}hc{q}.in", S, mean=1.0 / S, std=0.3)
            vec(f"{pre}hc{q}.out", S, mean=0.6, std=0.4)
            W[f"{pre}hc{q}.mix"] = (0.7 * torch.eye(S) + 0.3 / S + 0.1 * torch.randn(S, S, generator=g)).to(dtype)
        mp = pre + "mix."
        H, dim, dv = m["heads"], m["dim"], m["vdim"]
        mat(mp + "q", H * dim, d)
        if spec["type"] == "retention":
            mat(mp + "k", H * dim, d)
            mat(mp + "v", H * dv, d)
            mat(mp + "g", H * dv, d)
        else:
            if "kv_from" not in m:
                mat(mp + "k", m["kv_heads"] * dim, d)
                mat(mp + "v", m["kv_heads"] * dv, d)
            if spec["type"] == "attention":
                vec(mp + "q.norm", H * dim)
                if "kv_from" not in m:
                    vec(mp + "k.norm", m["kv_heads"] * dim)
            else:
                vec(mp + "sink", H, mean=0.0, std=1.0)
        mat(mp + "o", d, H * dv)
        if not f:
            continue
        fp = pre + "mlp."
        if f["kind"] == "dense":
            ffn(fp, f["ff"])
        else:
            r = f["router"]
            n = r["experts"] + r.get("identity", 0)
            mat(fp + "router", n, d)
            vec(fp + "correction", n, mean=-0.1, std=0.1)   # choice scores below zero occur
            for e in range(r["experts"]):
                ffn(f"{fp}e{e}.", f["expert"]["ff"])
            if f.get("shared"):
                ffn(fp + "shared.", f["shared"]["ff"])
    vec("final.norm", d)
    return W
