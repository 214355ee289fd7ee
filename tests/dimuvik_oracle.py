"""Plain float64 implementation of the Dimuvik design, one function per
mechanism, written token by token from the equations. It shares no code with
the product path; the tests compare the engine with it.

A model is (cfg, w): cfg is the checkpoint's config.json as a dict, w maps
checkpoint tensor names to float64 tensors.

    x = embed[token] * s
    each layer:  x <- x + dyt_1b(mixer(dyt_1(x)))
                 x <- x + dyt_2b(ff(dyt_2(x)))               (no ff: skipped)
    logits = head . dyt_final(x)
    dyt(v) = tanh(alpha v) w + b, alpha one number per norm
"""

import math

import torch

F64 = torch.float64


# --- small pieces -----------------------------------------------------------------

def dyt(w, name, v):
    return torch.tanh(w[name + ".alpha"] * v) * w[name] + w[name + ".b"]


def rms(v, eps):
    return v / torch.sqrt((v * v).mean(-1, keepdim=True) + eps)


def silu(z):
    return z * torch.sigmoid(z)


def rotate_pairs(vec, p, base, dims):
    """Entries 2i and 2i+1 of vec [..., D] turned by p base^(-2i/dims)."""
    out = vec.clone()
    for i in range(dims // 2):
        a = p * base ** (-2.0 * i / dims)
        u, v = vec[..., 2 * i], vec[..., 2 * i + 1]
        out[..., 2 * i] = u * math.cos(a) - v * math.sin(a)
        out[..., 2 * i + 1] = v * math.cos(a) + u * math.sin(a)
    return out


def short_conv(u, taps):
    """y_t[c] = sum_j taps[c, j] u_{t - K + 1 + j}[c], zeros before the sequence."""
    K = taps.shape[1]
    out = []
    for t in range(u.shape[0]):
        y = torch.zeros(u.shape[1], dtype=F64)
        for j in range(K):
            if t - K + 1 + j >= 0:
                y = y + taps[:, j] * u[t - K + 1 + j]
        out.append(y)
    return torch.stack(out)


def query_temperature(p, coef, every):
    return 1.0 + coef * math.log((p + 1) // every + 1)


# --- mixers: h [T, W], a whole sequence from position 0 -----------------------------

def project(w, pre, name, h):
    u = torch.stack([w[pre + name] @ x + w[pre + name + ".b"] for x in h])
    return short_conv(u, w[pre + name + ".conv"])


def diff_lambda(w, pre, diff):
    return float(torch.exp((w[pre + "lq1"] * w[pre + "lk1"]).sum()) - torch.exp((w[pre + "lq2"] * w[pre + "lk2"]).sum()) + diff)


def attention(w, pre, m, h, eps, kv=None, kv_out=None):
    """``kv``: the (keys, values) of the layer whose cache this one reads;
    ``kv_out`` (a list) receives this layer's own."""
    H, G, D, V = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    T = h.shape[0]
    q = project(w, pre, "q", h).view(T, H, 2, D)
    if kv is None:
        kv = project(w, pre, "k", h).view(T, G, 2, D), project(w, pre, "v", h).view(T, G, V)
        if kv_out is not None:
            kv_out.append(kv)
    k, v = kv
    lam = diff_lambda(w, pre, m["diff"])
    out = []
    for i in range(T):
        qi = q[i] * query_temperature(i, m["q_temp"]["coef"], m["q_temp"]["every"])
        heads = []
        for hd in range(H):
            g = hd // (H // G)
            a = [torch.softmax(k[:i + 1, g, mp] @ qi[hd, mp] * m["scale"], 0) @ v[:i + 1, g] for mp in range(2)]
            heads.append(rms(a[0] - lam * a[1], eps) * (1.0 - m["diff"]))
        out.append(w[pre + "o"] @ torch.cat(heads))
    return torch.stack(out)


def softmax_with_sink(scores, sink):
    """Weights of the scores when the denominator holds exp(sink) besides."""
    top = torch.maximum(scores.max(), sink)
    e = torch.exp(scores - top)
    return e / (e.sum() + torch.exp(sink - top))


def latent_query(w, pre, x, eps):
    return w[pre + "uq"] @ (rms(w[pre + "dq"] @ x, eps) * w[pre + "dq.norm"])


def latent_attention(w, pre, m, h, eps):
    H, D, R, V, C = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    base, dims = m["rot"]["base"], m["rot"]["dims"]
    qs, keys, vals = [], [], []
    for p, x in enumerate(h):
        q = latent_query(w, pre, x, eps).view(H, D + R)
        qs.append(torch.cat([q[:, :D], rotate_pairs(q[:, D:], p, base, dims)], -1))
        d = w[pre + "dkv"] @ x
        c = rms(d[:C], eps) * w[pre + "dkv.norm"]
        kr = rotate_pairs(d[C:], p, base, dims)
        keys.append(torch.cat([(w[pre + "uk"] @ c).view(H, D), kr.expand(H, R)], -1))
        vals.append((w[pre + "uv"] @ c).view(H, V))
    keys, vals = torch.stack(keys), torch.stack(vals)
    out = []
    for i in range(h.shape[0]):
        heads = []
        for hd in range(H):
            pr = softmax_with_sink((keys[:i + 1, hd] @ qs[i][hd]) * m["scale"], w[pre + "sink"][hd])
            heads.append(pr @ vals[:i + 1, hd])
        out.append(w[pre + "o"] @ torch.cat(heads))
    return torch.stack(out)


# --- feed-forwards ------------------------------------------------------------------

def dense_ff(w, pre, h):
    return torch.stack([w[pre + "down"] @ torch.clamp(w[pre + "up"] @ x, min=0.0) ** 2 for x in h])


def expert(w, pre, x):
    return w[pre + "down"] @ (silu(w[pre + "gate"] @ x) * (w[pre + "up"] @ x))


def route(z, correction, top, scale):
    """Chosen: the ``top`` largest of softmax + correction (ties to the lower
    index); weights: their softmax scores without it, times ``scale``."""
    s = torch.softmax(z, 0)
    c = s + correction
    order = sorted(range(z.numel()), key=lambda e: (-float(c[e]), e))[:top]
    return order, s[order] * scale


def moe_ff(w, pre, mlp, h):
    r = mlp["router"]
    out = []
    for x in h:
        idx, wt = route(w[pre + "router"] @ x, w[pre + "correction"], r["top"], r["scale"])
        y = sum(p * expert(w, f"{pre}e{e}.", x) for e, p in zip(idx, wt))
        if mlp.get("shared"):
            y = y + expert(w, pre + "shared.", x)
        out.append(y)
    return torch.stack(out)


# --- whole model --------------------------------------------------------------------

def forward(cfg, w, tokens, layers_out=None):
    """Logits [T, vocab] of one whole sequence; ``layers_out`` collects the
    stream after every layer."""
    eps = cfg["norm"]["eps"]
    x = w["embed"][torch.tensor(tokens)] * cfg["embedding"]["scale"]
    kv = {}
    for i, spec in enumerate(cfg["layers"]):
        m, mlp, pre = spec["mixer"], spec.get("mlp"), f"l{i}."
        h = dyt(w, pre + "norm1", x)
        if spec["type"] == "attention":
            own = []
            src = m.get("kv_from")
            y = attention(w, pre + "mix.", m, h, eps, kv[src] if src is not None else None, own)
            if own:
                kv[i] = own[0]
        else:
            y = latent_attention(w, pre + "mix.", m, h, eps)
        x = x + dyt(w, pre + "norm1b", y)
        if mlp:
            h = dyt(w, pre + "norm2", x)
            y = dense_ff(w, pre + "mlp.", h) if mlp["kind"] == "dense" else moe_ff(w, pre + "mlp.", mlp, h)
            x = x + dyt(w, pre + "norm2b", y)
        if layers_out is not None:
            layers_out.append(x.clone())
    return dyt(w, "final.norm", x) @ w["head"].T


def random_weights(cfg, seed=0):
    """Random float64 tensors (already rounded to bfloat16 values) under the
    checkpoint's names for a config in config.json form."""
    g = torch.Generator().manual_seed(seed)
    W = cfg["width"]
    w = {}

    def mat(o, i, std=None):
        return (torch.randn(o, i, generator=g, dtype=F64) * (std if std is not None else i ** -0.5)).bfloat16().double()

    def vec(n, about, std=0.2):
        return (about + std * torch.randn(n, generator=g, dtype=F64)).bfloat16().double()

    def norm(name, alpha):
        w[name], w[name + ".b"] = vec(W, 1.0), vec(W, 0.0)
        w[name + ".alpha"] = vec(1, alpha, 0.1)[0]

    w["embed"], w["head"] = mat(cfg["vocab"], W, 0.5), mat(cfg["vocab"], W)
    norm("final.norm", 0.5)
    for i, spec in enumerate(cfg["layers"]):
        m, mlp, pre = spec["mixer"], spec.get("mlp"), f"l{i}."
        H, D, V, mx = m["heads"], m["dim"], m["vdim"], f"l{i}.mix."
        norm(pre + "norm1", 0.7)
        norm(pre + "norm1b", 0.9)
        if spec["type"] == "attention":
            G = m["kv_heads"]
            parts = [("q", 2 * H * D)] + ([] if m.get("kv_from") is not None else [("k", 2 * G * D), ("v", G * V)])
            for n, size in parts:
                w[mx + n], w[mx + n + ".b"] = mat(size, W), vec(size, 0.0)
                w[mx + n + ".conv"] = mat(size, m["conv"], 0.6)
            for n in ("lq1", "lk1", "lq2", "lk2"):
                w[mx + n] = vec(D, 0.0, 0.8 * D ** -0.25)
        else:
            R, C, Q = m["rot_dim"], m["kv_rank"], m["q_rank"]
            w[mx + "dq"], w[mx + "dq.norm"], w[mx + "uq"] = mat(Q, W), vec(Q, 1.0), mat(H * (D + R), Q)
            w[mx + "dkv"], w[mx + "dkv.norm"] = mat(C + R, W), vec(C, 1.0)
            w[mx + "uk"], w[mx + "uv"] = mat(H * D, C), mat(H * V, C)
            w[mx + "sink"] = vec(H, 0.0, 1.5)
        w[mx + "o"] = mat(W, H * V)
        if not mlp:
            continue
        norm(pre + "norm2", 0.6)
        norm(pre + "norm2b", 0.8)
        mp = pre + "mlp."
        if mlp["kind"] == "dense":
            w[mp + "up"], w[mp + "down"] = mat(mlp["ff"], W), mat(W, mlp["ff"])
            continue
        n = mlp["router"]["experts"]
        w[mp + "router"], w[mp + "correction"] = mat(n, W, 1.5 * W ** -0.5), vec(n, 0.0)
        for e, ff in [(f"e{e}", mlp["expert"]["ff"]) for e in range(n)] + (
                [("shared", mlp["shared"]["ff"])] if mlp.get("shared") else []):
            w[f"{mp}{e}.gate"], w[f"{mp}{e}.up"], w[f"{mp}{e}.down"] = mat(ff, W), mat(ff, W), mat(W, ff)
    return w
