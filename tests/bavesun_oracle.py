"""Plain float64 implementation of the Bavesun design, one function per
mechanism, written token by token from the equations. It shares no code with
the product path; the tests compare the engine with it.

A model is (cfg, w): cfg is the checkpoint's config.json as a dict, w maps
checkpoint tensor names to float64 tensors.

    x = embed[token] * s
    each layer run (the looped range several times over, same weights):
        h = rms(x) (1 + w_norm1)
        x <- x + (mixer(h) + ff(h))                               (no ff: x + mixer(h))
        x <- x + rms(W_proj (gelu(W_gate x) e)) w_side            e = this layer's part of the token's side row
    logits = embed . (rms(x) (1 + w_final))
"""

import math

import torch

F64 = torch.float64


# --- small pieces -----------------------------------------------------------------

def rms(v, eps):
    return v / torch.sqrt((v * v).mean(-1, keepdim=True) + eps)


def norm_about_zero(v, w, eps):
    """The stored weight is the distance from one."""
    return rms(v, eps) * (1.0 + w)


def gelu_tanh(z):
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def silu(z):
    return z * torch.sigmoid(z)


def rotate(vec, p, base, dims, layout):
    """Rotary position on the first ``dims`` entries of vec [..., D] at position p.
    layout 'half': entry i pairs with i + dims/2; 'pairs': 2i with 2i+1."""
    out = vec.clone()
    for i in range(dims // 2):
        a = p * base ** (-2.0 * i / dims)
        i0, i1 = (i, i + dims // 2) if layout == "half" else (2 * i, 2 * i + 1)
        u, v = vec[..., i0], vec[..., i1]
        out[..., i0] = u * math.cos(a) - v * math.sin(a)
        out[..., i1] = v * math.cos(a) + u * math.sin(a)
    return out


# --- mixers: h [T, W], a whole sequence from position 0 -----------------------------

def retention(w, pre, m, h, eps):
    H, D, V = m["heads"], m["dim"], m["vdim"]
    rot = m.get("rot") or {"base": 1.0, "dims": 0}
    decay = torch.tensor(m["decay"], dtype=F64)[:, None, None]
    S = torch.zeros(H, D, V, dtype=F64)
    out = []
    for p, x in enumerate(h):
        q = rotate((w[pre + "q"] @ x).view(H, D), p, rot["base"], rot["dims"], "half")
        k = rotate((w[pre + "k"] @ x).view(H, D), p, rot["base"], rot["dims"], "half") * D ** -0.5
        v = (w[pre + "v"] @ x).view(H, V)
        S = decay * S + k[:, :, None] * v[:, None, :]
        o = rms((S * q[:, :, None]).sum(1), eps)
        out.append(w[pre + "o"] @ (o.reshape(-1) * silu(w[pre + "g"] @ x)))
    return torch.stack(out)


def softmax_with_sink(scores, sink):
    """Weights of the scores when the denominator holds exp(sink) besides."""
    top = torch.maximum(scores.max(), sink)
    e = torch.exp(scores - top)
    return e / (e.sum() + torch.exp(sink - top))


def latent_attention(w, pre, m, h, eps):
    H, D, R, V, C = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    base, dims = m["rot"]["base"], m["rot"]["dims"]
    qs, keys, vals = [], [], []
    for p, x in enumerate(h):
        q = (w[pre + "q"] @ x).view(H, D + R)
        qs.append(torch.cat([q[:, :D], rotate(q[:, D:], p, base, dims, "pairs")], -1))
        d = w[pre + "dkv"] @ x
        c = rms(d[:C], eps) * w[pre + "dkv.norm"]
        kr = rotate(d[C:], p, base, dims, "pairs")
        keys.append(torch.cat([(w[pre + "uk"] @ c).view(H, D), kr.expand(H, R)], -1))
        vals.append((w[pre + "uv"] @ c).view(H, V))
    keys, vals = torch.stack(keys), torch.stack(vals)
    out = []
    for i, x in enumerate(h):
        heads = []
        for hd in range(H):
            pr = softmax_with_sink((keys[:i + 1, hd] @ qs[i][hd]) * m["scale"], w[pre + "sink"][hd])
            heads.append((pr[:, None] * vals[:i + 1, hd]).sum(0))
        out.append(w[pre + "o"] @ (torch.cat(heads) * torch.sigmoid(w[pre + "g"] @ x)))
    return torch.stack(out)


# --- feed-forwards ------------------------------------------------------------------

def dense_ff(w, pre, h):
    return torch.stack([w[pre + "down"] @ (gelu_tanh(w[pre + "gate"] @ x) * (w[pre + "up"] @ x)) for x in h])


def route(z, top):
    """The ``top`` largest logits (ties to the lower index), softmax over them."""
    order = sorted(range(z.numel()), key=lambda e: (-float(z[e]), e))[:top]
    return order, torch.softmax(z[order], 0)


def expert(w, pre, x):
    return w[pre + "down"] @ torch.clamp(w[pre + "up"] @ x, min=0.0) ** 2


def moe_ff(w, pre, mlp, h):
    out = []
    for x in h:
        idx, wt = route(w[pre + "router"] @ x, mlp["router"]["top"])
        out.append(sum(p * expert(w, f"{pre}e{e}.", x) for e, p in zip(idx, wt)))
    return torch.stack(out)


def token_side(w, cfg, i, x, tokens, eps):
    """What layer i adds for the tokens after its feed-forward; x [T, W]."""
    dim, pre = cfg["token_side"]["dim"], f"l{i}.side."
    out = []
    for v, t in zip(x, tokens):
        e = w["side.embed"][t][i * dim:(i + 1) * dim]
        out.append(rms(w[pre + "proj"] @ (gelu_tanh(w[pre + "gate"] @ v) * e), eps) * w[pre + "norm"])
    return torch.stack(out)


# --- whole model --------------------------------------------------------------------

def layer_order(cfg):
    n, lp = len(cfg["layers"]), cfg.get("loop")
    if not lp:
        return list(range(n))
    a, b = lp["start"], lp["stop"]
    return list(range(a)) + list(range(a, b)) * lp["times"] + list(range(b, n))


def forward(cfg, w, tokens, layers_out=None):
    """Logits [T, vocab] of one whole sequence; ``layers_out`` collects the
    stream after every layer run."""
    eps = cfg["norm"]["eps"]
    x = w["embed"][torch.tensor(tokens)] * cfg["embedding"]["scale"]
    for i in layer_order(cfg):
        spec, pre = cfg["layers"][i], f"l{i}."
        h = norm_about_zero(x, w[pre + "norm1"], eps)
        mix = {"retention": retention, "latent_attention": latent_attention}[spec["type"]]
        y = mix(w, pre + "mix.", spec["mixer"], h, eps)
        mlp = spec.get("mlp")
        if mlp:
            y = y + (dense_ff(w, pre + "mlp.", h) if mlp["kind"] == "dense" else moe_ff(w, pre + "mlp.", mlp, h))
        x = x + y
        x = x + token_side(w, cfg, i, x, tokens, eps)
        if layers_out is not None:
            layers_out.append(x.clone())
    return norm_about_zero(x, w["final.norm"], eps) @ w["embed"].T


def random_weights(cfg, seed=0):
    """Random float64 tensors (already rounded to bfloat16 values) under the
    checkpoint's names for a config in config.json form."""
    g = torch.Generator().manual_seed(seed)
    W = cfg["width"]

    def mat(o, i, std=None):
        return (torch.randn(o, i, generator=g, dtype=F64) * (std if std is not None else i ** -0.5)).bfloat16().double()

    def vec(n, about, std=0.2):
        return (about + std * torch.randn(n, generator=g, dtype=F64)).bfloat16().double()

    dim = cfg["token_side"]["dim"]
    w = {"embed": mat(cfg["vocab"], W, 0.5), "side.embed": mat(cfg["vocab"], len(cfg["layers"]) * dim, 1.0),
         "final.norm": vec(W, 0.0)}
    for i, spec in enumerate(cfg["layers"]):
        m, pre = spec["mixer"], f"l{i}."
        H, D, V = m["heads"], m["dim"], m["vdim"]
        w[pre + "norm1"] = vec(W, 0.0)
        if spec["type"] == "retention":
            w[pre + "mix.q"], w[pre + "mix.k"] = mat(H * D, W), mat(H * D, W)
            w[pre + "mix.v"] = mat(H * V, W)
        else:
            R, C = m["rot_dim"], m["kv_rank"]
            w[pre + "mix.q"] = mat(H * (D + R), W)
            w[pre + "mix.dkv"] = mat(C + R, W)
            w[pre + "mix.dkv.norm"] = vec(C, 1.0)
            w[pre + "mix.uk"], w[pre + "mix.uv"] = mat(H * D, C), mat(H * V, C)
            w[pre + "mix.sink"] = vec(H, 0.0, 1.5)
        w[pre + "mix.g"] = mat(H * V, W)
        w[pre + "mix.o"] = mat(W, H * V)
        mlp = spec.get("mlp")
        if mlp and mlp["kind"] == "dense":
            w[pre + "mlp.gate"], w[pre + "mlp.up"] = mat(mlp["ff"], W), mat(mlp["ff"], W)
            w[pre + "mlp.down"] = mat(W, mlp["ff"])
        elif mlp:
            ff, n = mlp["expert"]["ff"], mlp["router"]["experts"]
            for e in range(n):
                w[f"{pre}mlp.e{e}.up"], w[f"{pre}mlp.e{e}.down"] = mat(ff, W), mat(W, ff)
            w[pre + "mlp.router"] = mat(n, W, 1.5 * W ** -0.5)
        w[pre + "side.gate"], w[pre + "side.proj"] = mat(dim, W), mat(W, dim)
        w[pre + "side.norm"] = vec(W, 0.5)
    return w
