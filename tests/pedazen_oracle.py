"""Plain float64 implementation of the Pedazen design, one function per
mechanism, written from the design's equations. It shares no code with the
package: tests compare the engine against it.

``cfg`` is the design's ``config.json`` as a dict, ``w`` maps checkpoint
tensor names to tensors. Every function takes one whole sequence.
"""

import math

import torch

F64 = torch.float64


def rms_unit(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def block_norm(x, weight, eps):
    """The layers' and the final norm: the weight is stored around zero."""
    return rms_unit(x, eps) * (1.0 + weight)


def silu(z):
    return z * torch.sigmoid(z)


def gelu_tanh(z):
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi)
                                       * (z + 0.044715 * z ** 3)))


def _lin(w, name, h):
    return h @ w[name].to(F64).t()


# ---------------------------------------------------------------- mixers

def linear_attention(q, k, v, decay):
    """S <- decay_h S + k v^T, o = S^T q per head, from S = 0. q, k [T, H, d],
    v [T, H, e] -> [T, H, e]."""
    T, H, d = q.shape
    lam = torch.tensor(decay, dtype=F64)[:, None, None]
    S = torch.zeros(H, d, v.shape[-1], dtype=F64)
    out = torch.zeros(T, H, v.shape[-1], dtype=F64)
    for t in range(T):
        S = lam * S + k[t][:, :, None] * v[t][:, None, :]
        out[t] = (S * q[t][:, :, None]).sum(1)
    return out


def lightning(mc, w, p, h, eps):
    T, H = h.shape[0], int(mc["heads"])
    q, k, v = (silu(_lin(w, p + n, h)).view(T, H, -1) for n in ("q", "k", "v"))
    o = linear_attention(q, k, v, mc["decay"]).reshape(T, -1)
    o = rms_unit(o, eps) * w[p + "norm"].to(F64)
    return _lin(w, p + "o", o * torch.sigmoid(_lin(w, p + "g", h)))


def rotate_halves(v, pos, rot):
    """v [..., n] at position pos: entry i pairs with entry i + dims/2."""
    dims = int((rot or {}).get("dims") or 0)
    out = v.clone()
    for i in range(dims // 2):
        f = float(rot["base"]) ** (-2.0 * i / dims)
        c, s = math.cos(pos * f), math.sin(pos * f)
        a, b = v[..., i], v[..., i + dims // 2]
        out[..., i] = a * c - b * s
        out[..., i + dims // 2] = b * c + a * s
    return out


def first_visible(i, mask):
    """Chunked attention: a position sees nothing before its own chunk."""
    size = int((mask or {}).get("size") or 0)
    return i // size * size if size > 0 else 0


def capped(s, cap):
    return cap * torch.tanh(s / cap) if cap else s


def sink_softmax(s, sink):
    """Weights whose denominator also holds exp(sink)."""
    m = max(float(s.max()), float(sink))
    e = torch.exp(s - m)
    return e / (e.sum() + math.exp(float(sink) - m))


def chunk_attention(mc, w, p, h, eps):
    """The left side of the pair."""
    T = h.shape[0]
    H, G, dk, dv = int(mc["heads"]), int(mc["kv_heads"]), int(mc["dim"]), int(mc["vdim"])
    q = rms_unit(_lin(w, p + "q", h).view(T, H, dk), eps) * w[p + "q.norm"].to(F64)
    k = rms_unit(_lin(w, p + "k", h).view(T, G, dk), eps) * w[p + "k.norm"].to(F64)
    v = _lin(w, p + "v", h).view(T, G, dv)
    q = torch.stack([rotate_halves(q[t], t, mc.get("rot")) for t in range(T)])
    k = torch.stack([rotate_halves(k[t], t, mc.get("rot")) for t in range(T)])
    sink = w[p + "sink"].to(F64)
    out = torch.zeros(T, H, dv, dtype=F64)
    for i in range(T):
        lo = first_visible(i, mc.get("mask"))
        for a in range(H):
            g = a // (H // G)
            s = capped((k[lo:i + 1, g] @ q[i, a]) * float(mc["scale"]),
                       float(mc.get("softcap") or 0.0))
            out[i, a] = sink_softmax(s, sink[a]) @ v[lo:i + 1, g]
    return _lin(w, p + "o", out.reshape(T, H * dv))


def short_conv(u, taps_w, bias):
    """y_t = bias + sum_j w[:, j] u_(t - taps + 1 + j), zeros before the start."""
    T, taps = u.shape[0], taps_w.shape[1]
    y = bias.expand(T, -1).clone()
    for t in range(T):
        for j in range(taps):
            s = t - taps + 1 + j
            if s >= 0:
                y[t] = y[t] + taps_w[:, j] * u[s]
    return y


def block_linear(m, b, u):
    """Square matrices on equal parts of u: m [parts, n, n] as [out, in]."""
    parts = u.view(u.shape[0], m.shape[0], m.shape[1])
    return torch.stack([parts[:, i] @ m[i].t() + b[i] for i in range(m.shape[0])],
                       1).reshape(u.shape)


def linear_unit(u, r, i, lam):
    """S <- a S + sqrt(1 - a^2) i u with log a = -8 r softplus(lam), from 0."""
    log_a = -8.0 * r * torch.nn.functional.softplus(lam)
    a = torch.exp(log_a)
    b = torch.sqrt(1.0 - a * a) * i * u
    S = torch.zeros(u.shape[1], dtype=F64)
    out = torch.zeros_like(u)
    for t in range(u.shape[0]):
        S = a[t] * S + b[t]
        out[t] = S
    return out


def recurrent_block(mc, w, p, h, eps):
    """The right side of the pair: real-gated linear recurrent unit."""
    y = gelu_tanh(_lin(w, p + "y", h) + w[p + "y.b"].to(F64))
    u = short_conv(_lin(w, p + "x", h) + w[p + "x.b"].to(F64), w[p + "conv"].to(F64),
                   w[p + "conv.b"].to(F64))
    r = torch.sigmoid(block_linear(w[p + "ra"].to(F64), w[p + "ra.b"].to(F64), u))
    i = torch.sigmoid(block_linear(w[p + "ri"].to(F64), w[p + "ri.b"].to(F64), u))
    return _lin(w, p + "o", linear_unit(u, r, i, w[p + "lam"].to(F64)) * y)


def pair(mc, w, p, h, eps):
    """Half the sum of both sides' outputs, each normed over the width."""
    left = chunk_attention(mc["left"], w, p + "left.", h, eps)
    right = recurrent_block(mc["right"], w, p + "right.", h, eps)
    return 0.5 * (rms_unit(left, eps) * w[p + "left.out"].to(F64)
                  + rms_unit(right, eps) * w[p + "right.out"].to(F64))


# ---------------------------------------------------------- feed-forwards

def dense_ff(w, p, h):
    return _lin(w, p + "down", gelu_tanh(_lin(w, p + "gate", h)) * _lin(w, p + "up", h))


def choose(z, rc):
    """Router logits of one token -> [(expert, weight)], best first."""
    s = torch.softmax(z, -1).tolist()
    n, gc = len(s), rc.get("groups")
    allowed = range(n)
    if gc:
        size = n // int(gc["count"])
        best = sorted(range(int(gc["count"])),
                      key=lambda g: -max(s[g * size:(g + 1) * size]))[:int(gc["keep"])]
        allowed = [e for e in range(n) if e // size in best]
    top = sorted(allowed, key=lambda e: -s[e])[:int(rc["top"])]
    total = sum(s[e] for e in top) + 1e-20
    return [(e, s[e] / total) for e in top]


def expert_ff(fc, w, p, h):
    z = _lin(w, p + "router", h)
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e, wt in choose(z[t], fc["router"]):
            a = torch.relu(_lin(w, f"{p}e{e}.up", h[t])) ** 2
            out[t] = out[t] + wt * _lin(w, f"{p}e{e}.down", a)
    return out


# ------------------------------------------------------------------ model

def layer_runs(cfg):
    """(layer, number of the pass that starts with it or None) in order."""
    n, loop = len(cfg["layers"]), cfg.get("loop")
    if not loop:
        return [(i, None) for i in range(n)]
    a, b, k = int(loop["start"]), int(loop["stop"]), int(loop["times"])
    runs = [(i, None) for i in range(a)]
    for t in range(k):
        runs += [(i, t if i == a else None) for i in range(a, b)]
    return runs + [(i, None) for i in range(b, n)]


def forward(cfg, w, tokens, layers_out=None):
    """Logits [T, vocab] of one sequence; ``layers_out`` (a list) receives
    the residual after every layer run."""
    eps = float(cfg["norm"]["eps"])
    e0 = w["embed"].to(F64)[torch.tensor(tokens)] * float(cfg["embedding"]["scale"])
    x = e0.clone()
    for i, start in layer_runs(cfg):
        lc, p = cfg["layers"][i], f"l{i}."
        if start is not None:
            if start > 0:
                x = x + e0
            x = x + w["loop.step"].to(F64)[start]
        h = block_norm(x, w[p + "norm1"].to(F64), eps)
        mix = {"lightning": lightning, "parallel": pair}[lc["type"]]
        d = mix(lc["mixer"], w, p + "mix.", h, eps)
        fc = lc.get("mlp")
        if fc is not None:
            d = d + (dense_ff(w, p + "mlp.", h) if fc["kind"] == "dense"
                     else expert_ff(fc, w, p + "mlp.", h))
        x = x + d
        if layers_out is not None:
            layers_out.append(x)
    return block_norm(x, w["final.norm"].to(F64), eps) @ w["embed"].to(F64).t()


# ------------------------------------------------- small configs for tests

def dense(ff=14):
    return {"kind": "dense", "ff": ff}


def moe(experts=6, top=2, ff=10, groups=(3, 2)):
    rc = {"experts": experts, "top": top}
    if groups:
        rc["groups"] = {"count": groups[0], "keep": groups[1]}
    return {"kind": "moe", "expert": {"ff": ff}, "router": rc}


def light_layer(heads=3, dim=6, vdim=10, decay=None, mlp=None):
    if decay is None:
        decay = [1.0 - 0.5 * 0.3 ** h for h in range(heads)]
    return {"type": "lightning", "mlp": mlp,
            "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "decay": list(decay)}}


def pair_layer(heads=4, kv_heads=2, dim=8, vdim=5, chunk=7, rot_dims=6, base=50.0, scale=None,
               softcap=3.0, width=12, blocks=3, conv=4, mlp=None):
    left = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim,
            "rot": {"base": base, "dims": rot_dims}, "mask": {"size": chunk},
            "scale": scale if scale is not None else dim ** -0.5, "softcap": softcap}
    return {"type": "parallel", "mlp": mlp,
            "mixer": {"left": left, "right": {"width": width, "blocks": blocks, "conv": conv}}}


def make_cfg(layers, width=20, vocab=37, loop=None, eps=1e-5, embed_scale=3.0):
    cfg = {"architecture": "Pedazen", "embedding": {"scale": embed_scale}, "layers": layers,
           "norm": {"eps": eps}, "vocab": vocab, "width": width}
    if loop:
        cfg["loop"] = dict(zip(("start", "stop", "times"), loop))
    return cfg


def random_weights(cfg, seed=0):
    """Checkpoint tensors of a configuration, rounded to bfloat16 as a
    checkpoint file holds them."""
    g = torch.Generator().manual_seed(seed)
    D = int(cfg["width"])
    w = {}

    def mat(name, rows, cols, gain=1.0):
        w[name] = gain * torch.randn(rows, cols, generator=g) / math.sqrt(cols)

    def vec(name, n, mean=0.0, std=0.1):
        w[name] = mean + std * torch.randn(n, generator=g)

    w["embed"] = torch.randn(int(cfg["vocab"]), D, generator=g) * 0.5
    vec("final.norm", D, 0.0, 0.2)
    if cfg.get("loop"):
        w["loop.step"] = 0.7 * torch.randn(int(cfg["loop"]["times"]), D, generator=g)
    for i, lc in enumerate(cfg["layers"]):
        p, mc = f"l{i}.", lc["mixer"]
        x = p + "mix."
        vec(p + "norm1", D, 0.0, 0.2)
        if lc["type"] == "lightning":
            nq, nv = mc["heads"] * mc["dim"], mc["heads"] * mc["vdim"]
            for nm, rows in (("q", nq), ("k", nq), ("v", nv), ("g", nv)):
                mat(x + nm, rows, D)
            vec(x + "norm", nv, 1.0)
            mat(x + "o", D, nv)
        else:
            lm, rm = mc["left"], mc["right"]
            H, G, dk, dv = lm["heads"], lm["kv_heads"], lm["dim"], lm["vdim"]
            y = x + "left."
            for nm, rows in (("q", H * dk), ("k", G * dk), ("v", G * dv)):
                mat(y + nm, rows, D)
            vec(y + "q.norm", dk, 1.5, 0.3)
            vec(y + "k.norm", dk, 1.5, 0.3)
            vec(y + "sink", H, 0.5, 1.0)
            mat(y + "o", D, H * dv)
            vec(y + "out", D, 1.0, 0.2)
            y, R, B = x + "right.", rm["width"], rm["blocks"]
            for nm in ("y", "x"):
                mat(y + nm, R, D)
                vec(y + nm + ".b", R, 0.0, 0.3)
            w[y + "conv"] = 0.6 * torch.randn(R, rm["conv"], generator=g)
            vec(y + "conv.b", R, 0.0, 0.3)
            for nm in ("ra", "ri"):
                w[y + nm] = torch.randn(B, R // B, R // B, generator=g) / math.sqrt(R // B)
                w[y + nm + ".b"] = 0.3 * torch.randn(B, R // B, generator=g)
            vec(y + "lam", R, -2.5, 1.0)
            mat(y + "o", D, R)
            vec(y + "out", D, 1.0, 0.2)
        f, x = lc.get("mlp"), p + "mlp."
        if f is not None and f["kind"] == "dense":
            for nm in ("gate", "up"):
                mat(x + nm, f["ff"], D)
            mat(x + "down", D, f["ff"])
        elif f is not None:
            # scores well apart: rounding must not change a choice
            mat(x + "router", f["router"]["experts"], D, 4.0)
            for e in range(f["router"]["experts"]):
                mat(f"{x}e{e}.up", f["expert"]["ff"], D)
                mat(f"{x}e{e}.down", D, f["expert"]["ff"])
    return {k: v.to(torch.bfloat16).float() for k, v in w.items()}
