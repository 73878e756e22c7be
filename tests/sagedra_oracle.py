"""Plain float64 implementation of the Sagedra design, one function per
mechanism, written position by position from the design's equations. It
shares no code with the package: tests compare the engine against it.

``cfg`` is the design's ``config.json`` as a dict, ``w`` maps checkpoint
tensor names to tensors. Every function takes one whole sequence.
"""

import math

import torch

F64 = torch.float64


def layer_norm(x, weight, eps):
    """Mean taken off, divided by the root of the mean squared deviation,
    times a plain weight."""
    c = x - x.mean(-1, keepdim=True)
    return c / torch.sqrt((c * c).mean(-1, keepdim=True) + eps) * weight


def rms_unit(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def unit_vector(x):
    return x / torch.sqrt((x * x).sum(-1, keepdim=True) + 1e-6)


def silu(z):
    return z * torch.sigmoid(z)


def gelu_tanh(z):
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi)
                                       * (z + 0.044715 * z ** 3)))


def rotary_table(rot):
    """Per-pair frequencies; slow pairs (long wavelengths) are slowed further."""
    dims, base = int(rot["dims"]), float(rot["base"])
    out = []
    sc = rot.get("scaling")
    for i in range(dims // 2):
        f = base ** (-2.0 * i / dims)
        if sc:
            wave, orig = 2.0 * math.pi / f, float(sc["original"])
            low, high = float(sc["low"]), float(sc["high"])
            if wave < orig / high:
                pass
            elif wave > orig / low:
                f = f / float(sc["factor"])
            else:
                s = (orig / wave - low) / (high - low)
                f = (1.0 - s) * f / float(sc["factor"]) + s * f
        out.append(f)
    return out


def rotate_halves(v, pos, rot):
    """v [..., n] at position pos: entry i pairs with entry i + dims/2."""
    if not rot or not int(rot.get("dims") or 0):
        return v
    f = rotary_table(rot)
    half = len(f)
    out = v.clone()
    for i, fi in enumerate(f):
        c, s = math.cos(pos * fi), math.sin(pos * fi)
        a, b = v[..., i], v[..., i + half]
        out[..., i] = a * c - b * s
        out[..., i + half] = b * c + a * s
    return out


def short_conv(u, taps_w):
    """y_t = sum_j w[:, j] u_(t - taps + 1 + j), zeros before the start."""
    T, taps = u.shape[0], taps_w.shape[1]
    y = torch.zeros_like(u)
    for t in range(T):
        for j in range(taps):
            s = t - taps + 1 + j
            if s >= 0:
                y[t] = y[t] + taps_w[:, j] * u[s]
    return y


def query_temperature(qt, p):
    if not qt:
        return 1.0
    return 1.0 + float(qt["coef"]) * math.log(math.floor((p + 1) / qt["every"]) + 1.0)


def first_visible(i, mask):
    size = int((mask or {}).get("size") or 0)
    return max(0, i - size + 1) if size > 0 else 0


def _lin(w, name, h):
    y = h @ w[name].to(F64).t()
    if name + ".b" in w:
        y = y + w[name + ".b"].to(F64)
    return y


def differential_lambda(w, p, diff):
    v = {n: w[p + n].to(F64) for n in ("lq1", "lk1", "lq2", "lk2")}
    return (math.exp(float((v["lq1"] * v["lk1"]).sum()))
            - math.exp(float((v["lq2"] * v["lk2"]).sum())) + float(diff))


def differential_attention(mc, w, p, h, eps):
    """The 'attention' mixer: two softmax maps per head over the same values,
    the second taken off the first, the difference normed per head."""
    T = h.shape[0]
    H, G, dk, dv = int(mc["heads"]), int(mc["kv_heads"]), int(mc["dim"]), int(mc["vdim"])
    rep = H // G
    qkv = []
    for nm in ("q", "k", "v"):
        u = _lin(w, p + nm, h)
        qkv.append(short_conv(u, w[p + nm + ".conv"].to(F64)))
    q, k, v = qkv[0].view(T, H, 2, dk), qkv[1].view(T, G, 2, dk), qkv[2].view(T, G, dv)
    lam, diff = differential_lambda(w, p, mc["diff"]), float(mc["diff"])
    out = torch.zeros(T, H, dv, dtype=F64)
    for i in range(T):
        qi = q[i] * query_temperature(mc.get("q_temp"), i)
        for a in range(H):
            g = a // rep
            maps = []
            for m in range(2):
                s = (k[:i + 1, g, m] @ qi[a, m]) * float(mc["scale"])
                maps.append(torch.softmax(s, -1) @ v[:i + 1, g])
            out[i, a] = rms_unit(maps[0] - lam * maps[1], eps) * (1.0 - diff)
    return _lin(w, p + "o", out.reshape(T, H * dv))


def window_attention(mc, w, p, h, eps):
    """The left side of the pair: rotary, then unweighted q/k norm, sliding
    window, a sigmoid gate on every entry of the result."""
    T = h.shape[0]
    H, G, dk, dv = int(mc["heads"]), int(mc["kv_heads"]), int(mc["dim"]), int(mc["vdim"])
    rep = H // G
    q = _lin(w, p + "q", h).view(T, H, dk)
    k = _lin(w, p + "k", h).view(T, G, dk)
    v = _lin(w, p + "v", h).view(T, G, dv)
    rot = mc.get("rot")
    q = rms_unit(torch.stack([rotate_halves(q[t], t, rot) for t in range(T)]), eps)
    k = rms_unit(torch.stack([rotate_halves(k[t], t, rot) for t in range(T)]), eps)
    out = torch.zeros(T, H, dv, dtype=F64)
    for i in range(T):
        lo = first_visible(i, mc.get("mask"))
        for a in range(H):
            s = (k[lo:i + 1, a // rep] @ q[i, a]) * float(mc["scale"])
            out[i, a] = torch.softmax(s, -1) @ v[lo:i + 1, a // rep]
    out = out.reshape(T, H * dv) * torch.sigmoid(_lin(w, p + "g", h))
    return _lin(w, p + "o", out)


def delta_rule(mc, w, p, h, eps):
    """The right side of the pair: gated delta rule with one decay per head."""
    T = h.shape[0]
    H, G, dk, dv = int(mc["heads"]), int(mc["kv_heads"]), int(mc["dim"]), int(mc["vdim"])
    rep = H // G
    q, k, v = (silu(short_conv(_lin(w, p + nm, h), w[p + nm + ".conv"].to(F64)))
               for nm in ("q", "k", "v"))
    q = unit_vector(q.view(T, G, dk)) * dk ** -0.5
    k = unit_vector(k.view(T, G, dk))
    v = v.view(T, H, dv)
    beta = torch.sigmoid(_lin(w, p + "b", h))
    step = torch.nn.functional.softplus(_lin(w, p + "a", h) + w[p + "dt_bias"].to(F64))
    decay = torch.exp(-torch.exp(w[p + "A_log"].to(F64)) * step)
    gate = silu(_lin(w, p + "g", h)).view(T, H, dv)
    norm = w[p + "norm"].to(F64)
    out = torch.zeros(T, H, dv, dtype=F64)
    for a in range(H):
        S = torch.zeros(dk, dv, dtype=F64)
        for t in range(T):
            kt, qt = k[t, a // rep], q[t, a // rep]
            S = decay[t, a] * S
            u = beta[t, a] * (v[t, a] - S.t() @ kt)
            S = S + torch.outer(kt, u)
            out[t, a] = rms_unit(S.t() @ qt, eps) * norm * gate[t, a]
    return _lin(w, p + "o", out.reshape(T, H * dv))


def parallel_pair(mc, w, p, h, eps):
    """Half the sum of both sides' outputs, each normed over the width."""
    left = window_attention(mc["left"], w, p + "left.", h, eps)
    right = delta_rule(mc["right"], w, p + "right.", h, eps)
    return 0.5 * (rms_unit(left, eps) * w[p + "left.out"].to(F64)
                  + rms_unit(right, eps) * w[p + "right.out"].to(F64))


def dense_ff(w, p, h):
    return (gelu_tanh(h @ w[p + "gate"].to(F64).t()) * (h @ w[p + "up"].to(F64).t())
            ) @ w[p + "down"].to(F64).t()


def hyper_sublayer(xs, w, p, q, norm_w, eps, sublayer):
    """xs: list of streams. The sublayer reads a weighted sum of the streams;
    every new stream is a mix of the old ones plus its share of the output."""
    r = w[f"{p}hc{q}.in"].to(F64)
    o = w[f"{p}hc{q}.out"].to(F64)
    M = w[f"{p}hc{q}.mix"].to(F64)
    u = sum(r[s] * xs[s] for s in range(len(xs)))
    y = sublayer(layer_norm(u, norm_w.to(F64), eps))
    return [sum(M[s, t] * xs[s] for s in range(len(xs))) + o[t] * y
            for t in range(len(xs))]


def layer_runs(cfg):
    """Layer indices in the order they run: a stretch of them several times."""
    n = len(cfg["layers"])
    loop = cfg.get("loop")
    if not loop:
        return list(range(n))
    a, b, k = int(loop["start"]), int(loop["stop"]), int(loop["times"])
    return list(range(a)) + list(range(a, b)) * k + list(range(b, n))


def forward(cfg, w, tokens, layers_out=None):
    """Logits [T, vocab] of one sequence; ``layers_out`` (a list) receives
    the sum of the streams after every layer run."""
    eps = float(cfg["norm"]["eps"])
    x0 = w["embed"].to(F64)[torch.tensor(tokens)] * float(cfg["embedding"]["scale"])
    xs = [x0.clone() for _ in range(int(cfg["streams"]))]
    for i in layer_runs(cfg):
        lc, p = cfg["layers"][i], f"l{i}."
        mixers = {"attention": differential_attention, "parallel": parallel_pair}
        mix = mixers[lc["type"]]
        xs = hyper_sublayer(xs, w, p, 1, w[p + "norm1"], eps,
                            lambda h: mix(lc["mixer"], w, p + "mix.", h, eps))
        if lc.get("mlp") is not None:
            xs = hyper_sublayer(xs, w, p, 2, w[p + "norm2"], eps,
                                lambda h: dense_ff(w, p + "mlp.", h))
        if layers_out is not None:
            layers_out.append(sum(xs))
    x = layer_norm(sum(xs), w["final.norm"].to(F64), eps)
    logits = x @ w["head"].to(F64).t()
    cap = float(cfg.get("logit_softcap") or 0.0)
    return cap * torch.tanh(logits / cap) if cap else logits


# ------------------------------------------------- small configs for tests

def diff_layer(heads=4, kv_heads=2, dim=6, vdim=10, conv=3, diff=0.4, coef=0.25, every=5,
               scale=None, mlp=14):
    """An 'attention' layer; ``mlp`` an int (feed-forward width) or None."""
    mc = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": conv,
          "diff": diff, "q_temp": {"coef": coef, "every": every},
          "scale": scale if scale is not None else dim ** -0.5}
    return {"type": "attention", "mixer": mc, "mlp": _mlp(mlp)}


def pair_layer(heads=6, kv_heads=2, dim=8, vdim=5, window=7, rot_dims=6, base=40.0,
               scaling=(4.0, 1.0, 3.0, 24), scale=None, r_heads=4, r_kv_heads=2, r_dim=5,
               r_vdim=7, conv=4, mlp=14):
    """A 'parallel' layer; ``scaling`` (factor, low, high, original) or None."""
    rot = {"base": base, "dims": rot_dims}
    if scaling:
        rot["scaling"] = dict(zip(("factor", "low", "high", "original"), scaling))
    left = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "rot": rot,
            "mask": {"size": window}, "scale": scale if scale is not None else dim ** -0.5}
    right = {"heads": r_heads, "kv_heads": r_kv_heads, "dim": r_dim, "vdim": r_vdim,
             "conv": conv}
    return {"type": "parallel", "mixer": {"left": left, "right": right}, "mlp": _mlp(mlp)}


def _mlp(ff):
    return None if ff is None else {"kind": "dense", "ff": ff}


def make_cfg(layers, width=24, vocab=37, streams=3, loop=None, eps=1e-5, embed_scale=3.0,
             softcap=9.0):
    cfg = {"architecture": "Sagedra", "embedding": {"scale": embed_scale}, "layers": layers,
           "logit_softcap": softcap, "norm": {"eps": eps}, "streams": streams,
           "vocab": vocab, "width": width}
    if loop:
        cfg["loop"] = dict(zip(("start", "stop", "times"), loop))
    return cfg


def random_weights(cfg, seed=0):
    """Checkpoint tensors of a configuration, rounded to bfloat16 as a
    checkpoint file holds them."""
    g = torch.Generator().manual_seed(seed)
    D, S = int(cfg["width"]), int(cfg["streams"])
    w = {}

    def mat(name, rows, cols):
        w[name] = torch.randn(rows, cols, generator=g) / math.sqrt(cols)

    def vec(name, n, mean=0.0, std=0.1):
        w[name] = mean + std * torch.randn(n, generator=g)

    w["embed"] = torch.randn(int(cfg["vocab"]), D, generator=g) * 0.5
    vec("final.norm", D, 1.0)
    mat("head", int(cfg["vocab"]), D)
    w["head"] *= 3.0
    for i, lc in enumerate(cfg["layers"]):
        p, mc = f"l{i}.", lc["mixer"]
        x = p + "mix."
        for q in (1, 2):
            if q == 2 and lc.get("mlp") is None:
                continue
            vec(f"{p}norm{q}", D, 1.0)
            vec(f"{p}hc{q}.in", S, 1.0 / S, 0.3)
            vec(f"{p}hc{q}.out", S, 1.0, 0.3)
            w[f"{p}hc{q}.mix"] = torch.eye(S) + 0.2 * torch.randn(S, S, generator=g)
        if lc["type"] == "attention":
            H, G, dk, dv = mc["heads"], mc["kv_heads"], mc["dim"], mc["vdim"]
            for nm, rows in (("q", H * 2 * dk), ("k", G * 2 * dk), ("v", G * dv)):
                mat(x + nm, rows, D)
                vec(x + nm + ".b", rows, 0.0, 0.3)
                w[x + nm + ".conv"] = 0.6 * torch.randn(rows, mc["conv"], generator=g)
            for nm in ("lq1", "lk1", "lq2", "lk2"):
                vec(x + nm, dk, 0.0, 0.3)
            mat(x + "o", D, H * dv)
            vec(x + "o.b", D, 0.0, 0.3)
        else:
            lm, rm = mc["left"], mc["right"]
            H, G, dk, dv = lm["heads"], lm["kv_heads"], lm["dim"], lm["vdim"]
            for nm, rows in (("q", H * dk), ("k", G * dk), ("v", G * dv), ("g", H * dv)):
                mat(x + "left." + nm, rows, D)
            mat(x + "left.o", D, H * dv)
            H, G, dk, dv = rm["heads"], rm["kv_heads"], rm["dim"], rm["vdim"]
            y = x + "right."
            for nm, rows in (("q", G * dk), ("k", G * dk), ("v", H * dv)):
                mat(y + nm, rows, D)
                w[y + nm + ".conv"] = 0.6 * torch.randn(rows, rm["conv"], generator=g)
            mat(y + "g", H * dv, D)
            mat(y + "a", H, D)
            mat(y + "b", H, D)
            vec(y + "A_log", H, -1.0, 0.5)
            vec(y + "dt_bias", H, -0.5, 0.5)
            vec(y + "norm", dv, 1.0)
            mat(y + "o", D, H * dv)
            vec(x + "left.out", D, 1.0, 0.2)
            vec(x + "right.out", D, 1.0, 0.2)
        if lc.get("mlp") is not None:
            ff = lc["mlp"]["ff"]
            mat(p + "mlp.gate", ff, D)
            mat(p + "mlp.up", ff, D)
            mat(p + "mlp.down", D, ff)
    return {k: v.to(torch.bfloat16).float() for k, v in w.items()}
