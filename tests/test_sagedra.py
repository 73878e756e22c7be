"""Sagedra (residual streams with layer norms, looped layers, differential
attention with short convolutions and query temperature, a normed pair of
windowed attention and gated delta rule, tanh-GELU GLU, capped logits) against
the plain oracle in sagedra_oracle.py.

Every test builds its own small configuration and random weights. The
``dev`` fixture runs each case on the CPU path and, marked ``gpu``, on the
HIP kernels (fp32 and bf16 models).
"""

import json
import math
import os
import subprocess
import sys

import pytest
import torch

import sagedra_oracle as O
from distrl_llm_amd.config import EngineConfig, SamplingParams
from distrl_llm_amd.engine.hybrid_engine import HybridEngine
from distrl_llm_amd.models.hybrid import (HybridLM, rotary_frequencies,
                                          sagedra_config_from_spec,
                                          sagedra_spec_from_config,
                                          save_sagedra_checkpoint)
from distrl_llm_amd.ops import seqmix as SM

CASES = [pytest.param(("cpu", torch.float32), id="cpu-f32"),
         pytest.param(("cuda", torch.float32), id="gpu-f32", marks=pytest.mark.gpu),
         pytest.param(("cuda", torch.bfloat16), id="gpu-bf16", marks=pytest.mark.gpu)]


@pytest.fixture(params=CASES)
def dev(request):
    return request.param


def tol(dtype):
    # bf16 is a coarse check of a deep, narrow model (its rounding noise on
    # the logits is a few percent); the same kernels are held to 2e-4 in fp32
    # and the bf16-only tiled kernel has tests of its own
    return 2e-4 if dtype == torch.float32 else 0.12


def rel_err(got, want):
    got, want = got.double().cpu(), want.double().cpu()
    d = got - want
    return float(d.pow(2).mean().sqrt() / want.pow(2).mean().sqrt().clamp_min(1e-9))


def mixed_cfg():
    """Both mixers twice, sizes unequal wherever the design allows: 1, 2 and 3
    query heads per kv head on either side of the pair, rotated part below and
    equal to the head size, with and without frequency rescaling, convolutions
    of 1 to 4 taps, a layer without feed-forward, and the middle layers looped."""
    return O.make_cfg([
        O.diff_layer(heads=4, kv_heads=2, dim=6, vdim=10, conv=3, every=5),
        O.pair_layer(heads=6, kv_heads=2, dim=8, vdim=5, window=7, rot_dims=6, r_heads=4,
                     r_kv_heads=2, r_dim=5, r_vdim=7, conv=4, mlp=10),
        O.diff_layer(heads=3, kv_heads=1, dim=8, vdim=8, conv=2, diff=0.2, coef=0.5, every=9,
                     mlp=None),
        O.pair_layer(heads=2, kv_heads=2, dim=6, vdim=9, window=11, rot_dims=6, scaling=None,
                     r_heads=3, r_kv_heads=3, r_dim=8, r_vdim=4, conv=1, mlp=18),
    ], width=20, vocab=37, streams=3, loop=(1, 3, 2))


def build(cfg, dev, seed=0, blocks=64, block_size=4, slots=4, W=None):
    device, dtype = dev
    W = W if W is not None else O.random_weights(cfg, seed)
    model = HybridLM(sagedra_spec_from_config(cfg), dtype=dtype, device=device)
    model.load_tensors(W)
    eng = HybridEngine(model, EngineConfig(max_seq_length=4096, kv_block_size=block_size,
                                           num_kv_blocks=blocks, num_state_slots=slots,
                                           max_num_seqs=slots), device=torch.device(device))
    return W, eng


def run_portions(eng, tokens, cuts, capture=None):
    q = eng.open_sequence()
    out, at = [], 0
    for n in cuts:
        out.append(eng.step([(q, tokens[at:at + n])], [list(range(n))], capture=capture))
        at += n
    assert at == len(tokens)
    eng.close_sequence(q)
    return torch.cat(out)


def toks(n, vocab, seed=1):
    g = torch.Generator().manual_seed(seed)
    return torch.randint(0, vocab, (n,), generator=g).tolist()


def ints(v, device):
    return torch.tensor(v, dtype=torch.int32, device=device)


# ------------------------------------------------------ mechanisms alone

@pytest.mark.parametrize("S,D,pair", [(1, 24, False), (2, 7, True), (3, 40, True), (4, 36, False),
                                      (5, 12, True), (9, 18, False)])
def test_stream_update(dev, S, D, pair):
    """Start, closing of a sublayer (with and without the normed sum of two
    sides) and final sum, with a large common offset on the streams so that a
    norm without the mean taken off would show."""
    device, dtype = dev
    g = torch.Generator().manual_seed(S)
    T, eps, V = 5, 1e-4, 11
    w = {"hc1.in": 0.5 + torch.randn(S, generator=g), "hc1.out": torch.randn(S, generator=g),
         "hc1.mix": torch.randn(S, S, generator=g)}
    nw, lw, rw = (1.0 + 0.3 * torch.randn(D, generator=g) for _ in range(3))
    y, y2 = (torch.randn(T, D, generator=g).to(dtype) for _ in range(2))
    y2 *= 8.0                                     # the sides have unequal sizes
    embed = torch.randn(V, D, generator=g).to(dtype)
    ids = torch.tensor([3, 0, 10, 3, 7])
    hb_tol = 2e-6 if dtype == torch.float32 else 5e-3

    def to(t):
        return t.to(device)

    x, h = SM.hyper_start(to(embed), to(ids), 2.5, S, to(w["hc1.in"]), to(nw), eps, dtype, True)
    e = embed[ids].double() * 2.5
    assert tuple(x.shape) == (T, S, D) and h.dtype == dtype
    assert rel_err(x, e[:, None].expand(T, S, D)) < 1e-6
    read = O.layer_norm(w["hc1.in"].double().sum() * e, nw.double(), eps)
    assert rel_err(h.float(), read) < hb_tol

    x0 = torch.randn(T, S, D, generator=g) + 30.0
    side = y.double()
    if pair:
        side = 0.5 * (O.rms_unit(y.double(), eps) * lw.double()
                      + O.rms_unit(y2.double(), eps) * rw.double())
    want = [x0[:, s].double() for s in range(S)]
    want = O.hyper_sublayer(want, w, "", 1, nw, eps, lambda h: side)
    for last in (False, True):
        x = to(x0.clone())
        h = SM.hyper_residual_norm(
            x, to(y), to(y2) if pair else None, to(lw) if pair else None,
            to(rw) if pair else None, 0.5 if pair else 1.0, 0.5, to(w["hc1.mix"]),
            to(w["hc1.out"]), None if last else to(w["hc1.in"]), None if last else to(nw), eps,
            dtype, True)
        assert rel_err(x, torch.stack(want, 1)) < 1e-6
        if last:
            assert h is None
            continue
        u = sum(w["hc1.in"][s].double() * want[s] for s in range(S))
        assert rel_err(h.float(), O.layer_norm(u, nw.double(), eps)) < 10 * hb_tol
        rms = SM.hyper_residual_norm(
            to(x0.clone()), to(y), None, None, None, 1.0, 1.0, to(w["hc1.mix"]),
            to(w["hc1.out"]), to(w["hc1.in"]), to(nw), eps, dtype, False)
        v = O.hyper_sublayer([x0[:, s].double() for s in range(S)], w, "", 1, nw, eps,
                             lambda h: y.double())
        v = sum(w["hc1.in"][s].double() * v[s] for s in range(S))
        assert rel_err(rms.float(), O.rms_unit(v, eps) * nw.double()) < hb_tol
    rows = torch.tensor([4, 1])
    h = SM.hyper_close_norm(x, to(rows), to(nw), eps, dtype, True)
    total = O.layer_norm(sum(want), nw.double(), eps)[rows]
    assert rel_err(h.float(), total) < 10 * hb_tol


def test_glu_and_logit_cap(dev):
    device, dtype = dev
    g = torch.Generator().manual_seed(0)
    for ff in (8, 13, 24):
        gu = (3.0 * torch.randn(5, 2 * ff, generator=g)).to(dtype)
        got = SM.gelu_glu(gu.to(device))
        want = O.gelu_tanh(gu[:, :ff].double()) * gu[:, ff:].double()
        assert got.dtype == dtype
        assert rel_err(got.float(), want) < (1e-6 if dtype == torch.float32 else 5e-3)
        other = SM.silu_glu(gu.to(device))
        assert rel_err(other.float(), O.silu(gu[:, :ff].double()) * gu[:, ff:].double()) < 5e-3
    z = (20.0 * torch.randn(3, 7, generator=g)).to(dtype)
    got = SM.cap_logits(z.to(device), 0.5, 6.0)
    assert got.dtype == torch.float32
    assert rel_err(got, 6.0 * torch.tanh(0.5 * z.double() / 6.0)) < 1e-6
    assert rel_err(SM.cap_logits(z.to(device), 0.5, 0.0), 0.5 * z.double()) < 1e-6


def test_rotary_table():
    for dims, base, sc in ((6, 40.0, (4.0, 1.0, 3.0, 24)), (8, 10000.0, (8.0, 1.0, 4.0, 100)),
                           (10, 3000.0, (16.0, 2.0, 2.5, 64)), (4, 10.0, None),
                           (12, 500.0, (3.0, 0.5, 8.0, 4000))):
        rot = {"dims": dims, "base": base}
        if sc:
            rot["scaling"] = dict(zip(("factor", "low", "high", "original"), sc))
        f, mag = rotary_frequencies(dims, base, ("wavelength", *sc) if sc else None)
        assert f == pytest.approx(O.rotary_table(rot), rel=1e-12) and mag == 1.0
    # all three ranges occur in the second table
    f, _ = rotary_frequencies(8, 10000.0, ("wavelength", 8.0, 1.0, 4.0, 100.0))
    ratio = [a / 10000.0 ** (-2.0 * i / 8) for i, a in enumerate(f)]
    assert ratio[0] == 1.0 and ratio[-1] == pytest.approx(1 / 8)
    assert 1 / 8 < ratio[1] < 1.0 or 1 / 8 < ratio[2] < 1.0


@pytest.mark.parametrize("H,G,dk,dv,maps,rot_dims,unit,temp,taps", [
    (4, 2, 6, 10, 2, 0, False, True, 3), (3, 3, 8, 5, 1, 6, True, False, 0),
    (6, 2, 5, 3, 2, 0, False, True, 4), (2, 1, 72, 4, 1, 70, True, True, 2),
    (1, 1, 2, 1, 2, 2, True, False, 1), (5, 1, 4, 6, 2, 0, False, False, 5),
    (2, 1, 8, 6, 2, 0, False, True, 4)])
def test_prepare(dev, H, G, dk, dv, maps, rot_dims, unit, temp, taps):
    """Convolution with carried tails, rotation, norm after it, query
    temperature and page write: two rows of a step cut into portions down to
    one token, from strided projection rows."""
    device, dtype = dev
    g = torch.Generator().manual_seed(2)
    eps, every, coef = 1e-3, 5, 0.7
    lengths, cuts = [13, 11], [[4, 1, 2, 6], [1, 1, 7, 2]]
    C = (H + G) * maps * dk + G * dv
    rot = {"dims": rot_dims, "base": 77.0,
           "scaling": dict(factor=3.0, low=0.5, high=2.0, original=12)}
    freqs = None
    if rot_dims:
        f, _ = rotary_frequencies(rot_dims, 77.0, ("wavelength", 3.0, 0.5, 2.0, 12.0))
        freqs = torch.tensor(f, dtype=torch.float64).float().to(device)
    cw = torch.randn(C, max(taps, 1), generator=g)
    tails = torch.zeros(4, max(taps, 1) - 1, C, device=device)
    full = [torch.randn(n, C + 6, generator=g).to(dtype) for n in lengths]
    cache = torch.zeros(40, G * (maps * dk + dv), dtype=dtype, device=device)
    slots = ints([2, 0], device)
    got_q, got_c, at = [[], []], [[], []], [0, 0]
    for step in range(4):
        parts = [full[b][at[b]:at[b] + cuts[b][step]] for b in (0, 1)]
        n = [p.shape[0] for p in parts]
        pos = [at[b] + k for b in (0, 1) for k in range(n[b])]
        page = [(7 * p + 3) % 20 + 20 * (i >= n[0]) for i, p in enumerate(pos)]
        cu, seq = [0, n[0], sum(n)], [0] * n[0] + [1] * n[1]
        proj = torch.cat(parts).to(device)[:, :C + 2]
        q = SM.qk_prepare_kv_write(
            proj, H, G, dk, dv, None, None, eps, ints(pos, device), freqs, 1.0, None,
            ints(page, device), cache, maps, unit, (coef, float(every)) if temp else None,
            (cw.to(device), tails, ints(cu, device), ints(seq, device), slots) if taps else None)
        assert tuple(q.shape) == (sum(n), H * maps, dk)
        rows = cache[torch.tensor(page).to(device)]
        for b in (0, 1):
            got_q[b].append(q[cu[b]:cu[b + 1]])
            got_c[b].append(rows[cu[b]:cu[b + 1]])
            at[b] += n[b]
    bound = 1e-5 if dtype == torch.float32 else 6e-3
    for b in (0, 1):
        x = full[b][:, :C].double()
        if taps:
            x = O.short_conv(x, cw.double())
        T = lengths[b]
        q = x[:, :H * maps * dk].reshape(T, H * maps, dk)
        k = x[:, H * maps * dk:(H + G) * maps * dk].reshape(T, G * maps, dk)
        q = torch.stack([O.rotate_halves(q[t], t, rot) for t in range(T)])
        k = torch.stack([O.rotate_halves(k[t], t, rot) for t in range(T)])
        if unit:
            q, k = O.rms_unit(q, eps), O.rms_unit(k, eps)
        if temp:
            q = torch.stack([q[t] * O.query_temperature({"coef": coef, "every": every}, t)
                             for t in range(T)])
        assert rel_err(torch.cat(got_q[b]).float(), q) < bound
        want = torch.cat([k.reshape(T, -1), x[:, (H + G) * maps * dk:]], -1)
        assert rel_err(torch.cat(got_c[b]).float(), want) < bound


def test_query_temperature_steps(dev):
    """The factor changes exactly where (p + 1) / every reaches the next
    whole number."""
    device, dtype = dev
    pos = [0, 2, 3, 6, 7, 62, 63, 4095, 4094]
    proj = torch.ones(len(pos), 4).to(dtype).to(device)
    cache = torch.zeros(16, 2, dtype=dtype, device=device)
    q = SM.qk_prepare_kv_write(proj, 2, 1, 1, 1, None, None, 1e-5, ints(pos, device), None, 1.0,
                               None, ints(list(range(len(pos))), device), cache, 1, False,
                               (0.5, 4.0), None)
    want = torch.tensor([O.query_temperature({"coef": 0.5, "every": 4}, p) for p in pos])
    assert rel_err(q.float()[:, 0, 0], want) < (1e-6 if dtype == torch.float32 else 4e-3)
    assert float(q[1, 0, 0]) < float(q[2, 0, 0]) and float(q[3, 0, 0]) < float(q[4, 0, 0])


def _paged(device, dtype, width, bs, lengths, seed):
    """Random cache rows for sequences of the given lengths, in pages of
    random order: (cache, block tables, rows per sequence)."""
    g = torch.Generator().manual_seed(seed)
    nblk = sum((n + bs - 1) // bs for n in lengths)
    perm = torch.randperm(nblk, generator=g).tolist()
    cache = torch.zeros((nblk + 1) * bs, width, dtype=dtype, device=device)
    tables, kv = [], []
    for n in lengths:
        tables.append([perm.pop() for _ in range((n + bs - 1) // bs)])
        rows = torch.randn(n, width, generator=g).to(dtype)
        kv.append(rows.float())
        idx = torch.tensor([tables[-1][j // bs] * bs + j % bs for j in range(n)])
        cache[idx.to(device)] = rows.to(device)
    most = max(len(t) for t in tables)
    return cache, [t + [0] * (most - len(t)) for t in tables], kv


def _attention(device, dtype, H, G, dk, dv, maps, window, gated, bs, lengths, news, seed=0,
               diff=0.3, eps=1e-4, tweak=None):
    """-> (kernel result, direct float64 result) for the last ``news`` tokens
    of every sequence. ``tweak(kv, q)`` may change rows and queries first."""
    W = G * (maps * dk + dv)
    cache, tables, kv = _paged(device, dtype, W, bs, lengths, seed)
    g = torch.Generator().manual_seed(seed + 50)
    T = sum(news)
    q = torch.randn(T, H * maps, dk, generator=g).to(dtype)
    if tweak is not None:
        tweak(kv, q)
        for b, rows in enumerate(kv):
            idx = torch.tensor([tables[b][j // bs] * bs + j % bs for j in range(lengths[b])])
            cache[idx.to(device)] = rows.to(dtype).to(device)
        kv = [r.to(dtype).float() for r in kv]
    lam_w = 0.4 * torch.randn(4, dk, generator=g)
    wide = torch.randn(T, H * dv + 5, generator=g).to(dtype) if gated else None
    pos, seq, cu = [], [], [0]
    for b, (n, m) in enumerate(zip(lengths, news)):
        pos += list(range(n - m, n))
        seq += [b] * m
        cu.append(cu[-1] + m)
    tiles, mt = SM.query_tiles(news, SM.WIDE_QUERY_TILE)
    got = SM.window_attention(
        q.to(device), cache, H, G, dk, dv, False, ints(tables, device), bs, ints(cu, device),
        ints(seq, device), ints(pos, device), 0.31, window, 0, None, None,
        None if wide is None else wide.to(device)[:, 3:3 + H * dv], dtype,
        tiles=ints(tiles, device), max_tile=mt, maps=maps,
        lam_w=lam_w.to(device) if maps == 2 else None, diff=diff, eps=eps)
    lam = O.differential_lambda({n: lam_w[i] for i, n in enumerate(("lq1", "lk1", "lq2", "lk2"))},
                                "", diff)
    want = torch.zeros(T, H, dv, dtype=torch.float64)
    for t in range(T):
        rows, p = kv[seq[t]].double(), pos[t]
        lo = O.first_visible(p, {"size": window})
        for a in range(H):
            c = a // (H // G)
            v = rows[lo:p + 1, G * maps * dk + c * dv:G * maps * dk + (c + 1) * dv]
            o = []
            for m in range(maps):
                k0 = (c * maps + m) * dk
                s = rows[lo:p + 1, k0:k0 + dk] @ q[t, a * maps + m].double() * 0.31
                o.append(torch.softmax(s, -1) @ v)
            r = o[0] if maps == 1 else O.rms_unit(o[0] - lam * o[1], eps) * (1.0 - diff)
            want[t, a] = r
    want = want.reshape(T, H * dv)
    if wide is not None:
        want = want * torch.sigmoid(wide[:, 3:3 + H * dv].double())
    return got, want


@pytest.mark.parametrize("H,G,dk,dv,maps,window,gated", [
    (4, 2, 6, 10, 2, 0, False), (3, 1, 8, 8, 2, 0, False), (6, 2, 8, 5, 1, 7, True),
    (2, 2, 8, 6, 1, 0, True), (5, 1, 7, 3, 2, 6, True), (3, 3, 8, 1, 1, 4, True)])
def test_attention_op(dev, H, G, dk, dv, maps, window, gated):
    """Prompt portions and single tokens in one step against direct softmaxes:
    two maps with their difference and norm, a gate per entry, windows, pages
    in random order."""
    got, want = _attention(*dev, H, G, dk, dv, maps, window, gated, 4, [23, 9, 14, 1],
                           [11, 1, 14, 1])
    assert rel_err(got.float(), want) < (1e-5 if dev[1] == torch.float32 else 1e-2)


@pytest.mark.parametrize("m", [1, 3, 9])
def test_standout_keys(dev, m):
    """One key made to stand out in one map only, near, at page borders,
    hundreds of tokens back and at the very first position: from a decoded
    token, a portion of three and a longer one."""
    H, G, dk, dv, n = 4, 2, 8, 8, 300
    for which in (0, 1):
        for j_star in (0, 1, 15, 16, 37, 255, 256, n - 2, n - 1):
            def tweak(kv, q):
                kv[0][:, :G * 2 * dk] *= 0.05
                kv[0][j_star].view(-1)[:G * 2 * dk].view(G, 2, dk)[:, which] = 4.0
                kv[0][j_star, G * 2 * dk:] = torch.arange(1, G * dv + 1).float()
                q.view(m, H, 2, dk)[:, :, which] = 4.0
            got, want = _attention(*dev, H, G, dk, dv, 2, 0, False, 16, [n], [m], tweak=tweak)
            assert rel_err(got.float(), want) < (1e-5 if dev[1] == torch.float32 else 2e-2)
            # without the key's own softmax the result is another one
            flat = want[-1].view(H, dv)
            peak = torch.arange(1, dv + 1).double() * (1 if which == 0 else -1)
            cos = torch.nn.functional.cosine_similarity(flat[0], peak, dim=0)
            assert float(cos) > 0.8


def test_window_edges_of_the_op(dev):
    """A standing-out key takes the softmax just inside the window and does
    not count just outside, from a decoded token and from a portion."""
    H, G, dk, dv, n, window = 2, 1, 8, 8, 60, 12
    for m in (1, 9):
        for j_star, seen in ((n - window, True), (n - window - 1, False), (n - 1, True), (3, False)):
            def tweak(kv, q):
                kv[0] *= 0.05
                kv[0][j_star, :dk] = 4.0
                kv[0][j_star, dk:] = torch.arange(1, dv + 1).float()
                q[:] = 4.0
            got, want = _attention(*dev, H, G, dk, dv, 1, window, False, 4, [n], [m], tweak=tweak)
            last = got[-1].float().cpu().view(H, dv)
            if seen:
                assert rel_err(last[0], torch.arange(1, dv + 1).double()) < 2e-2, (m, j_star)
            else:
                assert float(last.abs().max()) < 0.2, (m, j_star)


# ------------------------------------------------------------ whole models

@pytest.mark.parametrize("which", ["differential", "pair"])
def test_single_layer_models(dev, which):
    layer = O.diff_layer(mlp=None) if which == "differential" else O.pair_layer(mlp=None)
    cfg = O.make_cfg([layer], width=24, vocab=31, streams=2)
    W, eng = build(cfg, dev)
    t = toks(25, 31, seed=3)
    want = O.forward(cfg, W, t)
    assert rel_err(run_portions(eng, t, [25]), want) < tol(dev[1])
    assert rel_err(run_portions(eng, t, [9] + [1] * 16), want) < tol(dev[1])


def test_whole_prompt_and_layers(dev):
    cfg = mixed_cfg()
    W, eng = build(cfg, dev)
    t = toks(45, 37, seed=4)
    lay, cap = [], []
    want = O.forward(cfg, W, t, lay)
    got = run_portions(eng, t, [45], capture=cap)
    assert len(cap) == len(lay) == 6                # a looped layer counts each time
    for i, (a, b) in enumerate(zip(cap, lay)):
        assert rel_err(a, b) < tol(dev[1]), i
    assert rel_err(got, want) < tol(dev[1])


@pytest.mark.parametrize("loop", [None, (0, 1, 3), (1, 2, 3), (0, 2, 2), (1, 1, 4), (0, 2, 1)])
def test_loops(dev, loop):
    """Stretches of one and two layers at the start, at the end and over the
    whole model; an empty stretch and a single pass change nothing."""
    cfg = O.make_cfg([O.diff_layer(mlp=8), O.pair_layer(mlp=None)], width=16, vocab=31,
                     streams=2, loop=loop)
    W, eng = build(cfg, dev)
    runs = len(O.layer_runs(cfg))
    assert len(eng.slots.mixer_tails) == len(eng.pool.rows) == runs
    t = toks(23, 31, seed=8)
    want = O.forward(cfg, W, t)
    assert rel_err(run_portions(eng, t, [23]), want) < tol(dev[1])
    assert rel_err(run_portions(eng, t, [3, 2, 9] + [1] * 9), want) < tol(dev[1])


def test_first_tokens(dev):
    """Sequences of one to four tokens, alone and token by token."""
    cfg = mixed_cfg()
    W, eng = build(cfg, dev)
    for n in (1, 2, 3, 4):
        t = toks(n, 37, seed=5 + n)
        want = O.forward(cfg, W, t)
        assert rel_err(run_portions(eng, t, [n]), want) < tol(dev[1])
        assert rel_err(run_portions(eng, t, [1] * n), want) < tol(dev[1])


@pytest.mark.parametrize("cuts", [[1] * 30, [2] * 15, [7, 2, 2, 1, 11, 3, 4], [16, 14], [29, 1],
                                  [3, 27], [15, 2, 13], [5, 25]])
def test_portions(dev, cuts):
    cfg = mixed_cfg()
    W, eng = build(cfg, dev)
    t = toks(30, 37, seed=6)
    assert rel_err(run_portions(eng, t, cuts), O.forward(cfg, W, t)) < tol(dev[1])


def test_portions_do_not_change_fp32_results(dev):
    if dev[1] != torch.float32:
        pytest.skip("fp32 statement")
    cfg = mixed_cfg()
    W, eng = build(cfg, dev)
    t = toks(40, 37, seed=7)
    whole = run_portions(eng, t, [40])
    for cuts in ([1] * 40, [2] * 20, [13, 5, 2, 20], [39, 1]):
        assert rel_err(run_portions(eng, t, cuts), whole) < 2e-5


def test_mixed_batches_and_reuse(dev):
    """Unequal requests in one step (portions beside single tokens, requests
    sitting steps out), pages and slots given back and taken again; every
    position against the oracle and against the request run alone."""
    cfg = mixed_cfg()
    W, eng = build(cfg, dev, blocks=40, slots=3)
    V = 37
    reqs = {k: toks(n, V, seed=10 + i) for i, (k, n) in
            enumerate((("a", 26), ("b", 9), ("c", 17), ("d", 22), ("e", 5)))}
    plan = [[("a", 7), ("b", 2)], [("a", 1), ("b", 3), ("c", 9)], [("a", 1), ("c", 2)],
            [("a", 6), ("b", 4), ("c", 1)], [("c", 5), ("a", 1)], [("a", 10), ("d", 3)],
            [("d", 1), ("e", 2)], [("d", 12), ("e", 1)], [("d", 6), ("e", 2)]]
    live, at, got = {}, {k: 0 for k in reqs}, {k: [] for k in reqs}
    for stepn in plan:
        work, want = [], []
        for k, n in stepn:
            if k not in live:
                live[k] = eng.open_sequence()
            work.append((live[k], reqs[k][at[k]:at[k] + n]))
            want.append(list(range(n)))
        out = eng.step(work, want)
        o = 0
        for k, n in stepn:
            got[k].append(out[o:o + n])
            o += n
            at[k] += n
            if at[k] == len(reqs[k]):
                eng.close_sequence(live.pop(k))
    assert not live
    _, solo = build(cfg, dev, W=W)
    for k, t in reqs.items():
        g = torch.cat(got[k])
        assert rel_err(g, O.forward(cfg, W, t)) < tol(dev[1]), k
        alone = run_portions(solo, t, [len(t)])
        assert rel_err(g, alone) < (1e-5 if dev[1] == torch.float32 else 0.06), k


def test_dirty_pages_and_slots(dev):
    """Freed pages, states and convolution tails hold another request's
    leftovers."""
    cfg = mixed_cfg()
    W, eng = build(cfg, dev, blocks=12, slots=1)
    a, b = toks(40, 37, seed=20), toks(35, 37, seed=21)
    run_portions(eng, a, [40])
    for r in (list(eng.pool.rows.values()) + list(eng.slots.recurrent.values())
              + list(eng.slots.mixer_tails.values())):
        r.add_(5.0)
    assert rel_err(run_portions(eng, b, [20, 15]), O.forward(cfg, W, b)) < tol(dev[1])
    assert eng.pool.allocator.num_free == 12 and eng.slots.num_free == 1


def test_long_decode(dev):
    """120 single-token steps: the window passes over decoded tokens, the
    query temperature rises, the state carries on."""
    cfg = O.make_cfg([O.diff_layer(every=16, mlp=8), O.pair_layer(window=9, mlp=None)],
                     width=16, vocab=31, streams=3, loop=(0, 2, 2))
    W, eng = build(cfg, dev, blocks=48)
    t = toks(132, 31, seed=30)
    got = run_portions(eng, t, [12] + [1] * 120)
    want = O.forward(cfg, W, t)
    assert rel_err(got, want) < tol(dev[1])
    assert rel_err(got[-20:], want[-20:]) < tol(dev[1])


def test_far_key_in_model(dev):
    """Keys are made of the token before (through the convolution) with the
    queries' weights: a rare token at the end finds the place after its only
    earlier occurrence, hundreds of places back, from a portion and decoded.
    Without that occurrence the last logits are others."""
    cfg = O.make_cfg([O.diff_layer(heads=2, kv_heads=2, dim=8, vdim=8, conv=2, every=64, mlp=None)],
                     width=16, vocab=31, streams=2)
    W = O.random_weights(cfg, 5)
    wq = (3.0 * W["l0.mix.q"]).to(torch.bfloat16).float()
    for nm, taps in (("q", (0.0, 1.0)), ("k", (1.0, 0.0)), ("v", (0.0, 1.0))):
        x = f"l0.mix.{nm}"
        W[x + ".conv"] = torch.tensor(taps).repeat(W[x].shape[0], 1)
        if nm != "v":
            W[x], W[x + ".b"] = wq, torch.zeros_like(W[x + ".b"])
    W, eng = build(cfg, dev, blocks=96, W=W)
    base = [x % 30 for x in toks(260, 31, seed=41)]
    base[20] = base[259] = 30
    alt = list(base)
    alt[20] = 7
    far = [O.forward(cfg, W, t)[-1] for t in (base, alt)]
    assert rel_err(far[1], far[0]) > 0.1
    for t, want in zip((base, alt), far):
        for cuts in ([260], [130, 125] + [1] * 5):
            assert rel_err(run_portions(eng, t, cuts)[-1], want) < (
                1e-4 if dev[1] == torch.float32 else 0.05)


def test_window_edges_in_model(dev):
    """With the recurrent side silenced, moving the token just inside the
    window changes a later position's logits and the one just outside does
    not."""
    device, dtype = dev
    cfg = O.make_cfg([O.pair_layer(window=6, mlp=None)], width=16, vocab=31, streams=2)
    W = O.random_weights(cfg, 2)
    W["l0.mix.right.out"] = torch.zeros_like(W["l0.mix.right.out"])
    W, eng = build(cfg, dev, W=W)
    base = toks(20, 31, seed=40)
    ref = run_portions(eng, base, [10] + [1] * 10)[-1]
    for j, seen in ((19 - 5, True), (19 - 6, False), (0, False)):
        alt = list(base)
        alt[j] = (alt[j] + 7) % 31
        for cuts in ([20], [10] + [1] * 10, [13, 2, 5]):
            out = run_portions(eng, alt, cuts)[-1]
            moved = rel_err(out, ref)
            # between two ways of cutting, bf16 rounding moves logits a little
            floor = 1e-3 if dtype == torch.float32 else 3e-2
            assert (moved > floor) == seen, (j, cuts, moved)
            assert rel_err(out, O.forward(cfg, W, alt)[-1]) < tol(dtype)


def test_other_sizes(dev):
    """Values a model may happen to make equal or 1: one head, one stream,
    window 1, one tap, rotation over the whole head, unit scales, no cap, a
    step of one position per temperature level."""
    cfg = O.make_cfg([
        O.diff_layer(heads=1, kv_heads=1, dim=8, vdim=8, conv=1, diff=0.0, coef=0.0, every=1,
                     scale=1.0, mlp=8),
        O.pair_layer(heads=1, kv_heads=1, dim=8, vdim=8, window=1, rot_dims=8, scaling=None,
                     scale=1.0, r_heads=1, r_kv_heads=1, r_dim=8, r_vdim=8, conv=1, mlp=8),
        O.diff_layer(heads=8, kv_heads=8, dim=8, vdim=8, conv=8, every=1, mlp=8),
        O.pair_layer(heads=8, kv_heads=1, dim=8, vdim=8, window=8, rot_dims=8, r_heads=8,
                     r_kv_heads=1, r_dim=8, r_vdim=8, conv=8, mlp=8),
    ], width=8, vocab=11, streams=1, embed_scale=1.0, softcap=0.0)
    W, eng = build(cfg, dev)
    t = toks(21, 11, seed=50)
    want = O.forward(cfg, W, t)
    assert rel_err(run_portions(eng, t, [21]), want) < tol(dev[1])
    assert rel_err(run_portions(eng, t, [5, 2, 1, 13]), want) < tol(dev[1])
    cfg = O.make_cfg([O.diff_layer(heads=10, kv_heads=2, dim=3, vdim=7, conv=6),
                      O.pair_layer(heads=5, kv_heads=1, dim=10, vdim=14, window=3, rot_dims=4,
                                   r_heads=6, r_kv_heads=2, r_dim=9, r_vdim=3, conv=5)],
                     width=30, vocab=19, streams=5, loop=(0, 1, 2))
    W, eng = build(cfg, dev)
    t = toks(19, 19, seed=51)
    assert rel_err(run_portions(eng, t, [6, 13]), O.forward(cfg, W, t)) < tol(dev[1])
    assert rel_err(run_portions(eng, t, [6] + [1] * 13), O.forward(cfg, W, t)) < tol(dev[1])


def test_greedy_generate(dev):
    """Greedy decoding through generate() and its scheduler (small step
    budget, two prompts): every generated token is the oracle's argmax for
    its prefix wherever the oracle's margin is not a rounding matter."""
    cfg = mixed_cfg()
    W, eng = build(cfg, dev, blocks=64, slots=4)
    eng.cfg.step_token_budget = 8
    prompts = [toks(13, 37, seed=60), toks(6, 37, seed=61)]
    sp = SamplingParams(max_tokens=10, temperature=0.0, n=1)
    outs = eng.generate(prompts, sp)
    margin = 1e-3 if dev[1] == torch.float32 else 0.5
    checked = 0
    for p, o in zip(prompts, outs):
        gen = o[0]
        assert len(gen) == 10
        logits = O.forward(cfg, W, p + gen)
        for i, tok in enumerate(gen):
            row = logits[len(p) - 1 + i]
            top2 = torch.topk(row, 2).values
            if float(top2[0] - top2[1]) > margin:
                assert int(row.argmax()) == tok, (i, tok)
                checked += 1
    assert checked >= 5
    assert eng.slots.num_free == 4 and eng.pool.allocator.num_free == 64


def test_fork_shares_pages_and_copies_state(dev):
    cfg = mixed_cfg()
    W, eng = build(cfg, dev, blocks=20, block_size=4)
    t = toks(18, 37, seed=33)
    q = eng.open_sequence()
    eng.step([(q, t[:10])], [[]])
    c = eng.fork_sequence(q)
    tail2 = [(x + 3) % 37 for x in t[10:]]
    out = eng.step([(q, t[10:]), (c, tail2)], [list(range(8)), list(range(8))])
    assert rel_err(out[:8], O.forward(cfg, W, t)[10:]) < tol(dev[1])
    assert rel_err(out[8:], O.forward(cfg, W, t[:10] + tail2)[10:]) < tol(dev[1])
    eng.close_sequence(q)
    eng.close_sequence(c)
    assert eng.pool.allocator.num_free == 20


def test_served_through_the_batcher():
    """The server's app, batcher and sampler drive the design's engine like
    any other: greedy completions repeat, sampled ones fan out."""
    from fastapi.testclient import TestClient

    from distrl_llm_amd.serve import create_app
    from distrl_llm_amd.utils.tokenizer import ByteTokenizer
    cfg = O.make_cfg([O.diff_layer(mlp=8), O.pair_layer(mlp=6)], width=16, vocab=600, streams=2,
                     loop=(0, 1, 2))
    _, eng = build(cfg, ("cpu", torch.float32), blocks=128, block_size=8, slots=8)
    client = TestClient(create_app(eng, ByteTokenizer(vocab_size=600), "tiny-sagedra"))
    body = {"prompt": "2+2=", "max_tokens": 5, "temperature": 0.0}
    a = client.post("/v1/completions", json=body).json()
    b = client.post("/v1/completions", json=body).json()
    assert a["choices"][0]["text"] == b["choices"][0]["text"]
    assert a["usage"]["completion_tokens"] <= 5
    r = client.post("/v1/completions", json={"prompt": ["abcd", "wxyz"], "max_tokens": 3,
                                             "temperature": 1.0, "top_p": 0.9, "n": 2}).json()
    assert len(r["choices"]) == 4
    assert eng.pool.allocator.num_free == 128 and eng.slots.num_free == 8


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_captured_decode_matches_eager(dtype):
    """Every replay of the captured step against the eager step, with eager
    work (another sequence's portion) between the replays."""
    cfg = mixed_cfg()
    dev = ("cuda", dtype)
    W, eng = build(cfg, dev)
    _, eager = build(cfg, dev, W=W)
    eager.cfg.enforce_eager = True
    t, other = toks(30, 37, seed=70), toks(20, 37, seed=71)
    qa, qb, qc = eng.open_sequence(), eager.open_sequence(), eng.open_sequence()
    for q, e in ((qa, eng), (qb, eager)):
        e.step([(q, t[:10])], [[9]])
    for i in range(10, 30):
        a = eng.step([(qa, t[i:i + 1])])
        b = eager.step([(qb, t[i:i + 1])])
        assert rel_err(a, b) < 1e-5, i
        if i % 4 == 0:
            eng.step([(qc, other[i - 10:i - 8])], [[1]])
            torch.cuda.synchronize()
    assert len(eng._decode_graphs) >= 1


@pytest.mark.gpu
@pytest.mark.parametrize("H,G,dk,dv,maps,window,gated,lengths,news", [
    (4, 2, 64, 128, 2, 0, False, [300, 70, 129], [200, 70, 65]),
    (8, 2, 40, 80, 2, 0, False, [257, 64], [257, 5]),
    (2, 2, 128, 256, 2, 0, True, [190], [140]),
    (3, 1, 72, 64, 2, 50, False, [333, 21], [333, 21]),
    (8, 2, 64, 128, 1, 100, True, [450, 90], [300, 90]),
    (4, 4, 96, 40, 1, 33, True, [257], [257]),
])
def test_tiled_attention_kernel(H, G, dk, dv, maps, window, gated, lengths, news):
    """The bf16 MFMA kernel against float64: two maps at every register
    variant, windows that end inside tiles and blocks, a gate per entry."""
    got, want = _attention("cuda", torch.bfloat16, H, G, dk, dv, maps, window, gated, 16, lengths,
                           news, seed=7)
    assert rel_err(got.float(), want) < 1e-2


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("H,G,dk,dv,maps,window,gated,lengths", [
    (8, 2, 64, 128, 2, 0, False, [700, 40, 1, 333]),
    (4, 4, 32, 16, 2, 0, True, [1500, 9]),
    (6, 1, 16, 24, 2, 0, False, [64, 65, 63, 200]),
    (8, 1, 8, 250, 2, 70, True, [400, 90]),
    (3, 1, 40, 8, 2, 0, False, [129, 135, 600]),
    (4, 2, 24, 40, 2, 0, True, [513, 2]),
    (8, 2, 64, 96, 1, 300, True, [700, 40, 1]),
])
def test_grouped_attention_kernel(dtype, H, G, dk, dv, maps, window, gated, lengths):
    """Decode steps through the grouped kernel and its merge of key shares:
    head ratios 1-8, shares without a block, a value width above 128."""
    got, want = _attention("cuda", dtype, H, G, dk, dv, maps, window, gated, 16, lengths,
                           [1] * len(lengths), seed=9)
    assert rel_err(got.float(), want) < (1e-5 if dtype == torch.float32 else 1e-2)


# --------------------------------------------------- files, registry, tools

def test_checkpoint_registry_and_replay(tmp_path):
    """Save a checkpoint, load it through the registry, replay a step trace
    with the command-line tool and compare with the oracle."""
    from distrl_llm_amd.models.registry import hybrid_design_of, load_model_and_engine
    cfg = mixed_cfg()
    W = O.random_weights(cfg, 3)
    model = HybridLM(sagedra_spec_from_config(cfg), dtype=torch.float32, device="cpu")
    model.load_tensors(W)
    assert sagedra_spec_from_config(sagedra_config_from_spec(model.spec),
                                    model.spec.name) == model.spec
    path = str(tmp_path / "tiny")
    save_sagedra_checkpoint(model, path)
    assert hybrid_design_of(path) == "sagedra"
    m2, eng = load_model_and_engine(path, EngineConfig(max_seq_length=256, kv_block_size=4,
                                                       num_kv_blocks=32, num_state_slots=2,
                                                       max_num_seqs=2),
                                    dtype=torch.float32, device=torch.device("cpu"))
    again = m2.export_tensors()
    for k, v in model.export_tensors().items():
        assert torch.equal(v, again[k]), k
    a, b = toks(21, 37, seed=80), toks(11, 37, seed=81)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": a[:9], "want": [8]},
                                     {"id": "b", "tokens": b[:2], "want": []}], "end": []},
             {"step": 1, "entries": [{"id": "b", "tokens": b[2:], "want": [0, 8]},
                                     {"id": "a", "tokens": a[9:10], "want": [0]}], "end": ["b"]},
             {"step": 2, "entries": [{"id": "a", "tokens": a[10:], "want": [10]}], "end": ["a"]}]
    out = tmp_path / "out"
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    env = dict(os.environ, CUDA_VISIBLE_DEVICES="", HIP_VISIBLE_DEVICES="")
    r = subprocess.run([sys.executable, os.path.join(root, "bin", "trace_run"), "--model", path,
                        "--dtype", "float32", "--out", str(out), "--max-tokens", "64"],
                       input="\n".join(json.dumps(s) for s in steps) + "\n", text=True,
                       capture_output=True, env=env, timeout=300)
    assert r.returncode == 0, r.stderr[-2000:]
    assert [ln for ln in r.stdout.split("\n") if ln.startswith("done")] == [
        "done 0", "done 1", "done 2"]
    import numpy as np
    la, lb = O.forward(cfg, W, a), O.forward(cfg, W, b)
    want = {0: la[8:9], 1: torch.stack([lb[2], lb[10], la[9]]), 2: la[20:21]}
    for n, w in want.items():
        got = torch.from_numpy(np.fromfile(out / f"{n}.f32", dtype="<f4").reshape(-1, 37))
        assert rel_err(got, w) < 2e-4, n


def test_loader_names_what_is_missing(tmp_path):
    from safetensors.torch import load_file, save_file
    from distrl_llm_amd.models.hybrid import load_sagedra_checkpoint
    cfg = O.make_cfg([O.diff_layer()], width=16, vocab=31)
    model = HybridLM(sagedra_spec_from_config(cfg), dtype=torch.float32, device="cpu")
    model.random_init(1)
    path = str(tmp_path / "m")
    save_sagedra_checkpoint(model, path)
    f = os.path.join(path, "model.safetensors")
    t = load_file(f)
    save_file({**t, "extra.table": torch.zeros(2)}, f)       # unnamed tensors are left out
    load_sagedra_checkpoint(path, dtype=torch.float32)
    save_file({k: v for k, v in t.items() if k != "l0.hc1.mix"}, f)
    with pytest.raises(ValueError, match="hc1.mix"):
        load_sagedra_checkpoint(path, dtype=torch.float32)


def test_config_errors():
    good = mixed_cfg()
    sagedra_spec_from_config(good)

    def broken(change):
        cfg = json.loads(json.dumps(good))
        change(cfg)
        with pytest.raises((ValueError, KeyError)):
            sagedra_spec_from_config(cfg)

    broken(lambda c: c["layers"][0].update(type="attention_3"))
    broken(lambda c: c["layers"][0]["mixer"].update(kv_heads=3))
    broken(lambda c: c["layers"][0]["mixer"].update(conv=0))
    broken(lambda c: c["layers"][0]["mixer"]["q_temp"].update(every=0))
    broken(lambda c: c["layers"][1]["mixer"]["left"]["rot"].update(dims=5))
    broken(lambda c: c["layers"][1]["mixer"]["left"]["rot"].update(dims=10))
    broken(lambda c: c["layers"][1]["mixer"]["right"].update(kv_heads=3))
    broken(lambda c: c["layers"][1]["mlp"].update(kind="moe"))
    broken(lambda c: c["loop"].update(stop=5))
    broken(lambda c: c["loop"].update(times=0))
    broken(lambda c: c.update(streams=99))
    broken(lambda c: c["layers"][0]["mixer"].pop("scale"))
    assert math.isclose(sagedra_spec_from_config(good).logit_softcap, 9.0)
