"""Tugelorn on the GPU against tests/plain_tugelorn.py: every mechanism through its C entry points, then whole models through the
decoder -- prompts, portions, single tokens, memory that is used again, greedy generation."""
import ctypes as C
import os
import subprocess
import sys

import numpy as np
import pytest

import plain_hybrid as ph
import plain_tugelorn as pt
import tugelorn_models as tm
import ug_amd
from gpu_calls import BF16, F32, GLU, SWIGLU, Attention, Delta, Gpu, Product, RowStep, View, Z, close, get, p, rand, view
from ug_amd import rng

pytestmark = pytest.mark.gpu

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))


@pytest.fixture
def gpu(hip):
    return Gpu(hip)


# ---- products, norms and single rows -----------------------------------------------------------------------------------------
# limits that cut most and nearly nothing; sizes of every kernel a product with a gated unit takes
@pytest.mark.parametrize("m, n, k", [(1, 1, 1), (3, 5, 7), (70, 66, 130), (2, 300, 96), (200, 264, 320), (300, 1032, 256)])
@pytest.mark.parametrize("mode", [F32, BF16])
@pytest.mark.parametrize("limit, alpha, shift", [(0.4, 1.702, 1.0), (2.5, 1.0, 0.0), (0.0, 0.5, 2.0)])
def test_gated_units_with_a_limit(gpu, m, n, k, mode, limit, alpha, shift):
    x, w, bias = rand(1, m, k), rand(2, 2 * n, k, std=k ** -0.5), rand(3, 2 * n, std=0.5)
    y = x @ w.T + bias
    cut = limit or 1e9
    g, u = np.minimum(y[:, :n], cut), np.clip(y[:, n:], -cut, cut)
    want = g * pt.sigmoid(alpha * g) * (u + shift)
    db = gpu.up(bias)
    for half in ((False, True) if mode == BF16 else (False,)):
        dx, dw, dst = gpu.up(x, bf16=half), gpu.up(w, bf16=mode == BF16), gpu.out(m * n, bf16=half)
        q = Product(x=view(dx, 0, k), dst=view(dst, 0, n), w=dw.raw(), bias=db.raw(), m=m, n=n, k=k, product=mode, act=GLU, act_alpha=alpha, act_shift=shift, act_limit=limit)
        gpu.call("ughip_product_rows", C.byref(q))
        close(get(dst, (m, n)), want, 3e-5, rel=2.0 ** -8 if half else 0.0)
    row, out = gpu.up(x[0]), gpu.out(n)
    q = RowStep(x=row.raw(), w=dw.raw(), bias=db.raw(), n=n, k=k, dst=out.raw(), act=GLU, act_alpha=alpha, act_shift=shift, act_limit=limit)
    gpu.call("ughip_product_row", C.byref(q))
    close(get(out, (1, n)), want[:1], 3e-5)
    # the fields say nothing to the plain unit
    q = RowStep(x=row.raw(), w=dw.raw(), bias=db.raw(), n=n, k=k, dst=out.raw(), act=SWIGLU, act_alpha=9.0, act_shift=9.0, act_limit=1e-3)
    gpu.call("ughip_product_row", C.byref(q))
    close(get(out, (1, n)), (ph.silu(y[:, :n]) * y[:, n:])[:1], 3e-5)


@pytest.mark.parametrize("n", [1, 90, 256, 1028, 4096, 5000])
@pytest.mark.parametrize("pad", [0, 3])
def test_norms_behind_and_ahead(gpu, n, pad):
    """A normed output joins the residual (and rows that join as they are), and the sum leaves once more normed for the next sublayer."""
    m, eps, s = 7, 2e-3, n + pad
    x, y, e, w, nxt = rand(1, m, s), rand(2, m, s), rand(3, m, s), rand(4, n), rand(5, n)
    sx, sy, se, sw, sn = gpu.up(x), gpu.up(y), gpu.up(e), gpu.up(w), gpu.up(nxt)
    none = View(None, 0, 0)
    vx, vy, ve = view(sx, 0, s), view(sy, 0, s), view(se, 0, s)
    x, y, e = x[:, :n], y[:, :n], e[:, :n]
    for bf16 in (False, True):
        for yy, ee, second in ((True, False, True), (True, True, True), (False, True, True), (True, True, False), (False, True, False)):
            dst, copy = gpu.out(m * s), gpu.out(m * n, bf16=bf16)
            gpu.call("ughip_add_rms_norm_rows", vx, vy if yy else none, None, None, Z(0), Z(0), p(sw) if yy else None, C.c_float(eps), ve if ee else none, view(dst, 0, s),
                     p(sn) if second else None, p(copy), Z(m), Z(n))
            want = x + (ph.rms(y, eps) * w if yy else 0) + (e if ee else 0)
            close(get(dst, (m, s))[:, :n], want, 3e-6)
            close(get(copy, (m, n)), ph.rms(want, eps) * nxt if second else want, 5e-6, rel=2.0 ** -8 if bf16 else 0.0)


@pytest.mark.parametrize("k, groups", [(4, 1), (90, 3), (256, 64), (256, 8), (1024, 8), (2048, 16), (2048, 2), (3072, 24), (5632, 11), (96, 4)])
@pytest.mark.parametrize("bf16", [False, True])
def test_one_row_normed_then_gated(gpu, k, groups, bf16):
    """v = norm(x) per part, times sigmoid(gate); and a residual that other rows join, normed for the product."""
    eps, n = 1e-3, 37
    x, gate, norm, w, y, yn, e = rand(1, k), rand(2, k), rand(3, k) + 1, rand(4, n, k, std=k ** -0.5), rand(5, k), rand(6, k) + 1, rand(7, k)
    dw, dn, dyn = gpu.up(w, bf16=bf16), gpu.up(norm), gpu.up(yn)
    buf = gpu.up(np.concatenate([np.zeros(4), x, gate, y, e]))
    out = gpu.out(n)
    q = RowStep(x=buf.raw(), x_offset=4, gate=buf.raw(), gate_offset=4 + k, gate_after=1, norm=dn.raw(), norm_groups=groups, eps=eps, w=dw.raw(), n=n, k=k, dst=out.raw())
    gpu.call("ughip_product_row", C.byref(q))
    close(get(out, n), w @ (ph.rms(x.reshape(groups, -1), eps).reshape(-1) * norm * pt.sigmoid(gate)), 3e-5)
    dst = gpu.out(k + n)
    q = RowStep(x=buf.raw(), x_offset=4, y=buf.raw(), y_offset=4 + 2 * k, y_norm=dyn.raw(), extra=buf.raw(), extra_offset=4 + 3 * k, norm=dn.raw(), norm_groups=1, eps=eps, keep_x=1,
                w=dw.raw(), n=n, k=k, dst=dst.raw(), dst_offset=k)
    gpu.call("ughip_product_row", C.byref(q))
    joined = x + ph.rms(y, eps) * yn + e
    close(get(dst, k + n)[:k], joined, 3e-6)
    close(get(dst, k + n)[k:], w @ (ph.rms(joined, eps) * norm), 3e-5)


# ---- grouped attention -------------------------------------------------------------------------------------------------------
# (heads, kv_heads, dim, vdim, rot): one of everything, odd sizes, the sizes the kernels are built for, more pairs than a row block
HEADS = [(1, 1, 1, 1, 0), (1, 1, 2, 3, 2), (6, 3, 22, 27, 14), (4, 1, 17, 9, 16), (8, 2, 64, 64, 64), (6, 2, 128, 70, 32), (40, 1, 48, 128, 20), (4, 2, 190, 100, 190), (3, 3, 256, 200, 8)]


def attend(gpu, mode, qkv, caches, cap, t, pos, sizes, window, scale, tables, factor, out_bf16=False, pad=0):
    H, G, d, vd, rot = sizes
    wide = (H + G) * d + G * vd
    src = gpu.up(np.concatenate([qkv[pos : pos + t], np.full((t, pad), np.nan)], axis=1))
    dst = gpu.out(t * H * vd, bf16=out_bf16)
    q = Attention(view(src, 0, wide + pad), view(dst, 0, H * vd), caches[0].raw(), caches[1].raw(), tables[0].raw() if rot else None, tables[1].raw() if rot else None,
                  factor.raw() if factor is not None else None, cap, len(qkv), rot, window, t, pos, H, G, d, vd, scale)
    gpu.call("ughip_grouped_attention", C.byref(q))
    return get(dst, (t, H, vd))


def caches_for(gpu, G, d, vd, cap, bf16):
    rows, k, v = Z(), Z(), Z()
    assert gpu.lib.ughip_grouped_attention_cache(Z(G), Z(d), Z(vd), Z(cap), C.byref(rows), C.byref(k), C.byref(v)) == 0
    assert rows.value >= cap
    return gpu.out(k.value, bf16=bf16), gpu.out(v.value, bf16=bf16)      # not-a-number everywhere


@pytest.mark.parametrize("sizes", HEADS)
@pytest.mark.parametrize("cuts, window", [((1, 1, 1, 1), 0), ((150, 1, 1), 0), ((150, 1, 1), 64), ((61, 3, 16, 17, 40, 1), 33), ((64, 64, 1, 2), 1), ((130, 130, 1), 96), ((7, 2, 120, 1), 500),
                                          ((300, 1, 2, 1), 65), ((31, 1, 1, 31, 1), 32)])
@pytest.mark.parametrize("bf16", [False, True])
def test_grouped_attention(gpu, sizes, cuts, window, bf16):
    """Any cut of a sequence, caches that held something else.  One key of every query stands out (its score is some 8 above the rest):
    the first, the last, ones at the borders of tiles, the oldest the window shows and -- further up still -- the one just outside it."""
    H, G, d, vd, rot = sizes
    T, per, scale, base, factor = sum(cuts), H // G, 0.4 / np.sqrt(d), 300.0, 1.7
    qkv = rand(1, T, (H + G) * d + G * vd)
    k = qkv[:, H * d : (H + G) * d].reshape(T, G, d)
    v = qkv[:, (H + G) * d :].reshape(T, G, vd)
    turn = lambda x, pos: pt.rotate_pairs(x, pos, base, rot, factor) if rot else x
    k_rot = turn(k, np.arange(T))
    temp = pt.query_temperature(np.arange(T), 0.35, 20)
    q = qkv[:, : H * d].reshape(T, H, d)
    for i in range(T):
        oldest = max(0, i - window + 1) if window else 0
        marks = [oldest, oldest - 1, i, 0, i - 1, i // 32 * 32 - 1, i // 64 * 64, 31]
        for h in range(H):
            far = min(max(marks[(i + h) % len(marks)], 0), i)
            target = turn(k_rot[far, h // per][None, None], [-i])[0, 0]
            target = target * (8.0 / (scale * temp[i] * (target @ target) + 1e-3))
            q[i, h] = rng.bf16_round((0.3 * q[i, h] + target).astype(np.float32))
    want = pt.grouped_attention(turn(q, np.arange(T)) * temp[:, None, None], k_rot, v, scale, window or None)
    ang = np.arange(T)[:, None] * base ** (-2.0 * np.arange(max(rot, 2) // 2) / max(rot, 2)) / factor
    tables, factors = (gpu.up(np.cos(ang)), gpu.up(np.sin(ang))), gpu.up(temp)
    cap, pos = T + 1, 0
    caches = caches_for(gpu, G, d, vd, cap, bf16)
    out_bf16 = bf16 and d == 128
    for t in cuts:
        got = attend(gpu, bf16, qkv, caches, cap, t, pos, sizes, window, scale, tables, factors, out_bf16, pad=4 * (pos % 2))
        close(got, want[pos : pos + t], 0.12 if bf16 else 1e-4, rel=2.0 ** -8 if out_bf16 else 0.0)
        if bf16:  # single keys decide: a wrong one is far off, rounding is not
            assert np.sqrt(np.mean((got - want[pos : pos + t]) ** 2)) <= (0.012 if d > 16 else 0.06) * np.sqrt(np.mean(want[pos : pos + t] ** 2)), (t, pos)
        pos += t


def test_grouped_attention_over_many_splits(gpu):
    """One position behind thousands: every workgroup's share counts, with a window and without."""
    sizes, T, scale = (4, 2, 64, 64, 0), 5000, 0.05
    H, G, d, vd, _ = sizes
    qkv = rand(3, T, (H + G) * d + G * vd)
    k, v = qkv[:, H * d : (H + G) * d].reshape(T, G, d), qkv[:, (H + G) * d :].reshape(T, G, vd)
    for window in (0, 2900):
        caches = caches_for(gpu, G, d, vd, T, False)
        attend(gpu, False, qkv, caches, T, T - 3, 0, sizes, window, scale, None, None)
        for t, pos in ((1, T - 3), (2, T - 2)):
            got = attend(gpu, False, qkv, caches, T, t, pos, sizes, window, scale, None, None)
            want = pt.grouped_attention(qkv[pos : pos + t, : H * d].reshape(t, H, d), k[: pos + t], v[: pos + t], scale, window or None, first=pos)
            close(got, want, 1e-4)


# ---- delta rule --------------------------------------------------------------------------------------------------------------
# (heads, kv_heads, dim, vdim, taps, decay rank, gate rank)
DELTAS = [(1, 1, 1, 1, 1, 1, 1), (6, 2, 18, 21, 3, 7, 5), (4, 4, 64, 64, 4, 16, 8), (2, 1, 128, 128, 2, 24, 128), (3, 3, 100, 40, 5, 64, 136), (2, 2, 190, 24, 4, 8, 8), (1, 1, 256, 250, 3, 16, 16)]


@pytest.mark.parametrize("sizes", DELTAS)
@pytest.mark.parametrize("cuts", [(1, 1, 1, 1, 1, 1), (150,), (64, 64, 1), (65, 2, 3, 1, 63), (2, 2, 5), (17, 1, 130, 16), (33, 32, 31)])
@pytest.mark.parametrize("decay", ["mild", "strong", "none"])
def test_delta_rule_rows_and_steps(gpu, sizes, cuts, decay):
    """Any cut of a sequence gives the plain recurrence: chunks, single steps, the taps' ring -- from memory that held something else.
    Strong decays leave nothing of the state within a few positions in some channels and much in others."""
    H, G, d, vd, taps, ra, rg = sizes
    T, ch, eps, per = sum(cuts), 2 * G * d + H * vd, 1e-4, H // G
    wide = ch + ra + rg + H + 3
    row = rand(1, T, wide)
    bias = {"mild": rand(4, H * d) - 3, "strong": 6 * rand(4, H * d), "none": np.full(H * d, -30.0)}[decay]
    w = {"conv": rand(2, ch, taps), "a_log": rand(3, H), "dt_bias": bias, "norm": rand(5, vd) + 1, "w_a": rand(6, H * d, ra, std=ra ** -0.5), "w_z": rand(7, H * vd, rg, std=rg ** -0.5)}
    act = ph.silu(ph.causal_conv(row[:, 3 : 3 + ch], w["conv"], 0.0))
    q, k, v = act[:, : G * d].reshape(T, G, d), act[:, G * d : 2 * G * d].reshape(T, G, d), act[:, 2 * G * d :].reshape(T, H, vd)
    a_in, z_in, b = row[:, 3 + ch : 3 + ch + ra], row[:, 3 + ch + ra : 3 + ch + ra + rg], row[:, 3 + ch + ra + rg :]
    a, z = a_in @ w["w_a"].T, z_in @ w["w_z"].T
    log_g = -np.exp(w["a_log"])[:, None] * ph.softplus(a + w["dt_bias"]).reshape(T, H, d)
    o = pt.delta_scan(pt.unit(q) * d ** -0.5, pt.unit(k), v, log_g, pt.sigmoid(b))
    want = (ph.rms(o, eps) * w["norm"] * pt.sigmoid(z.reshape(T, H, vd))).reshape(T, H * vd)

    s = {n: gpu.up(x) for n, x in w.items()}
    src, sa, sz = gpu.up(row), gpu.up(a), gpu.up(z)
    S, ring, qkv, dst, step = gpu.out(H * d * vd), gpu.out(taps * ch), gpu.out(T * ch), gpu.out(T * H * vd), gpu.out(2 * H * vd)
    common = dict(heads=H, kv_heads=G, dim=d, vdim=vd, a_log=s["a_log"].raw(), dt_bias=s["dt_bias"].raw(), norm=s["norm"].raw(), s=S.raw(), eps=eps)
    pos, got = 0, np.zeros((T, H * vd))
    for t in cuts:
        if t == 1 and pos % 2 == 0:
            one = gpu.up(row[pos])
            gpu.call("ughip_delta_step", C.byref(Delta(t=1, pos=pos, p=one.raw(), qkv_offset=3, a_offset=3 + ch, z_offset=3 + ch + ra, b_offset=3 + ch + ra + rg, a_rank=ra, z_rank=rg,
                                                       n_taps=taps, taps=s["conv"].raw(), w_a=s["w_a"].raw(), w_z=s["w_z"].raw(), ring=ring.raw(), out=step.raw(), **common)))
            y = get(step, (2, H, vd))
            close(y[1].reshape(-1), z[pos], 3e-5)
            got[pos] = (ph.rms(y[0], eps) * w["norm"] * pt.sigmoid(y[1])).reshape(-1)
        else:
            gpu.call("ughip_conv_silu_rows", view(src, pos * wide + 3, wide), p(s["conv"]), None, Z(taps), p(ring), Z(pos), Z(t), Z(ch), view(qkv, pos * ch, ch))
            gpu.call("ughip_conv_ring_store", view(src, pos * wide + 3, wide), Z(taps), p(ring), Z(pos), Z(t), Z(ch))
            gpu.call("ughip_delta_rows", C.byref(Delta(t=t, pos=pos, qkv=view(qkv, pos * ch, ch), b=view(src, pos * wide + 3 + ch + ra + rg, wide), a=view(sa, pos * H * d, H * d),
                                                       z=view(sz, pos * H * vd, H * vd), dst=view(dst, pos * H * vd, H * vd), **common)))
            got[pos : pos + t] = get(dst, (T, H * vd))[pos : pos + t]
        pos += t
    # a read-out near zero is divided by its own size: the norm's eps is what bounds that
    close(got, want, 2e-3 if vd == 1 else 2e-4)
    assert np.sqrt(np.mean((got - want) ** 2)) <= 2e-5 * np.sqrt(np.mean(want ** 2))


def test_delta_rule_takes_bf16_matrices_and_leaves_bf16_rows(gpu):
    H, d, vd, ra, T, eps = 2, 64, 64, 16, 70, 1e-5
    act, b, a, z = rand(1, T, 3 * H * d), rand(2, T, H), rand(3, T, H * d), rand(4, T, H * vd)
    w = {"a_log": rand(5, H), "dt_bias": rand(6, H * d), "norm": rand(7, vd) + 1}
    q, k, v = (act[:, i * H * d : (i + 1) * H * d].reshape(T, H, d) for i in range(3))
    log_g = -np.exp(w["a_log"])[:, None] * ph.softplus(a + w["dt_bias"]).reshape(T, H, d)
    want = ph.rms(pt.delta_scan(pt.unit(q) * d ** -0.5, pt.unit(k), v, log_g, pt.sigmoid(b)), eps) * w["norm"] * pt.sigmoid(z.reshape(T, H, vd))
    s = {n: gpu.up(x) for n, x in {**w, "act": act, "b": b, "a": a, "z": z}.items()}
    S, dst = gpu.out(H * d * vd), gpu.out(T * H * vd, bf16=True)
    gpu.call("ughip_delta_rows", C.byref(Delta(t=T, heads=H, kv_heads=H, dim=d, vdim=vd, a_log=s["a_log"].raw(), dt_bias=s["dt_bias"].raw(), norm=s["norm"].raw(), s=S.raw(), eps=eps,
                                               qkv=view(s["act"], 0, 3 * H * d), b=view(s["b"], 0, H), a=view(s["a"], 0, H * d), z=view(s["z"], 0, H * vd), dst=view(dst, 0, H * vd))))
    close(get(dst, want.shape), want, 2e-4, rel=2.0 ** -8)
    w_a, w_z, row = rand(8, H * d, ra, std=0.25), rand(9, H * vd, ra, std=0.25), rand(10, 3 * H * d + 2 * ra + H)
    outs = []
    for bf16 in (False, True):
        sa, sz, sr, taps, ring, out = gpu.up(w_a, bf16=bf16), gpu.up(w_z, bf16=bf16), gpu.up(row), gpu.up(np.ones(3 * H * d)), gpu.out(3 * H * d), gpu.out(2 * H * vd)
        S = gpu.out(H * d * vd)
        gpu.call("ughip_delta_step", C.byref(Delta(t=1, pos=0, heads=H, kv_heads=H, dim=d, vdim=vd, a_log=s["a_log"].raw(), dt_bias=s["dt_bias"].raw(), s=S.raw(), eps=eps, p=sr.raw(),
                                                   a_offset=3 * H * d, z_offset=3 * H * d + ra, b_offset=3 * H * d + 2 * ra, a_rank=ra, z_rank=ra, n_taps=1, taps=taps.raw(), w_a=sa.raw(),
                                                   w_z=sz.raw(), ring=ring.raw(), out=out.raw())))
        outs.append(get(out, 2 * H * vd))
    close(outs[1], outs[0], 1e-6)


def test_entry_points_check_their_buffers(gpu):
    """What would run past a buffer is an error with a message, not a launch."""
    s = gpu.out(64)

    def refused(name, *args):
        fn = getattr(gpu.lib, name)
        fn.restype = C.c_int
        assert fn(C.c_void_p(gpu.dev.raw_hip()), *args) != 0 and gpu.lib.ughip_last_error()

    small = dict(qkv=view(s, 0, 12), dst=view(s, 0, 4), k_cache=s.raw(), v_cache=s.raw(), capacity=8, t=1, pos=0, heads=1, kv_heads=1, dim=4, vdim=4, scale=1.0)
    refused("ughip_grouped_attention", C.byref(Attention(**small)))                                    # caches of whole tiles are larger
    kc, vc = caches_for(gpu, 1, 4, 4, 8, False)
    ok = {**small, "k_cache": kc.raw(), "v_cache": vc.raw()}
    gpu.call("ughip_grouped_attention", C.byref(Attention(**ok)))
    for bad in ({"pos": 8}, {"t": 9}, {"heads": 3, "kv_heads": 2}, {"rot": 4}, {"rot": 6, "cos": s.raw(), "sin": s.raw(), "table_rows": 64}, {"dim": 300}, {"qkv": view(s, 60, 12)},
                {"q_factor": gpu.out(1).raw(), "pos": 3}, {"dst": view(s, 62, 4)}, {"kv_heads": 0}):
        refused("ughip_grouped_attention", C.byref(Attention(**{**ok, **bad})))
    one = gpu.out(1)
    delta = dict(t=1, pos=0, heads=1, kv_heads=1, dim=2, vdim=2, a_log=s.raw(), dt_bias=s.raw(), norm=s.raw(), s=s.raw(), qkv=view(s, 0, 6), b=view(s, 0, 1), a=view(s, 0, 2), z=view(s, 0, 2),
                 dst=view(gpu.out(2), 0, 2))
    for bad in ({"t": 99}, {"s": one.raw()}, {"dim": 257}, {"heads": 3, "kv_heads": 2}, {"dt_bias": one.raw()}, {"norm": one.raw()}, {"z": view(one, 0, 2)}):
        refused("ughip_delta_rows", C.byref(Delta(**{**delta, **bad})))
    step = dict(t=1, pos=0, heads=1, kv_heads=1, dim=2, vdim=2, a_log=s.raw(), dt_bias=s.raw(), s=s.raw(), p=s.raw(), a_rank=1, z_rank=1, n_taps=1, taps=s.raw(), w_a=s.raw(), w_z=s.raw(),
                ring=s.raw(), out=gpu.out(4).raw())
    for bad in ({"p": one.raw()}, {"ring": one.raw()}, {"w_z": one.raw()}, {"out": one.raw()}, {"n_taps": 0}, {"a_rank": 0}, {"out": s.raw()}):
        refused("ughip_delta_step", C.byref(Delta(**{**step, **bad})))


# ---- models ------------------------------------------------------------------------------------------------------------------
@pytest.fixture(scope="module")
def models(hip, tmp_path_factory):
    made = {}

    def load(name, bf16):
        if (name, bf16) not in made:
            cfg = tm.MODELS[name]
            w = tm.weights(cfg, tm.RANKS[name], 7)
            folder = tm.write(tmp_path_factory.mktemp("model"), cfg, w)
            made[name, bf16] = (cfg, w, ug_amd.Decoder.load(hip, folder, bf16=bf16), folder)
        return made[name, bf16]

    return load


@pytest.fixture
def used_memory(hip):
    """Fresh buffers hold what was there before (numbers of other sequences), as in serving."""
    hip.set_zero_fill(False)
    yield
    hip.set_zero_fill(True)


def run(model, tokens, cuts, state=None):
    state = state or model.new_state(len(tokens))
    out, at = [], 0
    for c in cuts:
        out.append(model.step(state, tokens[at : at + c], range(c)))
        at += c
    assert at == len(tokens) == len(state)
    return np.concatenate(out).astype(np.float64)


def off(got, want):
    """Per position: root mean square of the difference (mean taken off) over the logits' own."""
    d = got - want
    d -= d.mean(-1, keepdims=True)
    w = want - want.mean(-1, keepdims=True)
    return np.sqrt((d ** 2).mean(-1)) / np.sqrt((w ** 2).mean())


LIMIT = {False: 3e-4, True: 0.06}


@pytest.mark.parametrize("name", ["odd", "even", "ones"])
@pytest.mark.parametrize("bf16", [False, True])
def test_model_prompts_portions_and_single_tokens(models, used_memory, name, bf16):
    cfg, w, model, _ = models(name, bf16)
    n = 170
    tokens = rng.token_ids(11, n, cfg["vocab"])
    want = pt.forward(cfg, w, tokens)
    for cuts in ([n], [1] * n, [2] * (n // 2), [3, 2, 64, 1, 1, 33, 66], [100, 1, 2, 67], [128, 42], [130, 16, 17, 7], [169, 1]):
        got = run(model, tokens, cuts)
        assert np.all(np.isfinite(got)), cuts
        assert off(got, want).max() <= LIMIT[bf16], (cuts[:6], int(off(got, want).argmax()), off(got, want).max())


@pytest.mark.parametrize("name", ["odd", "even"])
@pytest.mark.parametrize("bf16", [False, True])
def test_model_residual_behind_every_layer_run(models, name, bf16):
    cfg, w, model, _ = models(name, bf16)
    tokens, layers = rng.token_ids(5, 160, cfg["vocab"]), []
    pt.forward(cfg, w, tokens, layers)
    assert len(layers) == len(pt.layer_runs(cfg)) > len(cfg["layers"])
    for cuts in ([160], [159, 1], [40, 20, 100]):
        st, at, got = model.new_state(160), 0, []
        for c in cuts:
            got.append(model.step(st, tokens[at : at + c], [c - 1], hidden=(len(layers), cfg["width"]))[1])
            at += c
        got = np.concatenate(got, axis=1)
        for i, want in enumerate(layers):
            close(got[i], want, 0.3 if bf16 else 5e-4)


def test_model_sequences_side_by_side_and_one_after_the_other(models, used_memory):
    """Sequences of different lengths advance in turn, end, and leave their memory to others."""
    cfg, w, model, _ = models("odd", False)
    seqs = [rng.token_ids(20 + i, n, cfg["vocab"]) for i, n in enumerate((90, 7, 41, 130))]
    want = [pt.forward(cfg, w, s) for s in seqs]
    for _ in range(2):
        states, at, got = [model.new_state(len(s)) for s in seqs], [0] * 4, [[] for _ in seqs]
        step = 0
        while any(a < len(s) for a, s in zip(at, seqs)):
            for i, s in enumerate(seqs):
                c = min(len(s) - at[i], (1, 5, 2, 31)[(step + i) % 4])
                if c:
                    got[i].append(model.step(states[i], s[at[i] : at[i] + c], range(c)))
                    at[i] += c
            step += 1
        for i in range(4):
            assert off(np.concatenate(got[i]).astype(np.float64), want[i]).max() <= LIMIT[False], i


def test_model_wanted_places_and_limits(models):
    cfg, w, model, _ = models("odd", False)
    tokens = rng.token_ids(3, 30, cfg["vocab"])
    st = model.new_state(30)
    full = run(model, tokens, [30])
    np.testing.assert_allclose(model.step(st, tokens[:20], [7, 0, 19]), full[[7, 0, 19]], rtol=1e-3, atol=2e-4)
    assert model.step(st, tokens[20:25], []).shape == (0, cfg["vocab"]) and len(st) == 25
    np.testing.assert_allclose(model.step(st, tokens[25:], [4]), full[[29]], rtol=1e-3, atol=2e-4)
    with pytest.raises(ug_amd.UgError, match="capacity of 30"):
        model.step(st, [1], [0])


@pytest.mark.parametrize("name", ["odd", "even"])
@pytest.mark.parametrize("bf16", [False, True])
def test_greedy_generation(models, used_memory, tune, name, bf16):
    """The framework's own loops (queued, and with the logits read back), decode steps folded or not: the ids of the plain statement
    wherever its margin is no close call."""
    cfg, w, model, _ = models(name, bf16)
    prompt, steps = rng.token_ids(31, 37, cfg["vocab"]), 60
    ids, st = model.generate(prompt, steps)
    logits = pt.forward(cfg, w, np.concatenate([prompt, ids[:-1]]))[len(prompt) - 1 :]
    top = np.sort(logits, axis=-1)
    clear = top[:, -1] - top[:, -2] > 2 * LIMIT[bf16] * logits.std()
    assert clear.mean() > 0.3
    assert np.array_equal(ids[clear], logits.argmax(-1)[clear])
    np.testing.assert_allclose(st["top1"], top[:, -1], atol=4 * LIMIT[bf16] * logits.std())
    few = st["decode_items"]
    for switch in ("UG_LLAMA_HOST_ARGMAX", "UG_LLAMA_NO_FUSED_STEP"):
        tune.setenv(switch, "1")
        again, st = model.generate(prompt, steps, forced=ids[:-1])
        assert np.array_equal(again[clear], ids[clear])
    assert few < st["decode_items"]


def test_long_decoding(models, used_memory):
    cfg, w, model, _ = models("odd", False)
    tokens = rng.token_ids(77, 420, cfg["vocab"])
    got = run(model, tokens, [4] + [1] * 416)
    assert off(got, pt.forward(cfg, w, tokens)).max() <= LIMIT[False]


def test_a_key_at_the_edge_of_the_window(hip, used_memory, tmp_path):
    """A model whose second layer looks for one token: as long as it lies in the window its value is the output, one position later it is
    not; and the layer without a window finds it from anywhere."""
    size = 50
    for kind in ("window", "full"):
        mixer = tm.window(1, 1, 16, 16, size, 0, scale=1.0) if kind == "window" else tm.full(1, 1, 16, 16, 0.0, 8, scale=1.0)
        cfg = tm.config(16, 20, [mixer], 1.0)
        w = {n: np.zeros(s) for n, s in tm.shapes(cfg, {}).items()}
        w["embed"][:, 0], w["embed"][7, 0], w["embed"][7, 1] = 4.0, 0.5, 4.0       # token 7 is the one
        for n in ("l0.norm1", "l0.norm1b", "final.norm"):
            w[n][:] = 1.0
        w["l0.mix.q"][0, 0], w["l0.mix.q"][0, 1] = 4.0, 4.0
        w["l0.mix.k"][0, 1] = 4.0
        w["l0.mix.v"][:3, :2] = [[0, 1], [1, 0], [0.5, 0.5]]
        w["l0.mix.o"][:] = np.eye(16)
        w["head"][:, :16] = rng.bf16_round(rng.normal(3, 20 * 16)).reshape(20, 16)
        folder = tm.write(tmp_path / kind, cfg, w)
        tokens = np.ones(130, np.int64)
        tokens[40] = 7
        want = pt.forward(cfg, w, tokens)
        seen = off(want[40 + size - 1 : 40 + size], want[40 + size : 40 + size + 1])[0]
        assert seen > 0.3 if kind == "window" else seen < 1e-6
        for bf16 in (False, True):
            model = ug_amd.Decoder.load(hip, folder, bf16=bf16)
            for cuts in ([130], [60] + [1] * 70, [41, 2, 40, 17, 30], [88, 2, 2, 38]):
                assert off(run(model, tokens, cuts), want).max() <= (0.02 if bf16 else 1e-4), (kind, cuts[:4])


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_trace_runner(models, tmp_path, dtype):
    """bin/trace_run: steps on standard input, logits of the wanted places in files, an answer per step."""
    cfg, w, _, folder = models("odd", dtype == "bfloat16")
    a, b = rng.token_ids(1, 25, cfg["vocab"]).tolist(), rng.token_ids(2, 9, cfg["vocab"]).tolist()
    steps = [([("a", a[:20], [0, 19])], []), ([("b", b, [])], []), ([("a", a[20:21], [0]), ("c", b[:3], [2, 0])], []), ([("a", a[21:], [3])], ["a", "b"]), ([("a", b[:5], [4])], ["a", "c"])]
    lines = ["{\"step\": %d, \"entries\": [%s], \"end\": %s}" % (i, ", ".join('{"id": "%s", "tokens": %s, "want": %s}' % e for e in entries), str(end).replace("'", '"'))
             for i, (entries, end) in enumerate(steps)]
    r = subprocess.run([sys.executable, os.path.join(ROOT, "bin", "trace_run"), "--model", folder, "--dtype", dtype, "--out", str(tmp_path), "--max-tokens", "25"],
                       input="\n".join(lines) + "\n", capture_output=True, text=True, timeout=100)
    assert r.returncode == 0, r.stderr
    assert [l for l in r.stdout.splitlines() if l.startswith("done")] == [f"done {i}" for i in range(5)]
    la, lb = pt.forward(cfg, w, a), pt.forward(cfg, w, b)
    for i, want in ((0, la[[0, 19]]), (2, np.concatenate([la[[20]], lb[[2, 0]]])), (3, la[[24]]), (4, lb[[4]])):
        got = np.fromfile(tmp_path / f"{i}.f32", "<f4").reshape(want.shape).astype(np.float64)
        assert off(got, want).max() <= LIMIT[dtype == "bfloat16"]


def test_generate_program_prints_ids(models):
    cfg, _, model, folder = models("odd", True)
    r = subprocess.run([sys.executable, os.path.join(ROOT, "bin", "generate"), "--model", folder, "--prompt", "5,9,2", "--steps", "6"], capture_output=True, text=True, timeout=100)
    assert r.returncode == 0, r.stderr
    assert [int(i) for i in r.stdout.split(",")] == model.generate([5, 9, 2], 6)[0].tolist()
