"""Tanolorn on the GPU against tests/plain_hybrid.py: every mechanism through its C entry points, then whole models through the
decoder -- prompts, portions, single tokens, memory that is used again, greedy generation."""
import ctypes as C
import os
import subprocess
import sys

import numpy as np
import pytest

import hybrid_models as hm
import plain_hybrid as ph
import ug_amd
from gpu_calls import BF16, F32, GELU_MUL, NONE, SWIGLU, Gpu, Product, RowStep, View, Z, close, get, p, rand, view
from ug_amd import rng

pytestmark = pytest.mark.gpu

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
@pytest.fixture
def gpu(hip):
    return Gpu(hip)


def product(gpu, x, w, n, k, mode, act=NONE, bias=None, out_bf16=False, x_bf16=False, table=None, ids=None, col=0, row_index=None, group_end=None, groups=0, m=None):
    m = m or len(x)
    pad = 8                                   # rows apart from each other, results inside a wider buffer
    xs = np.concatenate([x, np.full((len(x), pad), np.nan)], axis=1)
    dx, dw = gpu.up(xs, bf16=x_bf16), gpu.up(w, bf16=mode == BF16)
    dst = gpu.out(m * (n + pad) + 16, bf16=out_bf16)
    keep = [gpu.up(bias) if bias is not None else None, gpu.up(table, bf16=mode == BF16) if table is not None else None, gpu.up(ids) if ids is not None else None,
            gpu.up(row_index) if row_index is not None else None, gpu.up(group_end) if group_end is not None else None]
    raw = [s.raw() if s is not None else None for s in keep]
    q = Product(view(dx, 0, k + pad), view(dst, 16, n + pad), dw.raw(), raw[0], 0, m, n, k, mode, act, raw[1], raw[2], len(table) if table is not None else 0,
                table.shape[1] if table is not None else 0, col, raw[3], raw[4], groups, len(x))
    gpu.call("ughip_product_rows", C.byref(q))
    out = dst.to_vec()
    out = (rng.from_bf16_bits(out) if out_bf16 else out)[16:].reshape(m, n + pad).astype(np.float64)
    assert np.all(np.isnan(out[:, n:])), "wrote between the rows"
    return out[:, :n]


def acted(y, act, w, n, bias, table, ids, col):
    if act == SWIGLU:
        b = bias if bias is not None else np.zeros(2 * n)
        return ph.silu(y[:, :n] + b[:n]) * (y[:, n:] + b[n:])
    y = y + (bias if bias is not None else 0.0)
    return ph.gelu_tanh(y) * table[ids][:, col : col + n] if act == GELU_MUL else y


# (m, n, k): sizes nothing divides, single rows and columns, whole tiles, the one-wave-per-SIMD kernel's (k % 64 == 0, k >= 256)
@pytest.mark.parametrize("m, n, k", [(1, 1, 1), (3, 5, 7), (70, 66, 130), (130, 9, 33), (2, 300, 96), (200, 264, 320), (97, 1032, 256)])
@pytest.mark.parametrize("mode", [F32, BF16])
@pytest.mark.parametrize("act", [NONE, SWIGLU, GELU_MUL])
def test_products_of_rows(gpu, m, n, k, mode, act):
    rows = 2 * n if act == SWIGLU else n
    x, w, bias = rand(1, m, k), rand(2, rows, k, std=k ** -0.5), rand(3, rows, std=0.5)
    table, ids, col = rand(4, 13, n + 6), np.arange(m) * 5 % 13, 4
    kw = dict(table=table, ids=ids, col=col) if act == GELU_MUL else {}
    want = acted(x @ w.T, act, w, n, bias, table, ids, col)
    for x_bf16, out_bf16 in ((False, False), (True, True)) if mode == BF16 else ((False, False),):
        got = product(gpu, x, w, n, k, mode, act, bias, x_bf16=x_bf16, out_bf16=out_bf16, **kw)
        close(got, want, 2e-5, rel=2.0 ** -8 if out_bf16 else 0.0)
        if mode == BF16 and x_bf16 and k == 320 and act != GELU_MUL:
            assert "gemm_dma4" in ug_amd.last_kernel() and "rows" in ug_amd.last_kernel()
    assert np.all(np.isfinite(got))


@pytest.mark.parametrize("m, n, k, experts, top", [(1, 8, 16, 5, 3), (50, 40, 72, 7, 2), (150, 136, 320, 6, 2), (400, 72, 256, 3, 2)])
@pytest.mark.parametrize("mode", [F32, BF16])
@pytest.mark.parametrize("act", [NONE, SWIGLU])
def test_products_of_rows_sorted_by_expert(gpu, m, n, k, experts, top, mode, act):
    rows = 2 * n if act == SWIGLU else n
    x, w = rand(1, m, k), rand(2, experts, rows, k, std=k ** -0.5)
    # expert 1 is nobody's choice, expert 0 everybody's first
    ids = np.stack([np.zeros(m, int)] + [2 + (np.arange(m) * (j + 1)) % (experts - 2) for j in range(top - 1)], axis=1)
    d_ids, ri, sl, ge = gpu.up(ids), gpu.ints(m * top), gpu.ints(m * top), gpu.ints(experts)
    gpu.call("ughip_group_rows", p(d_ids), Z(m), Z(top), Z(experts), p(ri), p(sl), p(ge))
    ri, sl, ge = ri.to_vec(), sl.to_vec().reshape(m, top), ge.to_vec()
    order = np.argsort(ids.ravel(), kind="stable")
    assert np.array_equal(ri, order // top) and np.array_equal(sl.ravel()[order], np.arange(m * top))
    assert np.array_equal(ge, np.cumsum(np.bincount(ids.ravel(), minlength=experts)))
    got = product(gpu, x, w, n, k, mode, act, row_index=ri, group_end=ge, groups=experts, m=m * top, x_bf16=mode == BF16)
    want = acted(np.stack([w[e] @ x[r] for r in range(m) for e in ids[r]]), act, w, n, None, None, None, 0)
    close(got[sl.ravel()], want, 2e-5)


@pytest.mark.parametrize("experts, groups, keep, top", [(1, 1, 1, 1), (6, 3, 2, 2), (8, 4, 3, 3), (9, 9, 4, 4), (64, 8, 3, 6), (96, 4, 2, 7), (130, 13, 5, 5)])
def test_routing(gpu, experts, groups, keep, top):
    m, k = 37, 75
    x, w, corr = rand(1, m, k), rand(2, experts, k, std=2 * k ** -0.5), rand(3, experts, std=0.4) - 0.7       # many choice scores below zero
    ids, wts = gpu.ints(m * top), gpu.out(m * top)
    sx, sw, sc = gpu.up(x), gpu.up(w), gpu.up(corr)
    gpu.call("ughip_route_rows", view(sx, 0, k), p(sw), p(sc), Z(m), Z(k), Z(experts), Z(groups), Z(keep), Z(top), p(ids), p(wts))
    ids, wts = ids.to_vec().reshape(m, top), get(wts, (m, top))
    rc = {"experts": experts, "top": top, "groups": {"count": groups, "keep": keep}}
    for i in range(m):
        chosen, weight = ph.route(x[i], {"router": w, "correction": corr}, rc)
        assert ids[i].tolist() == chosen.tolist(), i
        np.testing.assert_allclose(wts[i], weight, rtol=2e-5)
    # the one-row form makes the same choice from given logits
    logits = gpu.up(np.concatenate([[9.0, 9.0], w @ x[5]]))
    n, kk = 3, 8
    row, mats, one_ids, one_w, dst = gpu.up(rand(4, kk)), rand(5, experts, 2 * n, kk), gpu.ints(top), gpu.out(top), gpu.out(top * n)
    dm = gpu.up(mats)
    q = RowStep(x=row.raw(), w=dm.raw(), n=n, k=kk, act=SWIGLU, route=1, logits=logits.raw(), logits_offset=2, correction=sc.raw(), experts=experts, groups=groups, keep=keep,
                top=top, route_ids=one_ids.raw(), route_weights=one_w.raw(), dst=dst.raw())
    gpu.call("ughip_product_row", C.byref(q))
    assert one_ids.to_vec().tolist() == ids[5].tolist()
    y = np.stack([mats[e] @ rand(4, kk) for e in ids[5]])
    close(get(dst, (top, n)), ph.silu(y[:, :n]) * y[:, n:], 2e-5)
    down = rand(6, experts, 5, n)
    dd, out = gpu.up(down), gpu.out(5)
    q = RowStep(x=dst.raw(), w=dd.raw(), n=5, k=n, route=2, experts=experts, groups=groups, keep=keep, top=top, route_ids=one_ids.raw(), route_weights=one_w.raw(), dst=out.raw())
    gpu.call("ughip_product_row", C.byref(q))
    a = get(dst, (top, n))
    close(get(out, 5), sum(wts[5][j] * (down[ids[5][j]] @ a[j]) for j in range(top)), 3e-5)


@pytest.mark.parametrize("k, n, groups", [(1, 1, 1), (90, 33, 3), (256, 40, 1), (1024, 70, 4), (2048, 8200, 8), (4096, 2050, 2), (5632, 37, 1), (9001, 5, 1)])
@pytest.mark.parametrize("bf16", [False, True])
def test_one_row_with_its_neighbours(gpu, k, n, groups, bf16):
    eps = 1e-3
    x, y, yn, gate, norm, w, bias = rand(1, k), rand(2, k), rand(3, k) + 1, rand(4, k), rand(5, k) + 1, rand(6, n, k, std=k ** -0.5), rand(7, n)
    dw, db, dyn, dn = gpu.up(w, bf16=bf16), gpu.up(bias), gpu.up(yn), gpu.up(norm)
    buf = gpu.up(np.concatenate([np.zeros(4), x, y, gate]))
    # residual + norm of what joins it, kept in front of the result
    dst = gpu.out(k + n)
    q = RowStep(x=buf.raw(), x_offset=4, y=buf.raw(), y_offset=4 + k, y_norm=dyn.raw(), eps=eps, keep_x=1, w=dw.raw(), bias=db.raw(), n=n, k=k, dst=dst.raw(), dst_offset=k)
    gpu.call("ughip_product_row", C.byref(q))
    joined = x + ph.rms(y, eps) * yn
    close(get(dst, k + n)[:k], joined, 3e-6)
    close(get(dst, k + n)[k:], w @ joined + bias, 3e-5)
    # gate, then a norm over parts of the row
    out = gpu.out(n)
    q = RowStep(x=buf.raw(), x_offset=4, gate=buf.raw(), gate_offset=4 + 2 * k, norm=dn.raw(), norm_groups=groups, eps=eps, w=dw.raw(), n=n, k=k, dst=out.raw())
    gpu.call("ughip_product_row", C.byref(q))
    g = x * ph.silu(gate)
    close(get(out, n), w @ (ph.rms(g.reshape(groups, -1), eps).reshape(-1) * norm), 3e-5)
    # both norms (the head), and the row as it is
    q = RowStep(x=buf.raw(), x_offset=4, y=buf.raw(), y_offset=4 + k, y_norm=dyn.raw(), norm=dn.raw(), eps=eps, w=dw.raw(), n=n, k=k, dst=out.raw())
    gpu.call("ughip_product_row", C.byref(q))
    close(get(out, n), w @ (ph.rms(joined, eps) * norm), 3e-5)
    table, ids = rand(8, 4, n + 3), gpu.up(np.array([2]))
    dt = gpu.up(table, bf16=bf16)
    q = RowStep(x=buf.raw(), x_offset=4, w=dw.raw(), n=n, k=k, dst=out.raw(), act=GELU_MUL, table=dt.raw(), ids=ids.raw(), table_rows=4, table_stride=n + 3, table_col=1)
    gpu.call("ughip_product_row", C.byref(q))
    close(get(out, n), ph.gelu_tanh(w @ x) * table[2, 1 : n + 1], 3e-5)


def test_norms_of_rows(gpu):
    m, n, eps = 9, 130, 2e-3
    x, y, w = rand(1, m, n), rand(2, m * 3, n), rand(3, n)
    sx, sy, sw, dst, half = gpu.up(x), gpu.up(y), gpu.up(w), gpu.out(m * n), gpu.out(m * n, bf16=True)
    none = View(None, 0, 0)
    gpu.call("ughip_add_rms_norm_rows", view(sx, 0, n), view(sy, n, 2 * n), None, None, Z(0), Z(0), p(sw), C.c_float(eps), none, view(dst, 0, n), None, p(half), Z(m), Z(n))
    want = x + ph.rms(y.reshape(-1)[n:][: (2 * m - 1) * n].reshape(-1, n)[::2], eps) * w
    close(get(dst, (m, n)), want, 3e-6)
    close(get(half, (m, n)), want, 3e-6, rel=2.0 ** -8)
    slots, weights = np.stack([np.arange(m) * 3 % 27, np.arange(m) + 11], axis=1), rand(4, m, 2)
    ss, sw2 = gpu.up(slots), gpu.up(weights)
    gpu.call("ughip_add_rms_norm_rows", none, view(sy, 0, n), p(ss), p(sw2), Z(2), Z(m * 3), p(sw), C.c_float(eps), none, view(dst, 0, n), None, None, Z(m), Z(n))
    close(get(dst, (m, n)), ph.rms((weights[:, :, None] * y[slots]).sum(1), eps) * w, 3e-6)
    for parts, cols in ((1, n), (5, n), (2, 128)):
        z = rand(5, m, cols)
        sz, sg = gpu.up(z), gpu.out(m * cols)
        gpu.call("ughip_gated_rms_norm_rows", view(sy, 0, n), view(sz, 0, cols), p(sw), C.c_float(eps), Z(parts), view(sg, 0, cols), Z(m), Z(cols))
        close(get(sg, (m, cols)), ph.grouped_gated_norm(y[:m, :cols], z, w[:cols], parts, eps), 1e-5)
    table, ids = rand(6, 11, 40), np.array([3, 10, 0, 3])
    st, si, out = gpu.up(table, bf16=True), gpu.up(ids), gpu.out(4 * 7)
    gpu.call("ughip_gather_rows", p(st), Z(11), Z(40), Z(33), Z(7), p(si), Z(4), view(out, 0, 7))
    assert np.array_equal(get(out, (4, 7)), table[ids, 33:])


# (heads, dim, rot, vdim, rank): odd, whole pieces, the sizes of the kernels' variants
LATENT = [(1, 1, 2, 1, 1), (3, 18, 14, 27, 41), (5, 64, 32, 48, 128), (2, 128, 64, 96, 320), (1, 192, 64, 200, 512), (17, 8, 8, 16, 24)]


@pytest.mark.parametrize("heads, dim, rot, vdim, rank", LATENT)
@pytest.mark.parametrize("pos, t", [(0, 1), (0, 150), (61, 3), (130, 130), (256, 1), (255, 2), (700, 1)])
@pytest.mark.parametrize("bf16", [False, True])
def test_latent_attention_both_ways(gpu, heads, dim, rot, vdim, rank, pos, t, bf16):
    """Keys expanded and keys absorbed agree with the plain statement, for cuts anywhere; one far key of every query stands out (its
    score is some 8 above the rest), so that a lost, shifted or unrotated key shows."""
    s, eps, L, mc = pos + t, 1e-4, rank + rot, {"heads": heads, "dim": dim, "rot_dim": rot, "vdim": vdim, "kv_rank": rank, "scale": 0.37 / np.sqrt(dim + rot),
                                                "rot": {"base": 300.0, "dims": rot}}
    w = {"uk": rand(1, heads * dim, rank, std=rank ** -0.5), "uv": rand(2, heads * vdim, rank, std=rank ** -0.5), "dkv.norm": rand(3, rank) * 0.2 + 1}
    kv, q = rand(4, s, L), rand(5, t, heads * (dim + rot))
    c = ph.rms(kv[:, :rank], eps) * w["dkv.norm"]
    k_rot = ph.rotate_half(kv[:, None, rank:], np.arange(s), 300.0, rot)[:, 0]
    k = (c @ w["uk"].T).reshape(s, heads, dim)
    # far keys: the first, the last, and ones at the borders of tiles of 32 and 64
    for i in range(t):
        far = [0, pos + i, 31, 32, 63, 64, 127, 128][(i + heads) % 8]
        far = min(far, pos + i)
        for h in range(heads):
            qh = q[i].reshape(heads, dim + rot)[h]
            target = np.concatenate([k[far, h], ph.rotate_half(k_rot[far][None, None], [-(pos + i)], 300.0, rot)[0, 0]])
            target *= 8.0 / (mc["scale"] * (target @ target))
            qh[:] = rng.bf16_round((0.3 * qh + target).astype(np.float32))
    q_rot = ph.rotate_half(q.reshape(t, heads, -1)[..., dim:], pos + np.arange(t), 300.0, rot)
    v = (c @ w["uv"].T).reshape(s, heads, vdim)
    want = np.zeros((t, heads, vdim))
    for i in range(t):
        for h in range(heads):
            sc = (k[: pos + i + 1, h] @ q[i].reshape(heads, -1)[h, :dim] + k_rot[: pos + i + 1] @ q_rot[i, h]) * mc["scale"]
            e = np.exp(sc - sc.max())
            want[i, h] = (e / e.sum()) @ v[: pos + i + 1, h]
    want = want.reshape(t, -1)

    cap, cs = s + 3, np.arange(s + 5)[:, None] * 300.0 ** (-2.0 * np.arange(rot // 2) / rot)
    cos, sin, rows = gpu.up(np.cos(cs)), gpu.up(np.sin(cs)), len(cs)
    cache = gpu.out(cap * L)
    skv, sq, sn, uk, uv = gpu.up(kv), gpu.up(q), gpu.up(w["dkv.norm"]), gpu.up(w["uk"], bf16=bf16), gpu.up(w["uv"], bf16=bf16)
    wide = heads * (dim + rot)
    gpu.call("ughip_latent_append", view(skv, 0, L), p(sn), C.c_float(eps), p(cos), p(sin), Z(rows), p(cache), Z(cap), Z(0), Z(pos), Z(rank), Z(rot))
    dst = gpu.out(t * heads * vdim)
    # the step's own rows come in on the way
    gpu.call("ughip_latent_attention_absorbed", view(sq, 0, wide), view(skv, pos * L, L), p(sn), C.c_float(eps), p(uk), p(uv), p(cache), Z(cap), p(cos), p(sin), Z(rows),
             view(dst, 0, heads * vdim), Z(t), Z(pos), Z(heads), Z(dim), Z(rot), Z(vdim), Z(rank), C.c_float(mc["scale"]))
    close(get(dst, want.shape), want, 1e-4)
    close(get(cache, (cap, L))[:s], np.concatenate([c, k_rot], axis=1), 3e-6)
    assert np.all(np.isnan(get(cache, (cap, L))[s:]))
    keys, v_stride = gpu.out(s * heads * dim, bf16=bf16), (s + 63) // 64 * 64
    vt = gpu.out(heads * vdim * v_stride, bf16=bf16)
    gpu.call("ughip_product_rows", C.byref(Product(view(cache, 0, L), view(keys, 0, heads * dim), uk.raw(), None, 0, s, heads * dim, rank, BF16 if bf16 else F32, NONE)))
    gpu.call("ughip_product_rows", C.byref(Product(view(uv, 0, rank), view(vt, 0, v_stride), cache.raw(), None, L, heads * vdim, s, rank, BF16 if bf16 else F32, NONE)))
    dst = gpu.out(t * heads * vdim)
    gpu.call("ughip_latent_attention_rows", view(sq, 0, wide), p(keys), p(vt), Z(v_stride), p(cache), p(cos), p(sin), Z(rows), view(dst, 0, heads * vdim), Z(t), Z(pos),
             Z(heads), Z(dim), Z(rot), Z(vdim), Z(rank), C.c_float(mc["scale"]))
    close(get(dst, want.shape), want, 0.12 if bf16 else 1e-4)


@pytest.mark.parametrize("heads, vdim, groups, state, taps", [(1, 1, 1, 1, 1), (6, 21, 3, 19, 3), (4, 64, 2, 128, 4), (2, 70, 1, 40, 4), (3, 16, 3, 200, 2), (8, 4, 4, 8, 5)])
@pytest.mark.parametrize("cuts", [(1, 1, 1, 1, 1, 1), (150,), (64, 64), (65, 2, 3, 1, 63), (2, 2, 5), (17, 1, 130)])
def test_state_space_rows_and_steps(gpu, heads, vdim, groups, state, taps, cuts):
    """Any cut of a sequence gives the plain recurrence: chunks, single steps, the taps' ring -- from memory that held something else."""
    T, inner, gn = sum(cuts), heads * vdim, groups * state
    ch, wide = inner + 2 * gn, inner + 2 * gn + heads + 5
    row = rand(1, T, wide)
    w = {"conv": rand(2, ch, taps), "conv.b": rand(3, ch), "dt_bias": rand(4, heads) - 1, "A_log": rand(5, heads), "D": rand(6, heads)}
    row[:, 5 + ch :] = 0.5 * row[:, 5 + ch :]
    act = ph.silu(ph.causal_conv(row[:, 5 : 5 + ch], w["conv"], w["conv.b"]))
    want = ph.ssm_scan(act[:, :inner].reshape(T, heads, vdim), act[:, inner : inner + gn].reshape(T, groups, state), act[:, inner + gn :].reshape(T, groups, state),
                       ph.softplus(row[:, 5 + ch :] + w["dt_bias"]), w["A_log"], w["D"]).reshape(T, inner)
    s = {k: gpu.up(v) for k, v in w.items()}
    src, S, ring, xbc, dst = gpu.up(row), gpu.out(heads * state * vdim), gpu.out(taps * ch), gpu.out(T * ch), gpu.out(T * inner)
    pos = 0
    for t in cuts:
        if t == 1 and pos % 2 == 0:
            gpu.call("ughip_ssm_step", p(gpu_row(gpu, row[pos])), Z(5), Z(5 + ch), p(s["conv"]), p(s["conv.b"]), Z(taps), p(ring), p(s["dt_bias"]), p(s["A_log"]), p(s["D"]), p(S),
                     Z(pos), Z(heads), Z(vdim), Z(groups), Z(state), view(dst, pos * inner, inner))
        else:
            gpu.call("ughip_conv_silu_rows", view(src, pos * wide + 5, wide), p(s["conv"]), p(s["conv.b"]), Z(taps), p(ring), Z(pos), Z(t), Z(ch), view(xbc, pos * ch, ch))
            gpu.call("ughip_conv_ring_store", view(src, pos * wide + 5, wide), Z(taps), p(ring), Z(pos), Z(t), Z(ch))
            gpu.call("ughip_ssm_rows", view(xbc, pos * ch, ch), view(src, pos * wide + 5 + ch, wide), p(s["dt_bias"]), p(s["A_log"]), p(s["D"]), p(S), Z(pos), Z(t), Z(heads),
                     Z(vdim), Z(groups), Z(state), view(dst, pos * inner, inner))
        pos += t
    close(get(dst, (T, inner)), want, 5e-5)


def gpu_row(gpu, row):
    gpu.kept = gpu.up(row)      # alive until the next one
    return gpu.kept


def test_entry_points_check_their_buffers(gpu):
    """What would run past a buffer is an error with a message, not a launch."""
    s, ids = gpu.out(64), gpu.ints(4)

    def refused(name, *args):
        fn = getattr(gpu.lib, name)
        fn.restype = C.c_int
        assert fn(C.c_void_p(gpu.dev.raw_hip()), *args) != 0 and gpu.lib.ughip_last_error()

    w = gpu.up(rand(1, 8, 8))
    refused("ughip_product_rows", C.byref(Product(view(s, 0, 8), view(s, 0, 8), w.raw(), None, 0, 9, 8, 8, F32, NONE)))
    refused("ughip_product_rows", C.byref(Product(view(w, 0, 8), view(s, 0, 8), w.raw(), None, 0, 8, 9, 8, F32, NONE)))
    refused("ughip_product_row", C.byref(RowStep(x=s.raw(), w=w.raw(), n=8, k=16, dst=w.raw())))
    refused("ughip_ssm_rows", view(s, 0, 8), view(s, 0, 1), p(s), p(s), p(s), p(s), Z(0), Z(9), Z(1), Z(4), Z(1), Z(2), view(s, 0, 4))
    refused("ughip_latent_append", view(s, 0, 8), p(s), C.c_float(0), p(s), p(s), Z(4), p(s), Z(4), Z(3), Z(2), Z(6), Z(2))
    refused("ughip_route_rows", view(s, 0, 8), p(w), None, Z(4), Z(8), Z(8), Z(3), Z(1), Z(1), p(ids), p(s))
    refused("ughip_group_rows", p(ids), Z(4), Z(2), Z(4), p(ids), p(ids), p(ids))


# ---- models ------------------------------------------------------------------------------------------------------------------
@pytest.fixture(scope="module")
def models(hip, tmp_path_factory):
    made = {}

    def load(name, bf16):
        if (name, bf16) not in made:
            cfg = {"odd": hm.ODD, "even": hm.EVEN, "ones": hm.ONES}[name]
            w = hm.weights(cfg, 7, steady_routing=bf16)
            folder = hm.write(tmp_path_factory.mktemp("model"), cfg, w)
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


LIMIT = {False: 2e-4, True: 0.06}


@pytest.mark.parametrize("name", ["odd", "even", "ones"])
@pytest.mark.parametrize("bf16", [False, True])
def test_model_prompts_portions_and_single_tokens(models, used_memory, name, bf16):
    cfg, w, model, _ = models(name, bf16)
    n = 170
    tokens = rng.token_ids(11, n, cfg["vocab"])
    want = ph.forward(cfg, w, tokens)
    for cuts in ([n], [1] * n, [2] * (n // 2), [3, 2, 64, 1, 1, 33, 66], [100, 1, 2, 67], [128, 42], [169, 1]):
        got = run(model, tokens, cuts)
        assert np.all(np.isfinite(got)), cuts
        assert off(got, want).max() <= LIMIT[bf16], (cuts[:6], int(off(got, want).argmax()), off(got, want).max())


@pytest.mark.parametrize("bf16", [False, True])
def test_model_residual_behind_every_layer(models, bf16):
    cfg, w, model, _ = models("even", bf16)
    tokens, layers = rng.token_ids(5, 110, cfg["vocab"]), []
    ph.forward(cfg, w, tokens, layers)
    for cuts in ([110], [109, 1]):
        st, at, got = model.new_state(110), 0, []
        for c in cuts:
            got.append(model.step(st, tokens[at : at + c], [c - 1], hidden=(len(cfg["layers"]), cfg["width"]))[1])
            at += c
        got = np.concatenate(got, axis=1)
        for i, want in enumerate(layers):
            close(got[i], want, 2.0 * (0.12 if bf16 else 1e-4))


def test_model_sequences_side_by_side_and_one_after_the_other(models, used_memory):
    """Sequences of different lengths advance in turn, end, and leave their memory to others."""
    cfg, w, model, _ = models("odd", False)
    seqs = [rng.token_ids(20 + i, n, cfg["vocab"]) for i, n in enumerate((90, 7, 41, 130))]
    want = [ph.forward(cfg, w, s) for s in seqs]
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
    np.testing.assert_allclose(model.step(st, tokens[:20], [7, 0, 19]), full[[7, 0, 19]], rtol=1e-3, atol=1e-4)
    assert model.step(st, tokens[20:25], []).shape == (0, cfg["vocab"]) and len(st) == 25
    np.testing.assert_allclose(model.step(st, tokens[25:], [4]), full[[29]], rtol=1e-3, atol=1e-4)
    for bad in (lambda: model.step(st, [1], [0]), lambda: model.step(model.new_state(4), [cfg["vocab"]], [0]), lambda: model.step(model.new_state(4), [-1], [0]),
                lambda: model.step(model.new_state(4), [1, 2], [2]), lambda: model.step(model.new_state(4), [], [])):
        with pytest.raises(ug_amd.UgError):
            bad()


@pytest.mark.parametrize("name", ["odd", "even"])
@pytest.mark.parametrize("bf16", [False, True])
def test_greedy_generation(models, used_memory, tune, name, bf16):
    """The framework's own loops (queued, and with the logits read back), decode steps folded or not: the ids of the plain statement
    wherever its margin is no close call."""
    cfg, w, model, _ = models(name, bf16)
    prompt, steps = rng.token_ids(31, 37, cfg["vocab"]), 60
    ids, st = model.generate(prompt, steps)
    logits = ph.forward(cfg, w, np.concatenate([prompt, ids[:-1]]))[len(prompt) - 1 :]
    top = np.sort(logits, axis=-1)
    clear = top[:, -1] - top[:, -2] > 2 * LIMIT[bf16] * logits.std()
    assert clear.mean() > 0.3
    assert np.array_equal(ids[clear], logits.argmax(-1)[clear])
    np.testing.assert_allclose(st["top1"], top[:, -1], atol=4 * LIMIT[bf16] * logits.std())
    forced = model.generate(prompt, steps, forced=ids[:-1])[0]
    assert np.array_equal(forced, ids)
    few = st["decode_items"]
    for switch in ("UG_LLAMA_HOST_ARGMAX", "UG_LLAMA_NO_FUSED_STEP"):
        tune.setenv(switch, "1")
        again, st = model.generate(prompt, steps, forced=ids[:-1])
        assert np.array_equal(again[clear], ids[clear])
    assert few < st["decode_items"]
    if not bf16:
        assert np.array_equal(ids, model.generate(prompt, steps)[0][: steps + 1])


def test_long_decoding(models, used_memory):
    cfg, w, model, _ = models("odd", False)
    tokens = rng.token_ids(77, 420, cfg["vocab"])
    got = run(model, tokens, [4] + [1] * 416)
    assert off(got, ph.forward(cfg, w, tokens)).max() <= LIMIT[False]


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
    la, lb = ph.forward(cfg, w, a), ph.forward(cfg, w, b)
    for i, want in ((0, la[[0, 19]]), (2, np.concatenate([la[[20]], lb[[2, 0]]])), (3, la[[24]]), (4, lb[[4]])):
        got = np.fromfile(tmp_path / f"{i}.f32", "<f4").reshape(want.shape).astype(np.float64)
        assert off(got, want).max() <= LIMIT[dtype == "bfloat16"]
    assert not os.path.exists(tmp_path / "1.f32")


def test_generate_program_prints_ids(models):
    cfg, _, model, folder = models("odd", True)
    r = subprocess.run([sys.executable, os.path.join(ROOT, "bin", "generate"), "--model", folder, "--prompt", "5,9,2", "--steps", "6"], capture_output=True, text=True, timeout=100)
    assert r.returncode == 0, r.stderr
    assert [int(i) for i in r.stdout.split(",")] == model.generate([5, 9, 2], 6)[0].tolist()


def test_llama_by_configuration_is_the_llama_model(hip, hip_ops, tmp_path):
    """The registry's llama gives the ids of LlamaModel on the same weights, and its step function the same logits for any cut."""
    c = {"model_type": "llama", "hidden_size": 256, "intermediate_size": 320, "max_position_embeddings": 64, "num_attention_heads": 8, "num_key_value_heads": 4,
         "num_hidden_layers": 2, "rms_norm_eps": 1e-5, "vocab_size": 90}
    cfg = ug_amd.LlamaConfig(hidden_size=256, intermediate_size=320, max_position_embeddings=64, num_attention_heads=8, num_key_value_heads=4, num_hidden_layers=2, vocab_size=90)
    dec = ug_amd.Decoder.random(hip, c, bf16=False, seed=9, std=0.3)
    ref = ug_amd.LlamaModel(hip, hip_ops, cfg, custom_softmax=True, seed=9, std=0.3, fused_attention=3)
    prompt = rng.token_ids(4, 20, 90)
    assert np.array_equal(dec.generate(prompt, 12)[0], ref.generate(prompt, 12)[0])
    whole, parts = run(dec, prompt, [20]), run(dec, prompt, [7, 1, 12])
    assert off(parts, whole).max() < 1e-4
