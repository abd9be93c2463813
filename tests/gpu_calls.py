"""Calls into libughip.so on numpy arrays, for the tests of ughip_layers.h's entry points."""
import ctypes as C

import numpy as np

import ug_amd
from ug_amd import rng

F32, BF16 = 0, 2                       # UGHIP_PRODUCT_*
NONE, SWIGLU, GELU_MUL, GLU = 0, 1, 2, 3       # UGHIP_ACT_*
Z = C.c_size_t


class View(C.Structure):
    _fields_ = [("s", C.c_void_p), ("offset", Z), ("stride", Z)]


class Product(C.Structure):
    _fields_ = [("x", View), ("dst", View), ("w", C.c_void_p), ("bias", C.c_void_p), ("w_stride", Z), ("m", Z), ("n", Z), ("k", Z), ("product", C.c_int), ("act", C.c_int),
                ("table", C.c_void_p), ("ids", C.c_void_p), ("table_rows", Z), ("table_stride", Z), ("table_col", Z), ("row_index", C.c_void_p), ("group_end", C.c_void_p),
                ("groups", Z), ("x_rows", Z), ("act_alpha", C.c_float), ("act_shift", C.c_float), ("act_limit", C.c_float)]


class RowStep(C.Structure):
    _fields_ = [("x", C.c_void_p), ("x_offset", Z), ("y", C.c_void_p), ("y_norm", C.c_void_p), ("gate", C.c_void_p), ("norm", C.c_void_p), ("y_offset", Z), ("gate_offset", Z),
                ("norm_groups", Z), ("eps", C.c_float), ("act", C.c_int), ("route", C.c_int), ("keep_x", C.c_int), ("w", C.c_void_p), ("bias", C.c_void_p), ("n", Z), ("k", Z),
                ("table", C.c_void_p), ("ids", C.c_void_p), ("table_rows", Z), ("table_stride", Z), ("table_col", Z), ("logits", C.c_void_p), ("correction", C.c_void_p),
                ("logits_offset", Z), ("experts", Z), ("groups", Z), ("keep", Z), ("top", Z), ("route_ids", C.c_void_p), ("route_weights", C.c_void_p), ("dst", C.c_void_p),
                ("dst_offset", Z), ("x_out", Z), ("extra", C.c_void_p), ("extra_offset", Z), ("gate_after", C.c_int), ("act_alpha", C.c_float), ("act_shift", C.c_float),
                ("act_limit", C.c_float)]


class Attention(C.Structure):
    _fields_ = [("qkv", View), ("dst", View), ("k_cache", C.c_void_p), ("v_cache", C.c_void_p), ("cos", C.c_void_p), ("sin", C.c_void_p), ("q_factor", C.c_void_p), ("capacity", Z),
                ("table_rows", Z), ("rot", Z), ("window", Z), ("t", Z), ("pos", Z), ("heads", Z), ("kv_heads", Z), ("dim", Z), ("vdim", Z), ("scale", C.c_float)]


class Delta(C.Structure):
    _fields_ = [("t", Z), ("pos", Z), ("heads", Z), ("kv_heads", Z), ("dim", Z), ("vdim", Z), ("a_log", C.c_void_p), ("dt_bias", C.c_void_p), ("norm", C.c_void_p), ("s", C.c_void_p),
                ("eps", C.c_float), ("qkv", View), ("b", View), ("a", View), ("z", View), ("dst", View), ("p", C.c_void_p), ("qkv_offset", Z), ("b_offset", Z), ("a_offset", Z),
                ("z_offset", Z), ("a_rank", Z), ("z_rank", Z), ("n_taps", Z), ("dst_offset", Z), ("taps", C.c_void_p), ("w_a", C.c_void_p), ("w_z", C.c_void_p), ("ring", C.c_void_p),
                ("out", C.c_void_p)]


class Gpu:
    """Calls into libughip.so on slices of numpy arrays."""

    def __init__(self, dev):
        self.dev, self.lib = dev, ug_amd.ughip_lib()

    def up(self, a, bf16=False):
        a = np.ascontiguousarray(a)
        if a.dtype.kind == "i":
            return self.dev.slice_from(a.astype(np.int32).ravel())
        a = a.astype(np.float32).ravel()
        if bf16:
            s = self.dev.allocate_uninit(ug_amd.BF16, a.size)
            s.copy_host_to_device(rng.to_bf16_bits(a), ug_amd.BF16)
            return s
        return self.dev.slice_from(a)

    def out(self, n, bf16=False):
        s = self.dev.allocate_uninit(ug_amd.BF16 if bf16 else ug_amd.F32, n)
        s.copy_host_to_device(np.full(n, 0x7fc0, np.uint16) if bf16 else np.full(n, np.nan, np.float32), ug_amd.BF16 if bf16 else ug_amd.F32)
        return s

    def ints(self, n):
        return self.dev.slice_from(np.full(n, -7, np.int32))

    def call(self, name, *args):
        fn = getattr(self.lib, name)
        fn.restype = C.c_int
        assert fn(C.c_void_p(self.dev.raw_hip()), *args) == 0, self.lib.ughip_last_error().decode()


def p(s):
    return C.c_void_p(s.raw()) if s is not None else None


def view(s, offset, stride):
    return View(s.raw() if s is not None else None, offset, stride)


def get(s, shape):
    v = s.to_vec()
    return (rng.from_bf16_bits(v) if s.dtype == ug_amd.BF16 else v).reshape(shape).astype(np.float64)


def rand(seed, *shape, std=1.0):
    """bf16 values, so that both product modes see the same operands."""
    return rng.bf16_round(rng.normal(seed, int(np.prod(shape)), std)).reshape(shape).astype(np.float64)


def close(got, want, tol, rel=0.0):
    """Within tol times the root mean square of `want`, plus rel times the element (a result rounded to bf16)."""
    scale = np.sqrt(np.mean(want ** 2)) + 1e-30
    assert np.all(np.isfinite(got)), "not finite"
    worst = np.max(np.abs(got - want) - rel * np.abs(want)) / scale
    assert worst <= tol, (worst, tol)
