"""ctypes binding of libcandy_hip.so (include/candy_hip.h).

There is no CPU fallback: importing works anywhere (so the symbol table can be checked
without a GPU), but every compute call goes to the HIP library and raises CandyHipError
when the library or the GPU is missing.
"""
from __future__ import annotations

import ctypes
import os
from ctypes import POINTER, byref, c_char_p, c_double, c_float, c_int, c_int32, c_int64, c_size_t, c_uint32, c_void_p

import numpy as np

_HERE = os.path.dirname(os.path.abspath(__file__))
LIB_PATH = os.path.join(_HERE, "libcandy_hip.so")

Q4_0, Q8_0, Q4_K, Q6_K, Q4_0_GGML = 2, 8, 12, 14, 102

W_ATTN_NORM, W_Q, W_K, W_V, W_O, W_FFN_NORM, W_GATE, W_UP, W_DOWN, W_OUT_NORM, W_HEAD, W_EMBED = range(12)


class CandyHipError(RuntimeError):
    def __init__(self, status: int, text: str):
        super().__init__(f"candy_hip status {status}: {text}")
        self.status = status
        self.text = text


class LlamaConfig(ctypes.Structure):
    _fields_ = [("n_layers", c_int32), ("d_model", c_int32), ("n_heads", c_int32), ("n_kv_heads", c_int32),
                ("head_dim", c_int32), ("d_ffn", c_int32), ("vocab", c_int32), ("max_pos", c_int32),
                ("rms_eps", c_float), ("rope_base", c_float)]


class AttnSpec(ctypes.Structure):
    _fields_ = [("n_heads", c_int32), ("n_kv_heads", c_int32), ("head_dim", c_int32), ("window", c_int32),
                ("rope_dims", c_int32), ("rope_original", c_int32), ("scale", c_float), ("softcap", c_float),
                ("rope_base", c_double), ("rope_factor", c_double), ("rope_low", c_double), ("rope_high", c_double)]


class SuvazenLayer(ctypes.Structure):
    _fields_ = [("attn", AttnSpec), ("d_ffn", c_int32), ("has_sink", c_int32)]


class SuvazenConfig(ctypes.Structure):
    _fields_ = [("n_layers", c_int32), ("d_model", c_int32), ("vocab", c_int32), ("max_pos", c_int32),
                ("loop_start", c_int32), ("loop_stop", c_int32), ("loop_times", c_int32), ("act", c_int32),
                ("norm_eps", c_float), ("residual_mult", c_float), ("logit_scale", c_float), ("logit_softcap", c_float)]


class LatentSpec(ctypes.Structure):
    _fields_ = [("n_heads", c_int32), ("dim", c_int32), ("rot_dim", c_int32), ("vdim", c_int32), ("kv_rank", c_int32),
                ("q_rank", c_int32), ("scale", c_float), ("rope_base", c_double)]


class LruSpec(ctypes.Structure):
    _fields_ = [("width", c_int32), ("blocks", c_int32), ("taps", c_int32)]


class LruParams(ctypes.Structure):
    _fields_ = [(name, c_void_p) for name in ("by", "bx", "conv", "conv_b", "ra_b", "ri_b", "lam")]


class ExpertSpec(ctypes.Structure):
    _fields_ = [("n_experts", c_int32), ("top", c_int32), ("d_ff", c_int32), ("shared_ff", c_int32)]


class ExpertWeights(ctypes.Structure):
    _fields_ = [(name, c_void_p) for name in ("router", "up", "down", "shared_up", "shared_down")]


class GulisunLayer(ctypes.Structure):
    _fields_ = [("mixer", c_int32), ("kv_from", c_int32), ("has_sink", c_int32), ("reserved", c_int32), ("latent", LatentSpec),
                ("lru", LruSpec), ("experts", ExpertSpec)]


class GulisunConfig(ctypes.Structure):
    _fields_ = [("n_layers", c_int32), ("d_model", c_int32), ("vocab", c_int32), ("max_pos", c_int32), ("act", c_int32),
                ("norm_eps", c_float), ("embed_scale", c_float)]


ACT_BF16, ACT_F32 = 0, 1
EPI_NONE, EPI_SQUARED_RELU, EPI_SOFTCAP, EPI_ACT = 0, 1, 2, 3
SV_QK, SV_O, SV_UP, SV_DOWN, SV_HEAD, SV_EMBED = range(6)
(SV_NORM1, SV_NORM1_BIAS, SV_NORM1B, SV_NORM1B_BIAS, SV_NORM2, SV_NORM2_BIAS, SV_NORM2B, SV_NORM2B_BIAS, SV_SINK, SV_STEP,
 SV_FINAL, SV_FINAL_BIAS) = range(12)
GL_LATENT, GL_LRU = 0, 1
(GL_IN, GL_UQ, GL_UKV, GL_UKT, GL_GATES, GL_O, GL_ROUTER, GL_UP, GL_DOWN, GL_SHARED_UP, GL_SHARED_DOWN, GL_EMBED) = range(12)
(GL_NORM1, GL_NORM2, GL_Q_NORM, GL_KV_NORM, GL_SINK, GL_Y_BIAS, GL_X_BIAS, GL_CONV, GL_CONV_BIAS, GL_RA_BIAS, GL_RI_BIAS, GL_LAM,
 GL_FINAL) = range(13)

# name -> (restype, argtypes); exactly the symbols include/candy_hip.h declares
SIGNATURES = {
    "candy_hip_last_error": (c_char_p, []),
    "candy_hip_version": (c_char_p, []),
    "candy_hip_device_count": (c_int, [POINTER(c_int)]),
    "candy_hip_open": (c_int, [c_int, POINTER(c_void_p)]),
    "candy_hip_close": (c_int, [c_void_p]),
    "candy_hip_device_ordinal": (c_int, [c_void_p, POINTER(c_int)]),
    "candy_hip_device_name": (c_int, [c_void_p, c_char_p, c_size_t]),
    "candy_hip_synchronize": (c_int, [c_void_p]),
    "candy_hip_set_option": (c_int, [c_void_p, c_char_p, c_int64]),
    "candy_hip_get_option": (c_int, [c_void_p, c_char_p, POINTER(c_int64)]),
    "candy_hip_alloc": (c_int, [c_void_p, c_size_t, POINTER(c_void_p)]),
    "candy_hip_free": (c_int, [c_void_p, c_void_p]),
    "candy_hip_zero": (c_int, [c_void_p, c_void_p, c_size_t]),
    "candy_hip_h2d": (c_int, [c_void_p, c_void_p, c_void_p, c_size_t]),
    "candy_hip_d2h": (c_int, [c_void_p, c_void_p, c_void_p, c_size_t]),
    "candy_hip_d2d": (c_int, [c_void_p, c_void_p, c_void_p, c_size_t]),
    "candy_hip_block_elems": (c_int, [c_int]),
    "candy_hip_block_bytes": (c_int, [c_int]),
    "candy_hip_qweight_bytes": (c_size_t, [c_int, c_int64, c_int64]),
    "candy_hip_qtensor_upload": (c_int, [c_void_p, c_int, c_int64, c_int64, c_void_p, c_size_t, POINTER(c_void_p)]),
    "candy_hip_qtensor_wrap": (c_int, [c_void_p, c_int, c_int64, c_int64, c_void_p, c_size_t, POINTER(c_void_p)]),
    "candy_hip_qtensor_free": (c_int, [c_void_p]),
    "candy_hip_qtensor_info": (c_int, [c_void_p, POINTER(c_int), POINTER(c_int64), POINTER(c_int64),
                                       POINTER(c_size_t), POINTER(c_void_p)]),
    "candy_hip_dequantize_blocks": (c_int, [c_void_p, c_int, c_void_p, c_int64, c_void_p]),
    "candy_hip_dequantize": (c_int, [c_void_p, c_void_p, c_void_p]),
    "candy_hip_dequantize_blocks_f16": (c_int, [c_void_p, c_int, c_void_p, c_int64, c_void_p]),
    "candy_hip_dequantize_f16": (c_int, [c_void_p, c_void_p, c_void_p]),
    "candy_hip_dequantize_blocks_f64": (c_int, [c_void_p, c_int, c_void_p, c_int64, c_void_p]),
    "candy_hip_dmmv": (c_int, [c_void_p, c_void_p, c_void_p, c_void_p]),
    "candy_hip_quantize_q8_0": (c_int, [c_void_p, c_void_p, c_int64, c_int64, c_void_p]),
    "candy_hip_quantize": (c_int, [c_void_p, c_int, c_void_p, c_int64, c_int64, c_void_p]),
    "candy_hip_qmatmul": (c_int, [c_void_p, c_void_p, c_void_p, c_int64, c_void_p]),
    "candy_hip_qmatmul_noalloc": (c_int, [c_void_p, c_void_p, c_void_p, c_int64, c_void_p]),
    "candy_hip_qmatmul_q8": (c_int, [c_void_p, c_void_p, c_void_p, c_int64, c_void_p]),
    "candy_hip_qact_create": (c_int, [c_void_p, c_int64, c_int64, POINTER(c_void_p)]),
    "candy_hip_qact_free": (c_int, [c_void_p]),
    "candy_hip_qact_quantize": (c_int, [c_void_p, c_void_p, c_int64, c_int64]),
    "candy_hip_qmatmul_qact": (c_int, [c_void_p, c_void_p, c_void_p, c_void_p]),
    "candy_hip_matmul_f32": (c_int, [c_void_p, c_void_p, c_void_p, c_void_p, c_int64, c_int64, c_int64, c_int64, c_int]),
    "candy_hip_matmul_f32_strided": (c_int, [c_void_p, c_void_p, c_void_p, c_void_p, c_int64, c_int64, c_int64, c_int64,
                                             c_int64, c_int64, c_int64]),
    "candy_hip_rms_norm": (c_int, [c_void_p, c_void_p, c_void_p, c_float, c_int64, c_int64, c_void_p]),
    "candy_hip_rope": (c_int, [c_void_p, c_void_p, c_void_p, c_void_p, c_int64, c_int64, c_int64, c_int64, c_void_p]),
    "candy_hip_rope_i": (c_int, [c_void_p, c_void_p, c_void_p, c_void_p, c_int64, c_int64, c_int64, c_void_p]),
    "candy_hip_rope_thd": (c_int, [c_void_p, c_void_p, c_void_p, c_void_p, c_int64, c_int64, c_int64, c_int64, c_int64,
                                   c_void_p]),
    "candy_hip_softmax": (c_int, [c_void_p, c_void_p, c_int64, c_int64, c_void_p]),
    "candy_hip_silu": (c_int, [c_void_p, c_void_p, c_int64, c_void_p]),
    "candy_hip_add": (c_int, [c_void_p, c_void_p, c_void_p, c_int64, c_void_p]),
    "candy_hip_mul": (c_int, [c_void_p, c_void_p, c_void_p, c_int64, c_void_p]),
    "candy_hip_silu_mul": (c_int, [c_void_p, c_void_p, c_void_p, c_int64, c_void_p]),
    "candy_hip_argmax": (c_int, [c_void_p, c_void_p, c_int64, c_int64, c_void_p]),
    "candy_hip_index_select": (c_int, [c_void_p, c_void_p, c_int64, c_int64, c_void_p, c_int64, c_void_p]),
    "candy_hip_qindex_select": (c_int, [c_void_p, c_void_p, c_void_p, c_int64, c_void_p]),
    "candy_hip_attention_decode": (c_int, [c_void_p, c_void_p, c_void_p, c_void_p, c_int64, c_int64, c_int64, c_int64,
                                           c_int64, c_float, c_void_p]),
    "candy_hip_llama_create": (c_int, [c_void_p, POINTER(LlamaConfig), POINTER(c_void_p)]),
    "candy_hip_llama_free": (c_int, [c_void_p]),
    "candy_hip_llama_set_qweight": (c_int, [c_void_p, c_int, c_int, c_void_p]),
    "candy_hip_llama_set_norm": (c_int, [c_void_p, c_int, c_int, c_void_p]),
    "candy_hip_llama_set_graph": (c_int, [c_void_p, c_int]),
    "candy_hip_llama_set_kv_f16": (c_int, [c_void_p, c_int]),
    "candy_hip_llama_kv_cache": (c_int, [c_void_p, POINTER(c_void_p), POINTER(c_void_p), POINTER(c_size_t)]),
    "candy_hip_llama_hidden": (c_int, [c_void_p, POINTER(c_void_p)]),
    "candy_hip_llama_decode": (c_int, [c_void_p, c_int32, c_int32, POINTER(c_void_p), POINTER(c_int32)]),
    "candy_hip_llama_generate": (c_int, [c_void_p, c_int32, c_int32, c_int32, POINTER(c_int32)]),
    "candy_hip_llama_decode_hidden": (c_int, [c_void_p, c_void_p, c_int32, POINTER(c_void_p), POINTER(c_int32)]),
    "candy_hip_llama_prefill": (c_int, [c_void_p, POINTER(c_int32), c_int32, c_int32, POINTER(c_void_p),
                                        POINTER(c_int32)]),
    "candy_hip_llama_decoder": (c_void_p, [c_void_p]),
    "candy_hip_dense_upload": (c_int, [c_void_p, c_int64, c_int64, c_void_p, POINTER(c_void_p)]),
    "candy_hip_dense_free": (c_int, [c_void_p]),
    "candy_hip_dense_info": (c_int, [c_void_p, POINTER(c_int64), POINTER(c_int64), POINTER(c_size_t)]),
    "candy_hip_dense_matmul": (c_int, [c_void_p, c_void_p, c_void_p, c_int64, c_int, c_int, c_float, c_float, c_void_p]),
    "candy_hip_dense_sweep": (c_int, [c_void_p, POINTER(c_void_p), c_int, c_void_p, c_int64, c_int, c_int, POINTER(c_float)]),
    "candy_hip_layer_norm": (c_int, [c_void_p, c_void_p, c_void_p, c_void_p, c_float, c_int64, c_int64, c_void_p]),
    "candy_hip_add_layer_norm": (c_int, [c_void_p, c_void_p, c_void_p, c_void_p, c_void_p, c_float, c_float, c_void_p,
                                         c_int64, c_int64]),
    "candy_hip_add_rms_norm": (c_int, [c_void_p, c_void_p, c_void_p, c_void_p, c_float, c_float, c_int64, c_int64]),
    "candy_hip_pad32": (c_int32, [c_int32]),
    "candy_hip_pad64": (c_int32, [c_int32]),
    "candy_hip_latent_row": (c_int32, [POINTER(LatentSpec)]),
    "candy_hip_latent_attention": (c_int, [c_void_p, POINTER(LatentSpec), c_int, c_void_p, c_void_p, c_void_p, c_float, c_void_p, c_void_p,
                                           c_void_p, c_int64, c_int32, c_int32, c_void_p, c_int, c_void_p]),
    "candy_hip_lru_state_floats": (c_int64, [POINTER(LruSpec)]),
    "candy_hip_lru_gate_rows": (c_int64, [POINTER(LruSpec)]),
    "candy_hip_lru": (c_int, [c_void_p, POINTER(LruSpec), c_int, c_void_p, POINTER(LruParams), c_void_p, c_void_p, c_int64, c_int32, c_int,
                              c_void_p]),
    "candy_hip_experts": (c_int, [c_void_p, POINTER(ExpertSpec), c_int, POINTER(ExpertWeights), c_void_p, c_int64, c_int, c_void_p,
                                  c_void_p, c_void_p]),
    "candy_hip_attn_row": (c_int, [c_int]),
    "candy_hip_window_attention": (c_int, [c_void_p, POINTER(AttnSpec), c_int, c_void_p, c_int64, c_int32, c_int32, c_void_p,
                                           c_void_p, c_void_p, c_int, c_void_p]),
    "candy_hip_decoder_free": (c_int, [c_void_p]),
    "candy_hip_decoder_set_graph": (c_int, [c_void_p, c_int]),
    "candy_hip_decoder_hidden": (c_int, [c_void_p, POINTER(c_void_p)]),
    "candy_hip_decoder_kv_cache": (c_int, [c_void_p, POINTER(c_void_p), POINTER(c_void_p), POINTER(c_size_t)]),
    "candy_hip_decoder_decode": (c_int, [c_void_p, c_int32, c_int32, POINTER(c_void_p), POINTER(c_int32)]),
    "candy_hip_decoder_decode_hidden": (c_int, [c_void_p, c_void_p, c_int32, POINTER(c_void_p), POINTER(c_int32)]),
    "candy_hip_decoder_generate": (c_int, [c_void_p, c_int32, c_int32, c_int32, POINTER(c_int32)]),
    "candy_hip_decoder_prefill": (c_int, [c_void_p, POINTER(c_int32), c_int32, c_int32, POINTER(c_void_p), POINTER(c_int32)]),
    "candy_hip_decoder_prefill_rows": (c_int, [c_void_p, POINTER(c_int32), c_int32, c_int32, POINTER(c_int32), c_int32,
                                               POINTER(c_void_p)]),
    "candy_hip_decoder_prompt_hidden": (c_int, [c_void_p, POINTER(c_void_p), POINTER(c_int64)]),
    "candy_hip_suvazen_create": (c_int, [c_void_p, POINTER(SuvazenConfig), POINTER(SuvazenLayer), POINTER(c_void_p)]),
    "candy_hip_suvazen_decoder": (c_void_p, [c_void_p]),
    "candy_hip_suvazen_set_matrix": (c_int, [c_void_p, c_int, c_int, c_void_p]),
    "candy_hip_suvazen_set_vector": (c_int, [c_void_p, c_int, c_int, c_void_p, c_int64]),
    "candy_hip_gulisun_create": (c_int, [c_void_p, POINTER(GulisunConfig), POINTER(GulisunLayer), POINTER(c_void_p)]),
    "candy_hip_gulisun_decoder": (c_void_p, [c_void_p]),
    "candy_hip_gulisun_set_matrix": (c_int, [c_void_p, c_int, c_int, c_void_p]),
    "candy_hip_gulisun_set_vector": (c_int, [c_void_p, c_int, c_int, c_void_p, c_int64]),
    "candy_hip_qmatmul_sweep": (c_int, [c_void_p, POINTER(c_void_p), c_int, c_void_p, c_int64, c_void_p, c_int, c_int,
                                        POINTER(c_float)]),
    "candy_hip_qmatmul_sustained_sweep": (c_int, [c_void_p, POINTER(c_void_p), c_int, c_int, c_int, c_void_p, c_void_p, c_int,
                                                  POINTER(c_float)]),
    "candy_hip_dequantize_sweep": (c_int, [c_void_p, POINTER(c_void_p), c_int, c_void_p, c_int, c_int, POINTER(c_float)]),
    "candy_hip_quantize_sweep": (c_int, [c_void_p, c_void_p, c_int64, c_int, c_int64, c_int64, c_void_p, c_int, c_int,
                                         POINTER(c_float)]),
    "candy_hip_stream_probe": (c_int, [c_void_p, c_size_t, c_size_t, c_int, POINTER(c_float)]),
    "candy_hip_launch_probe": (c_int, [c_void_p, c_int, c_int, POINTER(c_float)]),
    "candy_hip_timer_start": (c_int, [c_void_p]),
    "candy_hip_timer_stop": (c_int, [c_void_p, POINTER(c_float)]),
}

_lib = None


def lib() -> ctypes.CDLL:
    """Load libcandy_hip.so; raises if it has not been built (there is nothing to fall back to)."""
    global _lib
    if _lib is None:
        if not os.path.exists(LIB_PATH):
            raise CandyHipError(-1, f"{LIB_PATH} is missing: build it with `make -C candy_amd/csrc` "
                                    "(or __graft_entry__.build())")
        L = ctypes.CDLL(LIB_PATH)
        for name, (res, args) in SIGNATURES.items():
            fn = getattr(L, name)
            fn.restype = res
            fn.argtypes = args
        _lib = L
    return _lib


def _check(status: int):
    if status != 0:
        raise CandyHipError(status, lib().candy_hip_last_error().decode(errors="replace"))


def device_count() -> int:
    n = c_int(0)
    rc = lib().candy_hip_device_count(byref(n))
    return n.value if rc == 0 else 0


class Buffer:
    """A raw device allocation (what backs a BackendStorage)."""

    def __init__(self, dev: "Device", nbytes: int):
        self.dev, self.nbytes = dev, int(nbytes)
        p = c_void_p()
        _check(lib().candy_hip_alloc(dev.handle, self.nbytes, byref(p)))
        self.ptr = p.value

    def free(self):
        if self.ptr is not None and self.dev.handle is not None:
            _check(lib().candy_hip_free(self.dev.handle, self.ptr))
        self.ptr = None

    def __del__(self):
        try:
            self.free()
        except Exception:
            pass

    def upload(self, arr: np.ndarray, offset: int = 0) -> "Buffer":
        a = np.ascontiguousarray(arr)
        assert offset + a.nbytes <= self.nbytes
        _check(lib().candy_hip_h2d(self.dev.handle, self.ptr + offset, a.ctypes.data, a.nbytes))
        return self

    def download(self, dtype, count: int | None = None, offset: int = 0) -> np.ndarray:
        dt = np.dtype(dtype)
        if count is None:
            count = (self.nbytes - offset) // dt.itemsize
        out = np.empty(count, dt)
        _check(lib().candy_hip_d2h(self.dev.handle, out.ctypes.data, self.ptr + offset, out.nbytes))
        return out

    def zero(self) -> "Buffer":
        _check(lib().candy_hip_zero(self.dev.handle, self.ptr, self.nbytes))
        return self


class QTensor:
    """Device-resident quantized weight [rows, cols] in its original block layout."""

    def __init__(self, dev: "Device", fmt: int, rows: int, cols: int, blocks: np.ndarray):
        b = np.ascontiguousarray(blocks).view(np.uint8).reshape(-1)
        h = c_void_p()
        _check(lib().candy_hip_qtensor_upload(dev.handle, fmt, rows, cols, b.ctypes.data, b.nbytes, byref(h)))
        self.dev, self.fmt, self.rows, self.cols, self.nbytes, self.handle = dev, fmt, rows, cols, b.nbytes, h.value

    @classmethod
    def quantize(cls, dev: "Device", fmt: int, x: np.ndarray) -> "QTensor":
        """f32 [rows, cols] -> a weight of format fmt, quantized on the device and kept there."""
        x = np.ascontiguousarray(x, np.float32)
        rows, cols = x.reshape(-1, x.shape[-1]).shape
        nbytes = lib().candy_hip_qweight_bytes(fmt, rows, cols)
        src = dev.from_numpy(x)
        dst = dev.alloc(nbytes + 64)  # spare bytes after the blocks: every tile kernel may take the weight
        _check(lib().candy_hip_quantize(dev.handle, fmt, src.ptr, rows, cols, dst.ptr))
        q = cls.__new__(cls)
        h = c_void_p()
        _check(lib().candy_hip_qtensor_wrap(dev.handle, fmt, rows, cols, dst.ptr, nbytes + 64, byref(h)))
        q.dev, q.fmt, q.rows, q.cols, q.nbytes, q.handle = dev, fmt, rows, cols, nbytes, h.value
        q._blocks = dst  # the wrapped device memory stays owned here
        return q

    def free(self):
        if self.handle is not None and self.dev.handle is not None:
            _check(lib().candy_hip_qtensor_free(self.handle))
        self.handle = None

    def __del__(self):
        try:
            self.free()
        except Exception:
            pass


def bf16_bits(x: np.ndarray) -> np.ndarray:
    """float32 -> bfloat16 bit patterns, rounded to nearest even (finite inputs)."""
    u = np.ascontiguousarray(x, np.float32).view(np.uint32)
    return ((u + 0x7FFF + ((u >> 16) & 1)) >> 16).astype(np.uint16)


def bf16_values(bits: np.ndarray) -> np.ndarray:
    """bfloat16 bit patterns -> float32."""
    return (np.ascontiguousarray(bits, np.uint16).astype(np.uint32) << 16).view(np.float32)


class Dense:
    """Device-resident bfloat16 weight [rows, cols]; `bits` are the raw 16-bit values."""

    def __init__(self, dev: "Device", bits: np.ndarray):
        b = np.ascontiguousarray(bits)
        if b.dtype != np.uint16 or b.ndim != 2:
            raise ValueError("a dense weight is a 2-D array of bfloat16 bit patterns (uint16)")
        h = c_void_p()
        _check(lib().candy_hip_dense_upload(dev.handle, b.shape[0], b.shape[1], b.ctypes.data, byref(h)))
        self.dev, self.rows, self.cols, self.handle = dev, b.shape[0], b.shape[1], h.value

    @property
    def nbytes(self) -> int:
        n = c_size_t()
        _check(lib().candy_hip_dense_info(self.handle, None, None, byref(n)))
        return n.value

    def free(self):
        if self.handle is not None and self.dev.handle is not None:
            _check(lib().candy_hip_dense_free(self.handle))
        self.handle = None

    def __del__(self):
        try:
            self.free()
        except Exception:
            pass


class Device:
    """One GPU: candy.BackendDevice on the HIP side."""

    def __init__(self, ordinal: int = 0):
        h = c_void_p()
        _check(lib().candy_hip_open(ordinal, byref(h)))
        self.handle = h.value
        buf = ctypes.create_string_buffer(256)
        _check(lib().candy_hip_device_name(self.handle, buf, 256))
        self.name = buf.value.decode()

    def close(self):
        if self.handle is not None:
            lib().candy_hip_close(self.handle)
            self.handle = None

    # ---- switches (include/candy_hip.h lists the keys)
    def set_option(self, key: str, value: int):
        _check(lib().candy_hip_set_option(self.handle, key.encode(), int(value)))

    def get_option(self, key: str) -> int:
        v = c_int64(0)
        _check(lib().candy_hip_get_option(self.handle, key.encode(), byref(v)))
        return v.value

    # ---- memory
    def alloc(self, nbytes: int) -> Buffer:
        return Buffer(self, nbytes)

    def from_numpy(self, arr: np.ndarray) -> Buffer:
        a = np.ascontiguousarray(arr)
        return Buffer(self, max(a.nbytes, 1)).upload(a) if a.nbytes else Buffer(self, 1)

    def synchronize(self):
        _check(lib().candy_hip_synchronize(self.handle))

    def qtensor(self, fmt: int, rows: int, cols: int, blocks: np.ndarray) -> QTensor:
        return QTensor(self, fmt, rows, cols, blocks)

    # ---- quantized path
    def dequantize_blocks(self, fmt: int, blocks: np.ndarray) -> np.ndarray:
        b = np.ascontiguousarray(blocks).view(np.uint8).reshape(-1)
        bs, qk = lib().candy_hip_block_bytes(fmt), lib().candy_hip_block_elems(fmt)
        if bs == 0:
            _check(lib().candy_hip_dequantize_blocks(self.handle, fmt, None, 0, None))
        nb = b.size // bs
        src = self.from_numpy(b)
        dst = self.alloc(max(nb * qk * 4, 16))
        _check(lib().candy_hip_dequantize_blocks(self.handle, fmt, src.ptr, nb, dst.ptr))
        return dst.download(np.float32, nb * qk)

    def dequantize(self, q: QTensor) -> np.ndarray:
        dst = self.alloc(q.rows * q.cols * 4)
        _check(lib().candy_hip_dequantize(self.handle, q.handle, dst.ptr))
        return dst.download(np.float32, q.rows * q.cols).reshape(q.rows, q.cols)

    def dequantize_blocks_as(self, fmt: int, blocks: np.ndarray, dtype) -> np.ndarray:
        """Blocks -> float16 or float64 values (the reference's other dequantize outputs)."""
        dtype = np.dtype(dtype)
        entry = {np.dtype(np.float16): lib().candy_hip_dequantize_blocks_f16,
                 np.dtype(np.float64): lib().candy_hip_dequantize_blocks_f64}[dtype]
        b = np.ascontiguousarray(blocks).view(np.uint8).reshape(-1)
        bs, qk = lib().candy_hip_block_bytes(fmt), lib().candy_hip_block_elems(fmt)
        if bs == 0:
            _check(entry(self.handle, fmt, None, 0, None))
        nb = b.size // bs
        src = self.from_numpy(b)
        dst = self.alloc(max(nb * qk * dtype.itemsize, 16))
        _check(entry(self.handle, fmt, src.ptr, nb, dst.ptr))
        return dst.download(dtype, nb * qk)

    def dequantize_f16(self, q: QTensor) -> np.ndarray:
        dst = self.alloc(q.rows * q.cols * 2)
        _check(lib().candy_hip_dequantize_f16(self.handle, q.handle, dst.ptr))
        return dst.download(np.float16, q.rows * q.cols).reshape(q.rows, q.cols)

    def dmmv(self, q: QTensor, x: np.ndarray) -> np.ndarray:
        """y[rows] = dequantize(W) . x with f32 activations (no activation quantizer)."""
        x = np.ascontiguousarray(x, np.float32).reshape(-1)
        assert x.size == q.cols
        src = self.from_numpy(x)
        dst = self.alloc(max(q.rows * 4, 16))
        _check(lib().candy_hip_dmmv(self.handle, q.handle, src.ptr, dst.ptr))
        return dst.download(np.float32, q.rows)

    def quantize_q8_0(self, x: np.ndarray) -> np.ndarray:
        x = np.ascontiguousarray(x, np.float32)
        x2 = x.reshape(-1, x.shape[-1]) if x.ndim > 1 else x.reshape(1, -1)
        rows, cols = x2.shape
        src = self.from_numpy(x2)
        dst = self.alloc(max(rows * cols // 32 * 34, 2))
        _check(lib().candy_hip_quantize_q8_0(self.handle, src.ptr, rows, cols, dst.ptr))
        return dst.download(np.uint8, rows * cols // 32 * 34)

    def quantize(self, fmt: int, x: np.ndarray) -> np.ndarray:
        """f32 [rows, cols] -> the blocks of format fmt (host bytes), quantized on the device."""
        x = np.ascontiguousarray(x, np.float32)
        x2 = x.reshape(-1, x.shape[-1]) if x.ndim > 1 else x.reshape(1, -1)
        rows, cols = x2.shape
        nbytes = lib().candy_hip_qweight_bytes(fmt, rows, cols)
        src = self.from_numpy(x2)
        dst = self.alloc(max(nbytes, 2))
        _check(lib().candy_hip_quantize(self.handle, fmt, src.ptr, rows, cols, dst.ptr))
        return dst.download(np.uint8, nbytes)

    def qmatmul(self, w: QTensor, x: np.ndarray) -> np.ndarray:
        x = np.ascontiguousarray(x, np.float32).reshape(-1, w.cols)
        m = x.shape[0]
        src = self.from_numpy(x)
        dst = self.alloc(max(m * w.rows * 4, 4))
        _check(lib().candy_hip_qmatmul(self.handle, w.handle, src.ptr, m, dst.ptr))
        return dst.download(np.float32, m * w.rows).reshape(m, w.rows)

    def qmatmul_q8(self, w: QTensor, x_blocks: np.ndarray, m: int) -> np.ndarray:
        src = self.from_numpy(np.ascontiguousarray(x_blocks).view(np.uint8))
        dst = self.alloc(max(m * w.rows * 4, 4))
        _check(lib().candy_hip_qmatmul_q8(self.handle, w.handle, src.ptr, m, dst.ptr))
        return dst.download(np.float32, m * w.rows).reshape(m, w.rows)

    # ---- f32 ops (host arrays in, host arrays out; the C ABI itself works on device pointers)
    def _f32(self, a) -> Buffer:
        return self.from_numpy(np.ascontiguousarray(a, np.float32).reshape(-1))

    def matmul_f32(self, a, b, batch, m, n, k, rhs_transposed=False) -> np.ndarray:
        da, db = self._f32(a), self._f32(b)
        dc = self.alloc(max(batch * m * n * 4, 4))
        _check(lib().candy_hip_matmul_f32(self.handle, da.ptr, db.ptr, dc.ptr, batch, m, n, k, int(rhs_transposed)))
        return dc.download(np.float32, batch * m * n)

    def matmul_f32_strided(self, a, b, m, n, k, a_strides, b_strides, a_offset=0, b_offset=0) -> np.ndarray:
        """One batch; a_strides / b_strides are (row, column) element strides, the offsets the layouts' start offsets."""
        da, db = self._f32(a), self._f32(b)
        dc = self.alloc(m * n * 4)
        _check(lib().candy_hip_matmul_f32_strided(self.handle, da.ptr + 4 * a_offset, db.ptr + 4 * b_offset, dc.ptr, m, n, k,
                                                  a_strides[0], a_strides[1], b_strides[0], b_strides[1]))
        return dc.download(np.float32, m * n)

    def rms_norm(self, x, cols: int, eps: float, alpha=None) -> np.ndarray:
        x = np.ascontiguousarray(x, np.float32).reshape(-1)
        rows = x.size // cols if cols else 0
        dx = self._f32(x)
        da = self._f32(alpha) if alpha is not None else None
        out = self.alloc(max(x.nbytes, 4))
        _check(lib().candy_hip_rms_norm(self.handle, dx.ptr, da.ptr if da else None, eps, rows, cols, out.ptr))
        return out.download(np.float32, x.size)

    def rope(self, src, cos, sin, bh, td, d, stride_b=0) -> np.ndarray:
        src = np.ascontiguousarray(src, np.float32).reshape(-1)
        ds, dc, dn = self._f32(src), self._f32(cos), self._f32(sin)
        out = self.from_numpy(src)
        _check(lib().candy_hip_rope(self.handle, ds.ptr, dc.ptr, dn.ptr, bh, td, d, stride_b, out.ptr))
        return out.download(np.float32, src.size)

    def rope_i(self, src, cos, sin, bh, td, stride_b=0) -> np.ndarray:
        """RopeI (backend.go:156): adjacent pairs."""
        src = np.ascontiguousarray(src, np.float32).reshape(-1)
        if src.size == 0:
            return src.copy()
        ds, dc, dn = self._f32(src), self._f32(cos), self._f32(sin)
        out = self.from_numpy(src)
        _check(lib().candy_hip_rope_i(self.handle, ds.ptr, dc.ptr, dn.ptr, bh, td, stride_b, out.ptr))
        return out.download(np.float32, src.size)

    def rope_thd(self, src, cos, sin, b, t, h, d, stride_b=0) -> np.ndarray:
        """RopeThd (backend.go:162): [b, t, h, d] layout."""
        src = np.ascontiguousarray(src, np.float32).reshape(-1)
        if src.size == 0:
            return src.copy()
        ds, dc, dn = self._f32(src), self._f32(cos), self._f32(sin)
        out = self.from_numpy(src)
        _check(lib().candy_hip_rope_thd(self.handle, ds.ptr, dc.ptr, dn.ptr, b, t, h, d, stride_b, out.ptr))
        return out.download(np.float32, src.size)

    def softmax(self, src, cols: int) -> np.ndarray:
        src = np.ascontiguousarray(src, np.float32).reshape(-1)
        rows = src.size // cols if cols else 0
        ds = self._f32(src)
        out = self.alloc(max(src.nbytes, 4))
        _check(lib().candy_hip_softmax(self.handle, ds.ptr, rows, cols, out.ptr))
        return out.download(np.float32, src.size)

    def _binary(self, fn, a, b) -> np.ndarray:
        a = np.ascontiguousarray(a, np.float32).reshape(-1)
        da, db = self._f32(a), self._f32(b)
        out = self.alloc(max(a.nbytes, 4))
        _check(fn(self.handle, da.ptr, db.ptr, a.size, out.ptr))
        return out.download(np.float32, a.size)

    def add(self, a, b):
        return self._binary(lib().candy_hip_add, a, b)

    def mul(self, a, b):
        return self._binary(lib().candy_hip_mul, a, b)

    def silu_mul(self, gate, up):
        return self._binary(lib().candy_hip_silu_mul, gate, up)

    def silu(self, x) -> np.ndarray:
        x = np.ascontiguousarray(x, np.float32).reshape(-1)
        dx = self._f32(x)
        out = self.alloc(max(x.nbytes, 4))
        _check(lib().candy_hip_silu(self.handle, dx.ptr, x.size, out.ptr))
        return out.download(np.float32, x.size)

    def argmax(self, src, cols: int) -> np.ndarray:
        src = np.ascontiguousarray(src, np.float32).reshape(-1)
        rows = src.size // cols if cols else 0
        ds = self._f32(src)
        out = self.alloc(max(rows * 4, 4))
        _check(lib().candy_hip_argmax(self.handle, ds.ptr, rows, cols, out.ptr))
        return out.download(np.uint32, rows)

    def index_select(self, table, ids) -> np.ndarray:
        table = np.ascontiguousarray(table, np.float32)
        ids = np.ascontiguousarray(ids, np.int64)
        dt, di = self._f32(table), self.from_numpy(ids)
        out = self.alloc(max(ids.size * table.shape[1] * 4, 4))
        _check(lib().candy_hip_index_select(self.handle, dt.ptr, table.shape[0], table.shape[1], di.ptr, ids.size, out.ptr))
        return out.download(np.float32, ids.size * table.shape[1]).reshape(ids.size, table.shape[1])

    def qindex_select(self, q: QTensor, ids) -> np.ndarray:
        ids = np.ascontiguousarray(ids, np.int64)
        di = self.from_numpy(ids)
        out = self.alloc(max(ids.size * q.cols * 4, 16))
        _check(lib().candy_hip_qindex_select(self.handle, q.handle, di.ptr, ids.size, out.ptr))
        return out.download(np.float32, ids.size * q.cols).reshape(ids.size, q.cols)

    def attention_decode(self, q, k_cache, v_cache, n_heads, n_kv_heads, head_dim, n_pos, cache_stride, scale):
        dq, dk, dv = self._f32(q), self._f32(k_cache), self._f32(v_cache)
        out = self.alloc(n_heads * head_dim * 4)
        _check(lib().candy_hip_attention_decode(self.handle, dq.ptr, dk.ptr, dv.ptr, n_heads, n_kv_heads, head_dim,
                                                n_pos, cache_stride, scale, out.ptr))
        return out.download(np.float32, n_heads * head_dim)

    # ---- bfloat16 weights, layer norms, windowed attention
    def dense(self, bits: np.ndarray) -> Dense:
        return Dense(self, bits)

    def dense_matmul(self, w: Dense, x, act: int = ACT_BF16, epilogue: int = EPI_NONE, scale: float = 1.0,
                     cap: float = 0.0) -> np.ndarray:
        x = np.ascontiguousarray(x, np.float32).reshape(-1, w.cols)
        m = x.shape[0]
        src, dst = self.from_numpy(x), self.alloc(max(m * w.rows * 4, 4))
        _check(lib().candy_hip_dense_matmul(self.handle, w.handle, src.ptr, m, act, epilogue, scale, cap, dst.ptr))
        return dst.download(np.float32, m * w.rows).reshape(m, w.rows)

    def dense_sweep(self, weights: list, x_buf: "Buffer", m: int, iters: int, epilogue: int = EPI_NONE) -> float:
        """Elapsed milliseconds of `iters` back-to-back bfloat16 contractions rotating over `weights`."""
        arr = (c_void_p * len(weights))(*[w.handle for w in weights])
        ms = c_float(0)
        _check(lib().candy_hip_dense_sweep(self.handle, arr, len(weights), x_buf.ptr, m, epilogue, iters, byref(ms)))
        return ms.value

    def layer_norm(self, x, w, b, eps: float) -> np.ndarray:
        x = np.ascontiguousarray(x, np.float32)
        cols = x.shape[-1]
        dx, dw, db, out = self._f32(x), self._f32(w), self._f32(b), self.alloc(max(x.nbytes, 4))
        _check(lib().candy_hip_layer_norm(self.handle, dx.ptr, dw.ptr, db.ptr, eps, x.size // cols, cols, out.ptr))
        return out.download(np.float32, x.size).reshape(x.shape)

    def add_layer_norm(self, x, y, w, b, eps: float, mult: float, step=None) -> np.ndarray:
        """x + mult * layer_norm(y) (+ step)"""
        x = np.ascontiguousarray(x, np.float32)
        cols = x.shape[-1]
        dx, dy, dw, db = self._f32(x), self._f32(y), self._f32(w), self._f32(b)
        ds = self._f32(step) if step is not None else None
        _check(lib().candy_hip_add_layer_norm(self.handle, dx.ptr, dy.ptr, dw.ptr, db.ptr, eps, mult,
                                              ds.ptr if ds else None, x.size // cols, cols))
        return dx.download(np.float32, x.size).reshape(x.shape)

    def window_attention(self, spec: AttnSpec, act: int, qk, pos0: int, max_pos: int, k_cache: "Buffer", v_cache: "Buffer",
                         sink=None, decode: bool = False) -> np.ndarray:
        """qk [n, (n_heads + n_kv_heads) * head_dim] at positions pos0 ..; the caches receive the new rows."""
        qk = np.ascontiguousarray(qk, np.float32)
        n, width = qk.shape[0], spec.n_heads * spec.head_dim
        if qk.shape[1] != width + spec.n_kv_heads * spec.head_dim:
            raise ValueError("qk rows do not fit the spec")
        need = spec.n_kv_heads * max_pos * lib().candy_hip_attn_row(spec.head_dim) * (4 if act == ACT_F32 else 2)
        if k_cache.nbytes < need or v_cache.nbytes < need:
            raise ValueError("cache too small")
        dq, out = self._f32(qk), self.alloc(n * width * 4)
        ds = self._f32(sink) if sink is not None else None
        _check(lib().candy_hip_window_attention(self.handle, byref(spec), act, dq.ptr, n, pos0, max_pos, k_cache.ptr,
                                                v_cache.ptr, ds.ptr if ds else None, int(decode), out.ptr))
        return out.download(np.float32, n * width).reshape(n, width)

    # ---- latent attention, recurrent unit, experts, RMS norm of a result
    def add_rms_norm(self, x, y, w, eps: float, mult: float) -> np.ndarray:
        """x + mult * rms_norm(y)"""
        x = np.ascontiguousarray(x, np.float32)
        cols = x.shape[-1]
        dx, dy, dw = self._f32(x), self._f32(y), self._f32(w)
        _check(lib().candy_hip_add_rms_norm(self.handle, dx.ptr, dy.ptr, dw.ptr, eps, mult, x.size // cols, cols))
        return dx.download(np.float32, x.size).reshape(x.shape)

    def latent_attention(self, spec: LatentSpec, act: int, q, dkv, kv_norm, eps: float, ukv: Dense, ukt: Dense, pos0: int, max_pos: int,
                         cache: "Buffer", sink=None, decode: bool = False) -> np.ndarray:
        """Rows at positions pos0 .. in the padded layouts of include/candy_hip.h; dkv None: the cache holds them already."""
        q = np.ascontiguousarray(q, np.float32)
        n, width = q.shape[0], spec.n_heads * lib().candy_hip_pad32(spec.vdim)
        row = lib().candy_hip_latent_row(byref(spec))
        dk = lib().candy_hip_pad32(spec.dim) + lib().candy_hip_pad32(spec.rot_dim)
        if q.shape[1] != spec.n_heads * dk or (dkv is not None and np.shape(dkv) != (n, row)):
            raise ValueError("rows do not fit the spec")
        if cache.nbytes < max_pos * row * (4 if act == ACT_F32 else 2):
            raise ValueError("cache too small")
        dq, out = self._f32(q), self.alloc(n * width * 4)
        dd = self._f32(dkv) if dkv is not None else None
        dn = self._f32(kv_norm) if dkv is not None else None
        ds = self._f32(sink) if sink is not None else None
        _check(lib().candy_hip_latent_attention(self.handle, byref(spec), act, dq.ptr, dd.ptr if dd else None, dn.ptr if dn else None, eps,
                                                ukv.handle, ukt.handle, ds.ptr if ds else None, n, pos0, max_pos, cache.ptr, int(decode),
                                                out.ptr))
        return out.download(np.float32, n * width).reshape(n, width)

    def lru(self, spec: LruSpec, act: int, z, params: dict, gates: Dense, state: "Buffer", pos0: int, decode: bool = False) -> np.ndarray:
        """z [n, 2 * pad64(width)]; params: the fields of LruParams, padded."""
        z = np.ascontiguousarray(z, np.float32)
        n, wp = z.shape[0], lib().candy_hip_pad64(spec.width)
        if z.shape[1] != 2 * wp or state.nbytes < 4 * lib().candy_hip_lru_state_floats(byref(spec)):
            raise ValueError("rows or state do not fit the spec")
        bufs = {k: self._f32(np.ascontiguousarray(v, np.float32)) for k, v in params.items()}
        for k, b in bufs.items():
            if b.nbytes < 4 * wp * (spec.taps if k == "conv" else 1):
                raise ValueError(f"{k} is not padded")
        p = LruParams(**{k: b.ptr for k, b in bufs.items()})
        dz, out = self._f32(z), self.alloc(n * spec.width * 4)
        _check(lib().candy_hip_lru(self.handle, byref(spec), act, dz.ptr, byref(p), gates.handle, state.ptr, n, pos0, int(decode), out.ptr))
        return out.download(np.float32, n * spec.width).reshape(n, spec.width)

    def experts(self, spec: ExpertSpec, act: int, weights: dict, x, decode: bool = False):
        """weights: the fields of ExpertWeights as Dense; returns the result, and for several rows the choice and its weights."""
        x = np.ascontiguousarray(x, np.float32)
        n, d = x.shape
        w = ExpertWeights(**{k: v.handle for k, v in weights.items()})
        dx, out = self._f32(x), self.alloc(n * d * 4)
        ids, wts = (None, None) if decode else (self.alloc(n * spec.top * 4), self.alloc(n * spec.top * 4))
        _check(lib().candy_hip_experts(self.handle, byref(spec), act, byref(w), dx.ptr, n, int(decode), out.ptr,
                                       ids.ptr if ids else None, wts.ptr if wts else None))
        y = out.download(np.float32, n * d).reshape(n, d)
        if decode:
            return y
        return y, ids.download(np.int32, n * spec.top).reshape(n, -1), wts.download(np.float32, n * spec.top).reshape(n, -1)

    # ---- timing
    def qmatmul_sweep(self, weights: list, x_buf: "Buffer", m: int, y_buf: "Buffer", iters: int,
                      quantize_each: bool = True) -> float:
        """Elapsed milliseconds of `iters` back-to-back contractions rotating over `weights`."""
        arr = (c_void_p * len(weights))(*[w.handle for w in weights])
        ms = c_float(0)
        _check(lib().candy_hip_qmatmul_sweep(self.handle, arr, len(weights), x_buf.ptr, m, y_buf.ptr, iters,
                                             int(quantize_each), byref(ms)))
        return ms.value

    def qmatmul_sustained_sweep(self, weights: list, group: int, n_streams: int, x_buf: "Buffer", y_buf: "Buffer",
                                iters: int) -> float:
        """Elapsed milliseconds of `iters` batch-1 launches of `group` weights each, alternating over `n_streams`
        streams (y_buf: n_streams * group * rows floats)."""
        arr = (c_void_p * len(weights))(*[w.handle for w in weights])
        ms = c_float(0)
        _check(lib().candy_hip_qmatmul_sustained_sweep(self.handle, arr, len(weights), group, n_streams, x_buf.ptr,
                                                       y_buf.ptr, iters, byref(ms)))
        return ms.value

    def dequantize_sweep(self, weights: list, out_buf: "Buffer", iters: int, n_out: int = 1) -> float:
        """out_buf holds n_out outputs of rows*cols f32 end to end; iteration i writes output i % n_out."""
        arr = (c_void_p * len(weights))(*[w.handle for w in weights])
        ms = c_float(0)
        _check(lib().candy_hip_dequantize_sweep(self.handle, arr, len(weights), out_buf.ptr, n_out, iters, byref(ms)))
        return ms.value

    def quantize_sweep(self, x_buf: "Buffer", x_stride: int, n_x: int, rows: int, cols: int, out_buf: "Buffer",
                       iters: int, n_out: int = 1) -> float:
        ms = c_float(0)
        _check(lib().candy_hip_quantize_sweep(self.handle, x_buf.ptr, x_stride, n_x, rows, cols, out_buf.ptr, n_out,
                                              iters, byref(ms)))
        return ms.value

    def stream_probe(self, bytes_per_launch: int, span_bytes: int, iters: int) -> float:
        """Elapsed milliseconds of `iters` read-only launches (0 bytes: empty kernels)."""
        ms = c_float(0)
        _check(lib().candy_hip_stream_probe(self.handle, bytes_per_launch, span_bytes, iters, byref(ms)))
        return ms.value

    def launch_probe(self, kind: int, iters: int) -> float:
        """Elapsed milliseconds of `iters` launches of an empty kernel (kind 0: one wavefront, 1: 1024 workgroups) or
        of a kernel whose wavefronts issue one load each (2: cache-warm, 3: cold)."""
        ms = c_float(0)
        _check(lib().candy_hip_launch_probe(self.handle, kind, iters, byref(ms)))
        return ms.value

    def timer_start(self):
        _check(lib().candy_hip_timer_start(self.handle))

    def timer_stop(self) -> float:
        ms = c_float(0)
        _check(lib().candy_hip_timer_stop(self.handle, byref(ms)))
        return ms.value


class Decoder:
    """Any decoder of the library: one sequence in its cache, fed token by token or in portions.

    Subclasses create the model and set `self.handle` to its decoder handle, `self.width`, `self.vocab`, `self.max_pos`."""

    handle = None

    def free(self):
        if self.handle is not None and self.dev.handle is not None:
            _check(lib().candy_hip_decoder_free(self.handle))
        self.handle = None

    def __del__(self):
        try:
            self.free()
        except Exception:
            pass

    def set_graph(self, enable: bool):
        _check(lib().candy_hip_decoder_set_graph(self.handle, int(enable)))

    def kv_cache(self):
        k, v, n = c_void_p(), c_void_p(), c_size_t()
        _check(lib().candy_hip_decoder_kv_cache(self.handle, byref(k), byref(v), byref(n)))
        return k.value, v.value, n.value

    def hidden(self) -> np.ndarray:
        """The residual stream as the last decode step left it behind the last layer (before the final norm)."""
        p = c_void_p()
        _check(lib().candy_hip_decoder_hidden(self.handle, byref(p)))
        return self._download(p.value, self.width)

    def prompt_hidden(self, n_tokens: int) -> np.ndarray:
        """The residual stream of the last prompt pass's first n_tokens tokens behind the last layer."""
        p, ld = c_void_p(), c_int64()
        _check(lib().candy_hip_decoder_prompt_hidden(self.handle, byref(p), byref(ld)))
        return self._download(p.value, n_tokens * ld.value).reshape(n_tokens, ld.value)[:, :self.width].copy()

    def decode(self, token: int, pos: int, want_logits: bool = True):
        lg, nt = c_void_p(), c_int32(-1)
        _check(lib().candy_hip_decoder_decode(self.handle, token, pos, byref(lg), byref(nt)))
        return nt.value, self._download(lg.value, self.vocab) if want_logits else None

    def generate(self, token: int, pos: int, n_steps: int):
        """n_steps greedy steps without a host round trip between them; returns the chosen tokens."""
        out = (c_int32 * n_steps)()
        _check(lib().candy_hip_decoder_generate(self.handle, token, pos, n_steps, out))
        return [int(t) for t in out]

    def decode_hidden(self, hidden: np.ndarray, pos: int, want_logits: bool = True):
        buf = self.dev.from_numpy(np.ascontiguousarray(hidden, np.float32))
        lg, nt = c_void_p(), c_int32(-1)
        _check(lib().candy_hip_decoder_decode_hidden(self.handle, buf.ptr, pos, byref(lg), byref(nt)))
        return nt.value, self._download(lg.value, self.vocab) if want_logits else None

    def prefill(self, tokens, pos0: int = 0, want_logits: bool = True):
        """Batched prompt pass; returns (greedy next token, logits) of the last prompt token."""
        ids = (c_int32 * len(tokens))(*[int(t) for t in tokens])
        lg, nt = c_void_p(), c_int32(-1)
        _check(lib().candy_hip_decoder_prefill(self.handle, ids, len(tokens), pos0, byref(lg), byref(nt)))
        return nt.value, self._download(lg.value, self.vocab) if want_logits else None

    def feed(self, tokens, pos0: int = 0, want=()) -> np.ndarray:
        """The next tokens of the sequence, at positions pos0 ..; logits [len(want), vocab] of the chosen ones (counted
        from the first of `tokens`).  One token takes the decode step, more take the prompt pass."""
        want = [int(w) for w in want]
        if any(w < 0 or w >= len(tokens) for w in want):
            raise ValueError("a wanted place lies outside the tokens fed")
        if len(tokens) == 1:
            lg = c_void_p()
            _check(lib().candy_hip_decoder_decode(self.handle, int(tokens[0]), pos0, byref(lg), None))
            if not want:
                return np.empty((0, self.vocab), np.float32)
            return np.tile(self._download(lg.value, self.vocab), (len(want), 1))
        ids = (c_int32 * len(tokens))(*[int(t) for t in tokens])
        rows = (c_int32 * max(len(want), 1))(*want)
        lg = c_void_p()
        _check(lib().candy_hip_decoder_prefill_rows(self.handle, ids, len(tokens), pos0, rows, len(want), byref(lg)))
        return self._download(lg.value, len(want) * self.vocab).reshape(len(want), self.vocab) if want \
            else np.empty((0, self.vocab), np.float32)

    def greedy(self, prompt, n_steps: int):
        """The n_steps tokens greedy decoding appends to a prompt."""
        tok, _ = self.prefill(prompt, 0, want_logits=False)
        return [tok] + (self.generate(tok, len(prompt), n_steps - 1) if n_steps > 1 else [])

    def _download(self, ptr: int, count: int) -> np.ndarray:
        out = np.empty(count, np.float32)
        _check(lib().candy_hip_d2h(self.dev.handle, out.ctypes.data, ptr, out.nbytes))
        return out


class Llama(Decoder):
    """Llama-style decoder on the device (weights stay owned by the caller)."""

    def __init__(self, dev: Device, **cfg):
        self.dev = dev
        self.cfg = LlamaConfig(**cfg)
        h = c_void_p()
        _check(lib().candy_hip_llama_create(dev.handle, byref(self.cfg), byref(h)))
        self.model = h.value
        self.handle = lib().candy_hip_llama_decoder(self.model)
        self.width, self.vocab, self.max_pos = self.cfg.d_model, self.cfg.vocab, self.cfg.max_pos
        self._keep = []

    def set_qweight(self, which: int, layer: int, w: QTensor):
        self._keep.append(w)
        _check(lib().candy_hip_llama_set_qweight(self.model, which, layer, w.handle))

    def set_norm(self, which: int, layer: int, alpha: np.ndarray):
        buf = self.dev.from_numpy(np.ascontiguousarray(alpha, np.float32))
        self._keep.append(buf)
        _check(lib().candy_hip_llama_set_norm(self.model, which, layer, buf.ptr))

    def set_kv_f16(self, enable: bool):
        """fp16 KV cache (clears the cache); kv_cache() then reports half the bytes."""
        _check(lib().candy_hip_llama_set_kv_f16(self.model, int(enable)))


class _LayerModel(Decoder):
    """A decoder created from a configuration and a list of layers (weights stay owned by the caller, vectors are copied)."""

    NAME, LAYER = "", None

    def __init__(self, dev: Device, cfg, layers: list):
        self.dev, self.cfg = dev, cfg
        self.layers = (self.LAYER * len(layers))(*layers)
        h = c_void_p()
        _check(self._call("create")(dev.handle, byref(cfg), self.layers, byref(h)))
        self.model = h.value
        self.handle = self._call("decoder")(self.model)
        self.width, self.vocab, self.max_pos = cfg.d_model, cfg.vocab, cfg.max_pos
        self._keep = []

    def _call(self, what: str):
        return getattr(lib(), f"candy_hip_{self.NAME}_{what}")

    def set_matrix(self, which: int, layer: int, w: Dense):
        self._keep.append(w)
        _check(self._call("set_matrix")(self.model, which, layer, w.handle))

    def set_vector(self, which: int, layer: int, values: np.ndarray):
        v = np.ascontiguousarray(values, np.float32).reshape(-1)
        _check(self._call("set_vector")(self.model, which, layer, v.ctypes.data, v.size))


class Suvazen(_LayerModel):
    """Suvazen decoder on the device (candy_amd/suvazen.py builds one from a model folder)."""

    NAME, LAYER = "suvazen", SuvazenLayer


class Gulisun(_LayerModel):
    """Gulisun decoder on the device (candy_amd/gulisun.py builds one from a model folder)."""

    NAME, LAYER = "gulisun", GulisunLayer
