"""ctypes binding of the kernel library: argument types, error translation.

The library is loaded (and, if need be, compiled) at the first use of ``lib()``.
There is no fallback: if it cannot be built or loaded, the caller gets the error.
"""

from __future__ import annotations

import ctypes
from ctypes import c_float, c_int, c_long, c_void_p

from pyre_amd.hip import build as _build

ABI_VERSION = 30


class KernelError(RuntimeError):
    """A kernel entry point refused its arguments or failed to launch."""


P, I, L, F = c_void_p, c_int, c_long, c_float

_SIGNATURES = {
    "pyre_read_probe": [P, ctypes.c_size_t, I, P, P],
    "pyre_embed": [P, I, P, P, P, I, P, I, I, F, P],
    "pyre_add_rmsnorm": [P, P, I, I, L, P, I, P, I, P, I, P, I, I, F, P],
    "pyre_rope_kv_write": [P, I, I, L, P, I, P, I, P, P, I, P, P, I, P, P, I, I, I, I, I, I, P],
    "pyre_silu_mul": [P, I, I, L, P, I, I, I, P],
    "pyre_reduce_partials": [P, I, I, L, P, I, P, I, I, I, P],
    "pyre_fill_rows": [P, I, L, I, I, L, P, I, ctypes.c_uint, P],
    "pyre_gemm_generic": [P, I, L, P, P, I, L, P, I, P, I, L, I, I, I, P],
    "pyre_gemm_f32": [P, L, P, L, P, I, P, L, L, I, I, I, I, P],
    "pyre_attn_generic": [P, P, I, P, P, I, P, P, P, P, I, I, I, I, I, I, F, I, I, P, I, P],
    "pyre_attn_generic_spans": [I],
    "pyre_attn_prefill_f32": [P, P, P, P, P, I, P, P, P, I, I, I, I, I, F, I, P],
    "pyre_attn_mfma_supports": [I, I, I, I],
    "pyre_attn_decode_work_bf16": [P, P, P, P, P, I, P, P, P, I, P, P, P, I, I, I, I, I, F, I, P],
    "pyre_attn_decode_work_rope_supports": [I, I, I, I, L],
    "pyre_attn_decode_work_rope_bf16": [P, I, L, P, I, P, P, P, I, I, P, P, P, P, I, P, P, P, I, P, P, P, I, I, I, I, I, F, I, P],
    "pyre_attn_prefill_bf16": [P, P, P, P, P, I, P, P, P, I, I, I, I, I, F, I, P],
    "pyre_attn_prefill_waves": [I, I],
    "pyre_attn_prefill_work_bf16": [P, P, P, P, P, I, P, P, I, P, P, P, I, I, I, I, I, F, I, P],
    "pyre_argmax": [P, L, P, P, I, I, P],
    "pyre_argmax_static": [P, L, P, I, I, P],
    "pyre_argmax_static_init": [],
    "pyre_compute_units": [],
    "pyre_gemm_skinny_supports": [I, I, I, L, L],
    "pyre_gemm_skinny_bf16": [P, L, P, L, P, I, I, I, I, P],
    "pyre_gemm_skinny_silu_bf16": [P, L, P, L, P, I, I, I, P],
    "pyre_gemm_mid_supports": [I, I, I, L, L],
    "pyre_gemm_mid_bf16": [P, L, P, L, P, I, I, I, I, I, P],
    "pyre_gemm_mid_silu_blocks": [I, I],
    "pyre_gemm_mid_silu_bf16": [P, L, P, L, P, I, I, I, P],
    "pyre_sample": [P, L, P, P, P, I, I, P],
    "pyre_feed_tokens": [P, P, P, I, P],
    "pyre_gemm_skinny_glu_bf16": [P, L, P, L, P, I, I, I, F, F, F, F, P],
    "pyre_gemm_mid_glu_bf16": [P, L, P, L, P, I, I, I, F, F, F, F, P],
    "pyre_add_layernorm": [P, P, I, I, L, P, I, P, I, P, I, F, P, P, I, P, I, P, I, I, F, P],
    "pyre_clipped_glu": [P, I, I, L, P, I, I, I, F, F, F, F, P],
    "pyre_scale": [P, L, F, P],
    "pyre_stream_norm": [P, I, P, I, P, I, I, L, P, P, P, P, P, I, F, P, I, P, I, I, P],
    "pyre_poly_norm": [P, I, I, L, P, F, P, I, I, I, P],
    "pyre_unit_qkv_write": [P, I, I, L, I, I, P, I, P, P, I, P, P, I, I, I, I, I, I, I, F, I, P],
    "pyre_attn_biased_tile": [P, P, I, I, P, P, P, F, P, I, P, P, P, I, I, I, I, I, I, F, F, P, I, I, I, I, P, I, P, I, I, P],
    "pyre_attn_biased_single": [P, P, I, I, P, P, P, F, P, I, P, P, P, I, I, I, I, I, I, F, F, P, I, I, I, I, P, I, P, I, P],
    "pyre_attn_biased_spans": [I, I, I, I],
    "pyre_gla_prepare": [P, I, I, L, I, I, P, I, P, I, F, P, I, I, I, I, I, P],
    "pyre_gla_scan": [P, P, P, P, P, I, I, I, I, F, P, P],
    "pyre_gla_chunks": [P, P, P, P, P, P, I, I, I, I, I, I, F, P],
    "pyre_gla_chunks_scratch": [I, I, I, I, I],
    "pyre_gla_finish": [P, P, P, I, F, F, P, I, I, I, I, I, I, P],
    "pyre_add_tanhnorm": [P, P, I, I, L, P, I, F, P, I, I, L, P, I, F, P, P, P, I, P, I, P, I, I, P],
    "pyre_softcap": [P, L, F, P],
    "pyre_rope_tied_write": [P, I, I, L, I, I, P, I, P, I, P, P, I, P, P, I, P, P, I, I, I, I, I, I, P],
    "pyre_latent_rows": [P, I, I, L, I, I, P, P, I, P, I, I, I, I, I, I, P, P, P, I, P, P, P, I, I, P, F, I, P],
    "pyre_head_matmul": [P, L, L, P, P, L, L, P, I, I, I, I, I, P],
    "pyre_latent_attn_tile": [P, P, P, I, P, I, P, P, P, I, I, I, I, I, F, I, P, P],
    "pyre_latent_attn_spans": [I, I],
    "pyre_latent_attn_single": [P, P, P, I, P, I, P, P, P, I, I, I, I, I, F, I, P, P, P],
    "pyre_route_topk": [P, I, I, L, P, I, P, I, I, I, I, I, P],
    "pyre_expert_act": [P, I, I, L, P, P, I, I, I, I, I, P],
    "pyre_add_rms_terms": [P, P, I, I, L, P, I, F, P, I, I, L, P, I, F, F, P, I, F, P, I, F, P, I, P, I, I, P],
    "pyre_bigram_embed": [P, P, I, P, P, P, P, P, P, P, I, P, I, I, I, I, I, P],
    "pyre_conv_qkv_write": [P, I, I, L, I, I, P, I, P, P, P, P, I, P, P, F, P, P, I, I, P, P, I, P, P, I, P, P, I, I, I, I,
                            I, I, I, I, P],
    "pyre_retention_prepare": [P, I, I, L, I, I, P, P, P, I, I, P, F, I, P, I, I, I, I, P],
    "pyre_gla_finish_wide": [P, P, P, I, F, F, P, I, L, I, I, I, I, P],
    "pyre_ssm_conv": [P, I, I, L, I, I, P, P, I, P, P, P, P, P, I, I, P, I, I, I, P],
    "pyre_ssm_low": [P, I, I, L, I, P, I, I, I, I, P],
    "pyre_ssm_scan": [P, I, I, L, P, P, I, P, I, I, L, I, I, P, I, I, L, I, P, I, P, P, P, P, P, I, F, P, I, L, I, I, P],
    "pyre_ssm_step": [P, I, L, P, P, I, P, I, I, L, I, I, P, I, I, L, I, P, I, P, P, P, P, I, F, P, I, L, I, I, P],
    "pyre_route_grouped": [P, I, I, L, P, I, P, P, I, I, I, I, I, P],
    "pyre_expert_glu_act": [P, I, I, L, P, L, P, I, I, I, I, I, I, P],
    "pyre_add_weighted_rows": [P, P, I, L, P, L, I, I, I, I, P],
    "pyre_wide_norm_qkv_write": [P, I, I, L, I, I, P, P, P, F, P, P, I, P, P, I, P, P, I, P, I, I, I, I, I, I, I, P],
    "pyre_gdr_prepare": [P, I, I, L, I, I, P, P, I, P, P, P, P, I, P, I, P, P, P, I, F, P, I, I, I, I, I, I, I, P],
    "pyre_gdr_scan": [P, P, P, P, P, I, I, I, I, I, I, P],
    "pyre_gdr_finish": [P, P, P, I, F, F, P, I, L, I, I, I, I, I, P],
    "pyre_token_side_gate": [P, I, I, L, P, I, P, I, I, I, P, P, I, I, I, P],
}

_lib = None


def _open(path) -> ctypes.CDLL:
    handle = ctypes.CDLL(str(path))
    handle.pyre_last_error.restype = ctypes.c_char_p
    handle.pyre_abi_version.restype = c_int
    return handle


def _fits(handle) -> bool:
    """The library speaks this binding's ABI and was compiled from the sources of this tree."""
    if handle.pyre_abi_version() != ABI_VERSION or not hasattr(handle, "pyre_sources_digest"):
        return False
    handle.pyre_sources_digest.restype = ctypes.c_char_p
    return handle.pyre_sources_digest().decode() == _build.sources_digest()


def lib() -> ctypes.CDLL:
    global _lib
    if _lib is None:
        handle = _open(_build.ensure_built())
        if not _fits(handle):
            # A library from other sources under a stamp that says otherwise (a copied build
            # folder, an older checkout): rebuild once. The loader keeps the mapping of a path
            # it has already opened, so the new build is opened under a name of its own.
            import os
            import shutil

            path = _build.build(force=True)
            fresh = path.with_name(f"{path.stem}.{os.getpid()}{path.suffix}")
            shutil.copyfile(path, fresh)
            try:
                handle = _open(fresh)
            finally:
                os.unlink(fresh)
            if not _fits(handle):
                raise KernelError(f"kernel library has ABI {handle.pyre_abi_version()} and the binding expects "
                                  f"{ABI_VERSION}, or it does not carry the digest of the sources it was built "
                                  "from: sources and binding are out of step")
        for name, argtypes in _SIGNATURES.items():
            fn = getattr(handle, name)
            fn.argtypes = argtypes
            fn.restype = c_int
        _lib = handle
    return _lib


def loaded_path() -> str | None:
    return None if _lib is None else _lib._name


_entry_points: dict = {}


def call(name: str, *args) -> None:
    fn = _entry_points.get(name)
    if fn is None:
        fn = _entry_points[name] = getattr(lib(), name)
    if fn(*args) != 0:
        raise KernelError(lib().pyre_last_error().decode(errors="replace"))
