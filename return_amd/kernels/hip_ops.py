"""The kernel set of the engine: thin, checked bindings of the HIP library.

Every method checks on the host that shapes, dtypes and contiguity are what the
kernel and its grid assume, and raises before anything is launched otherwise.
There is no other implementation behind these names: if the library cannot be
built or loaded, constructing HipOps raises.
"""
from __future__ import annotations

import ctypes
from typing import Optional

import torch

from ..parts.runtime import RowSums, ScaledRows, Slabs
from . import build as _build

_F32, _BF16 = 0, 1
_c_int, _c_ll, _c_float, _c_ptr = ctypes.c_int, ctypes.c_longlong, ctypes.c_float, ctypes.c_void_p


class KernelError(RuntimeError):
    pass


def _code(dtype: torch.dtype) -> int:
    if dtype == torch.float32:
        return _F32
    if dtype == torch.bfloat16:
        return _BF16
    raise KernelError(f"kernels take float32 or bfloat16 tensors, got {dtype}")


_LIB = None


def load_library():
    """The HIP library, built first if it is not there. Raises if that is impossible."""
    global _LIB
    if _LIB is None:
        path = _build.ensure_built()
        try:
            _LIB = ctypes.CDLL(path)
        except OSError as e:
            raise KernelError(f"cannot load the HIP library {path}: {e}") from e
        _declare(_LIB)
    return _LIB


def _declare(lib):
    P, I, L, F = _c_ptr, _c_int, _c_ll, _c_float
    sigs = {
        "ra_embed": [P, P, P, I, I, I, I, P],
        "ra_embed_scaled": [P, P, P, I, I, I, I, F, P],
        "ra_post_norm_add": [P, P, P, F, P, F, P, I, I, I, P],
        "ra_depth_mix": [P, L, I, P, P, P, F, P, I, I, I, P],
        "ra_post_norm_mix": [P, L, I, P, P, P, F, P, P, F, P, I, I, I, P],
        "ra_heads_gate": [P, P, L, P, I, I, I, I, P],
        "ra_silu_mul_bias": [P, P, P, I, I, I, P],
        "ra_latent_kv_prepare": [P, L, I, I, I, I, P, P, F, P, P, P, I, P, P, P, P, I, P, L, I, I, P, I, P],
        "ra_latent_q_prepare": [P, P, I, I, I, I, I, P, P, P, I, P, I, P],
        "ra_attention_latent_plain": [P, P, P, P, P, P, P, P, P, P, I, I, I, I, I, I, I, F, P, I, I, P],
        "ra_attention_latent_plain_window": [P, P, P, P, P, P, P, P, P, P, I, I, I, I, I, I, I, F, P, I, I, I, P],
        "ra_attention_latent_mfma_window_bf16": [P, P, P, P, P, P, P, P, P, P, I, I, I, I, I, I, F, P, I, P, I, P],
        "ra_add_rmsnorm_pair": [P, P, P, P, F, P, P, F, P, I, I, I, P],
        "ra_qkv_blend_prepare": [P, L, I, I, I, I, P, P, P, I, F, P, P, P, I, P, P, P, P, I, L, P, I, I, F, I, P],
        "ra_gated_rows": [P, I, L, P, I, I, I, F, F, I, P],
        "ra_gate_rows": [P, L, P, L, I, I, I, P],
        "ra_qkv_rows_prepare": [P, L, I, I, I, I, P, P, I, I, F, P, P, P, I, P, P, P, P, I, L, I, P],
        "ra_causal_conv_bias": [P, L, P, P, P, P, P, P, P, L, I, I, I, I, I, I, P],
        "ra_scalar_rule": [P, L, P, L, P, L, P, P, P, P, I, F, P, P, P, P, P, I, I, I, I, I, I, I, I, P],
        "ra_attention_latent_plain_fits": [I, I],
        "ra_attention_latent_mfma_bf16": [P, P, P, P, P, P, P, P, P, P, I, I, I, I, I, I, F, P, I, P, P],
        "ra_attention_latent_mfma_fits": [I, I, I],
        "ra_attention_latent_mfma_tile_tokens": [I],
        "ra_outer_rule": [P, L, P, L, P, L, P, F, P, F, P, P, P, P, P, I, I, I, I, I, I, I, P],
        "ra_moe_route_law": [P, L, P, I, I, I, I, I, F, P, P, I, P],
        "ra_moe_product_act": [P, P, P, P, P, P, I, I, I, I, I, I, I, F, F, P, I, P],
        "ra_add_rmsnorm": [P, P, P, F, P, P, I, I, I, P],
        "ra_add_scaled_rmsnorm": [P, P, F, P, F, P, P, I, I, I, P],
        "ra_stream_pair_rows": [P, P, F, P, P, L, I, I, P],
        "ra_maps_qkv_prepare": [P, I, I, I, I, I, I, P, P, P, I, I, P, P, P, P, I, I, P],
        "ra_attention_diff_plain": [P, P, P, P, P, P, P, P, P, P, I, I, I, I, I, I, I, I, F, I, I, F, F, F, I, P],
        "ra_attention_diff_mfma_bf16": [P, P, P, P, P, P, P, P, P, P, I, I, I, I, I, I, F, I, I, F, F, F, I, P, I, P],
        "ra_attention_diff_mfma_fits": [I, I],
        "ra_attention_diff_plain_fits": [I, I],
        "ra_moe_route": [P, P, I, I, I, I, I, F, P, P, P],
        "ra_moe_plan": [P, I, I, I, P, P, P, P],
        "ra_moe_tile_rows": [I, I, I, I],
        "ra_moe_product": [P, P, P, P, P, P, I, I, I, I, I, I, I, P],
        "ra_moe_combine": [P, P, P, I, I, I, I, P],
        "ra_moe_combine_extra": [P, P, P, I, I, I, P, P, I, L, I, P],
        "ra_add_slabs_rmsnorm": [P, P, I, L, P, F, P, P, I, I, I, P],
        "ra_residual_add": [P, P, L, I, P],
        "ra_head_rmsnorm": [P, P, F, L, I, I, P],
        "ra_rope": [P, P, P, P, I, I, I, I, I, P],
        "ra_split_heads": [P, P, P, P, I, I, I, I, P],
        "ra_kv_write": [P, P, P, P, P, I, I, I, I, L, I, P],
        "ra_qkv_prepare": [P, I, I, I, I, P, P, F, P, P, P, I, P, P, P, P, I, L, I, P],
        "ra_silu_mul": [P, P, I, I, I, P],
        "ra_gemm_nt": [P, P, P, I, I, I, I, I, P],
        "ra_gemm_skinny_bf16": [P, P, P, I, I, I, I, I, P],
        "ra_gemm_skinny_gated_bf16": [P, P, P, I, I, I, P],
        "ra_gemm_mfma_bf16": [P, P, P, I, I, I, I, P],
        "ra_gemm_resident_bf16": [P, P, P, I, I, I, I, I, I, P],
        "ra_gemm_resident_fits": [I, I, I],
        "ra_gemm_sweep_bf16": [P, P, P, I, I, I, I, I, I, P],
        "ra_gemm_sweep_fits": [I, I],
        "ra_gemm_sweep_workgroups": [I, I],
        "ra_gemm_sweep_norm_bf16": [P, P, P, I, I, I, I, I, I, P, I, I, F, P, P, P, P],
        "ra_attention_plain": [P, P, P, P, P, P, P, P, P, P, I, I, I, I, I, I, F, I, I, P, F, I, I, P, F, L, P],
        "ra_causal_conv": [P, L, P, P, P, P, P, L, I, I, I, I, I, I, P],
        "ra_delta_rule": [P, L, P, L, P, L, P, P, P, F, P, P, P, P, P, I, I, I, I, I, I, I, I, P],
        "ra_delta_rule_head": [P, L, P, L, P, L, P, L, P, P, P, F, P, P, P, P, P, I, I, I, I, I, I, I, I, P],
        "ra_channel_recurrence": [P, P, P, P, P, L, P, P, P, P, P, F, P, L, I, I, I, I, I, I, I, P],
        "ra_channel_recurrence_chunk": [I],
        "ra_channel_recurrence_mfma": [I, I, I],
        "ra_layer_norm_add": [P, P, P, F, P, I, I, I, P],
        "ra_stream_layer_norm": [P, P, P, I, P, P, P, L, P, P, F, P, P, I, I, I, P],
        "ra_stream_rows": [P, P, L, I, P],
        "ra_softcap": [P, F, L, P],
        "ra_delta_rule_fits": [I, I],
        "ra_token_side": [P, P, P, P, L, I, P, P, P, F, I, I, I, I, P],
        "ra_relu_sq": [P, L, I, P],
        "ra_add_bias": [P, P, L, I, I, P],
        "ra_qk_prepare": [P, I, I, I, I, P, P, P, P, I, P, P, P, P, I, L, I, P],
        "ra_attention_decode_bf16": [P, P, P, P, P, P, P, P, P, P, P, P, I, I, I, I, I, F, I, I, I, I, P],
        "ra_attention_decode_extras_bf16": [P, P, P, P, P, P, P, P, P, P, P, P, I, I, I, I, I, F, I, I, I, I, P, F, I, I, P, F, L, I,
                                            P],
        "ra_attention_decode_fused_bf16": [P, P, P, P, P, P, P, P, P, P, P, P, I, I, I, I, I, F, I, I, I, P, P, F, P, P, I, P],
        "ra_attention_decode_static_bf16": [P, P, P, P, P, P, P, P, P, P, I, I, I, I, I, F, I, I, I, I, P],
        "ra_attention_decode_merge_waves": [I],
        "ra_attention_prefill_bf16": [P, P, P, P, P, P, P, P, P, P, I, I, I, I, I, I, I, F, I, P, F, I, I, P, F, L, I, P],
        "ra_attention_prefill_tile_rows": [I],
        "ra_sample": [P, I, I, P, P, P, P, P, P],
        "ra_sample_traced": [P, I, I, P, P, P, P, P, P, P],
        "ra_stream_read": [P, L, P, I, P],
    }
    for name, args in sigs.items():
        fn = getattr(lib, name)
        fn.argtypes = args
        fn.restype = _c_int


def _ptr(t: Optional[torch.Tensor]):
    return None if t is None else t.data_ptr()


# What tune_products has measured in this process: (row step, N, K, gated, result dtype) -> the way that
# beat the rule's, or None where the rule stands. Every kernel set that tunes gets the same answers.
_PRODUCTS_MEASURED = {}
_PRODUCT_TIMES = {}        # the same keys -> {way: seconds}, as measured
_NORM_PAIRS_MEASURED = {}  # (row step, shape of the product before a norm, of the one after, gated) -> the norm inside them is faster


class HipOps:
    def __init__(self, device="cuda:0"):
        self.device = torch.device(device)
        if self.device.type != "cuda":
            raise KernelError(f"the HIP kernels run on a GPU, not on {self.device}")
        if not torch.cuda.is_available():
            raise KernelError("no GPU is visible to this process")
        self.lib = load_library()
        # float32 products must be true 32-bit wherever a library routine is used
        torch.backends.cuda.matmul.allow_tf32 = False
        torch.backends.cudnn.allow_tf32 = False
        self.decode_split_tokens = 0         # keys per split of the decode attention; 0: by batch size
        # a request's splits as one workgroup that merges them itself: one such workgroup fills a CU
        # (LDS), so it pays when the (request, kv head) pairs come to whole rounds over the CUs
        self.cu_count = torch.cuda.get_device_properties(self.device).multi_processor_count
        self.decode_merge_round = self.cu_count
        self.decode_merge_waves = 0          # waves of such a workgroup; 0: by the number of pairs and the context
        self.prefill_key_split = 0           # groups of waves that share a q tile's keys (1 or 2); 0: by the number of tiles
        self.prefill_small_tiles = True      # q tiles of 64 rows instead of 128 while those would not fill the chip
        self.overlap_attention = True        # mixed steps: the decode and the prefill attention side by side on two streams
        self._side_stream = None
        self.skinny_max_grid = 0             # 0: one workgroup per 16 weight rows
        self.gated_skinny_rows = 8           # up to this many rows gate-up and SiLU-mul are one kernel
        self.own_gemm = False                # True: bf16 products of many rows use the hand-written MFMA kernel
        self.defer_norms = True              # finish RMSNorms inside the products around them where the sweep takes both
        try:                                 # whether the library multiplies bf16 operands into fp32 results
            a = torch.ones(1, 8, dtype=torch.bfloat16, device=self.device)
            self._library_fp32_out = torch.mm(a, a.t(), out_dtype=torch.float32).dtype == torch.float32
        except (TypeError, RuntimeError):
            self._library_fp32_out = False
        try:                                 # and the same for a batch of products
            a = torch.ones(2, 1, 8, dtype=torch.bfloat16, device=self.device)
            self._library_bmm_fp32 = torch.bmm(a, a.transpose(1, 2).contiguous(), out_dtype=torch.float32).dtype == torch.float32
        except (TypeError, RuntimeError):
            self._library_bmm_fp32 = False
        # whether the library's float32 product is a true 32-bit one (against a 64-bit product; operands
        # rounded to a shorter mantissa would be off by 1e-3)
        g = torch.Generator(device="cpu").manual_seed(0)
        a = torch.randn(32, 512, generator=g).to(self.device)
        b = torch.randn(48, 512, generator=g).to(self.device)
        want = a.double() @ b.double().t()
        self._library_fp32_exact = bool(((torch.matmul(a, b.t()).double() - want).abs().max()
                                         <= 2e-5 * want.abs().max()).item())
        self._unit_tiles = self._make_unit_tiles(1024)    # (i, 0) for i = 0, 1, ...: q tiles of requests that bring one token each
        self.product_plan = {}               # (row step, N, K, gated, result dtype) -> way, where measured faster than the rule
        self._measured = _PRODUCTS_MEASURED
        self._times = _PRODUCT_TIMES
        self._defer = {}                     # as _NORM_PAIRS_MEASURED, for the pairs this kernel set has been shown

    def _make_unit_tiles(self, n):
        t = torch.zeros(n, 2, dtype=torch.int32, device=self.device)
        t[:, 0] = torch.arange(n, dtype=torch.int32, device=self.device)
        return t

    def use_skinny(self, M, N, K, out_dtype):
        """Whether the hand-written skinny product beats the library for x [M, K] @ W[N, K]^T
        (measured on MI355X: it wins for one to four rows, up to 16 rows on small weights and up
        to 32 rows on the smallest)."""
        if K % 8 or M > 64:
            return False
        if out_dtype == torch.float32:
            return M <= 16                   # more rows: the library, or the tiled MFMA product
        return M <= 4 or (M <= 16 and N * K <= (32 << 20)) or (M <= 32 and N * K <= (16 << 20))

    def use_sweep(self, M, N, K, gated):
        """Whether the product that reads W as one sweep through memory (one workgroup per CU, column
        c with workgroup c % CUs) is the rule's choice for x [M, K] and N result columns. Measured on
        MI355X at 1 to 16 rows: 12 against 15 µs (q/k/v of the 8B shape), 10 against 11 (o), 36 against
        41 (gate-up), 100 against 118 (gate-up of the 32B shape, K = 5,120) for the x-resident and
        skinny products; on the output head's 152 thousand rows the x-resident product is ahead (two
        workgroups per CU hide each other's tile ends), and on few rows of many columns (down: one tile
        a workgroup, K = 12,288) the library."""
        if not self.lib.ra_gemm_sweep_fits(M, K):
            return False
        if M > 16 and not gated:             # 17 to 32 rows: 41 to 44 µs against the library's 49 and the SiLU-mul's 5
            return False                     # for gate-up, but q/k/v 17 to 19 against 15, o 14 to 16 against 13
        rows = N * (2 if gated else 1)
        least = 8 if K <= 4096 or M <= 2 else 32         # rows a workgroup, at least (down at 1 and 2 rows: 20 against 21 to 23 µs)
        return least * self.cu_count <= rows <= 256 * self.cu_count

    def use_resident(self, M, N, K, gated):
        """Whether the product with x resident in LDS beats the skinny product for x [M, K] and
        N result columns (measured on MI355X): when there are tiles of 16 columns enough for
        every workgroup (two per CU); few tiles are the skinny product's."""
        if not self.lib.ra_gemm_resident_fits(M, K, 1 if gated else 0):
            return False
        tiles = -(-N // 16)
        if 1 <= M <= 8:
            return tiles >= 384
        return M > 8 and tiles >= 2048

    # ------------------------------------------------------------------ helpers
    def _stream(self):
        return torch.cuda.current_stream(self.device).cuda_stream

    def _check(self, status: int, name: str):
        if status != 0:
            why = {1: "arguments outside what the kernel takes", 2: "launch failed",
                   3: "more partial results than the library's own buffer holds",
                   4: "the library's own buffer was not found on this device"}.get(status, "?")
            raise KernelError(f"{name}: {why} (status {status})")

    def _want(self, t, name, dtype=None, dims=None):
        if t.device != self.device:
            raise KernelError(f"{name} is on {t.device}, kernels run on {self.device}")
        if not t.is_contiguous():
            raise KernelError(f"{name} must be contiguous")
        if dtype is not None and t.dtype != dtype:
            raise KernelError(f"{name} must be {dtype}, got {t.dtype}")
        if dims is not None and t.dim() != dims:
            raise KernelError(f"{name} must have {dims} dimensions, got shape {tuple(t.shape)}")

    # ------------------------------------------------------------------ rows
    def embed(self, table, ids, out, scale=1.0):
        """out[t] = table[ids[t]] * scale (the product in 32-bit)."""
        self._want(table, "embedding table", dims=2)
        self._want(ids, "token ids", torch.int32, 1)
        self._want(out, "embedding output", torch.float32, 2)
        T, H = out.shape
        if ids.shape[0] != T or table.shape[1] != H:
            raise KernelError(f"embed: ids {tuple(ids.shape)}, table {tuple(table.shape)}, out {tuple(out.shape)}")
        self._check(self.lib.ra_embed_scaled(_ptr(table), _ptr(ids), _ptr(out), T, H, table.shape[0],
                                             _code(table.dtype), float(scale), self._stream()), "embed")

    def post_norm_add(self, h, y, weight, eps, next_weight=None, next_eps=0.0, out=None):
        """h += y / sqrt(mean(y^2) + eps) * weight, row by row, in 32-bit; with next_weight also
        out = h / sqrt(mean(h^2) + next_eps) * next_weight (the norm in front of the next sublayer)."""
        self._want(h, "residual stream", torch.float32, 2)
        self._want(y, "sublayer output", dims=2)
        self._want(weight, "norm weight", torch.float32, 1)
        R, H = h.shape
        if tuple(y.shape) != (R, H) or weight.shape[0] != H:
            raise KernelError(f"post_norm_add: h {tuple(h.shape)}, y {tuple(y.shape)}, weight {tuple(weight.shape)}")
        if next_weight is not None:
            self._want(next_weight, "next norm weight", torch.float32, 1)
            self._want(out, "norm output", y.dtype, 2)
            if next_weight.shape[0] != H or tuple(out.shape) != (R, H):
                raise KernelError(f"post_norm_add: next weight {tuple(next_weight.shape)}, out {tuple(out.shape)}")
        self._check(self.lib.ra_post_norm_add(_ptr(h), _ptr(y), _ptr(weight), float(eps), _ptr(next_weight), float(next_eps),
                                              _ptr(out) if next_weight is not None else None, R, H, _code(y.dtype),
                                              self._stream()), "post_norm_add")

    def depth_mix(self, results, count, weights, out, norm_weight=None, eps=0.0, normed=None):
        """out = sum_{j < count} weights[j] * results[j] (32-bit, terms in order); results fp32 [n, T, H], out fp32
        [T, H], which may be a later row of results; with norm_weight also normed = rmsnorm(out) * norm_weight."""
        self._want(results, "results", torch.float32, 3)
        self._want(weights, "mix weights", torch.float32, 1)
        self._want(out, "stream", torch.float32, 2)
        n, R, H = results.shape
        if not 1 <= count <= n or weights.shape[0] != count or tuple(out.shape) != (R, H) or count > 256:
            raise KernelError(f"depth_mix: {count} of results {tuple(results.shape)}, weights {tuple(weights.shape)}, "
                              f"out {tuple(out.shape)}")
        lo, hi = results.data_ptr(), results.data_ptr() + count * R * H * 4
        if lo <= out.data_ptr() < hi:
            raise KernelError("depth_mix: the output lies among the terms of the sum")
        code = _F32
        if norm_weight is not None:
            self._want(norm_weight, "norm weight", torch.float32, 1)
            self._want(normed, "norm output", dims=2)
            if norm_weight.shape[0] != H or tuple(normed.shape) != (R, H):
                raise KernelError(f"depth_mix: norm weight {tuple(norm_weight.shape)}, normed {tuple(normed.shape)}")
            code = _code(normed.dtype)
        self._check(self.lib.ra_depth_mix(_ptr(results), R * H, int(count), _ptr(weights), _ptr(out), _ptr(norm_weight),
                                          float(eps), _ptr(normed) if norm_weight is not None else None, R, H, code,
                                          self._stream()), "depth_mix")

    def post_norm_mix(self, results, count, weights, y, weight, eps, out, norm_weight=None, norm_eps=0.0, normed=None):
        """post_norm_add(results[count - 1], y, weight, eps) and depth_mix(results, count, weights, out, ...) in one pass
        over a row (the same bits as the two one after the other)."""
        n, R, H = results.shape
        if H > 4096:                                     # rows that a thread cannot keep: the two kernels
            self.post_norm_add(results[count - 1], y, weight, eps)
            return self.depth_mix(results, count, weights, out, norm_weight, norm_eps, normed)
        self._want(results, "results", torch.float32, 3)
        self._want(weights, "mix weights", torch.float32, 1)
        self._want(out, "stream", torch.float32, 2)
        self._want(y, "sublayer output", dims=2)
        self._want(weight, "norm weight", torch.float32, 1)
        if not 1 <= count <= n or weights.shape[0] != count or tuple(out.shape) != (R, H) or count > 256 \
                or tuple(y.shape) != (R, H) or weight.shape[0] != H:
            raise KernelError(f"post_norm_mix: {count} of results {tuple(results.shape)}, weights {tuple(weights.shape)}, "
                              f"out {tuple(out.shape)}, y {tuple(y.shape)}, norm weight {tuple(weight.shape)}")
        lo, hi = results.data_ptr(), results.data_ptr() + count * R * H * 4
        if lo <= out.data_ptr() < hi:
            raise KernelError("post_norm_mix: the output lies among the terms of the sum")
        if norm_weight is not None:
            self._want(norm_weight, "next norm weight", torch.float32, 1)
            self._want(normed, "norm output", y.dtype, 2)
            if norm_weight.shape[0] != H or tuple(normed.shape) != (R, H):
                raise KernelError(f"post_norm_mix: norm weight {tuple(norm_weight.shape)}, normed {tuple(normed.shape)}")
        self._check(self.lib.ra_post_norm_mix(_ptr(results), R * H, int(count), _ptr(weights), _ptr(y), _ptr(weight),
                                              float(eps), _ptr(out), _ptr(norm_weight), float(norm_eps),
                                              _ptr(normed) if norm_weight is not None else None, R, H, _code(y.dtype),
                                              self._stream()), "post_norm_mix")

    def heads_gate(self, o, gate, out):
        """o [H, T, Dv] (a product batched over heads), gate [T, H] logits (a column slice of wider rows, or None)
        -> out [T, H * Dv] = o * sigmoid(gate), head by head."""
        self._want(o, "heads", dims=3)
        self._want(out, "gated heads", o.dtype, 2)
        Hn, T, Dv = o.shape
        if tuple(out.shape) != (T, Hn * Dv):
            raise KernelError(f"heads_gate: o {tuple(o.shape)}, out {tuple(out.shape)}")
        ld = 0
        if gate is not None:
            ld = self._want_rows(gate, "head gates", o.dtype)
            if tuple(gate.shape) != (T, Hn):
                raise KernelError(f"heads_gate: gate {tuple(gate.shape)} for {T} tokens of {Hn} heads")
        self._check(self.lib.ra_heads_gate(_ptr(o), _ptr(gate), ld, _ptr(out), T, Hn, Dv, _code(o.dtype), self._stream()),
                    "heads_gate")

    def batched_product(self, a, b, out=None):
        """[B, M, K] x [B, K, N] -> [B, M, N] in a's dtype, by the library (32-bit operands: a true 32-bit product). out:
        where the result goes (rows of N elements side by side, apart by any distance: the rows of all b's batches may be
        columns of the same wider rows); None: a new tensor."""
        if a.dim() != 3 or b.dim() != 3 or a.shape[0] != b.shape[0] or a.shape[2] != b.shape[1] or a.dtype != b.dtype \
                or not b.is_contiguous():
            raise KernelError(f"batched_product: {tuple(a.shape)} x {tuple(b.shape)}")
        if out is None:
            return torch.bmm(a, b)
        if tuple(out.shape) != (a.shape[0], a.shape[1], b.shape[2]) or out.dtype != a.dtype or (out.shape[2] > 1 and out.stride(2) != 1):
            raise KernelError(f"batched_product: {tuple(a.shape)} x {tuple(b.shape)} into {tuple(out.shape)}, strides {out.stride()}")
        return torch.bmm(a, b, out=out)

    def add_rmsnorm(self, h, delta, weight, eps, out, rows=None, delta_scale=1.0):
        """h += delta_scale * delta (in place, unless a row list is given); out = norm(h) * weight."""
        self._want(h, "residual stream", torch.float32, 2)
        self._want(weight, "norm weight", torch.float32, 1)
        self._want(out, "norm output", dims=2)
        R, H = h.shape
        if weight.shape[0] != H or out.shape[1] != H:
            raise KernelError(f"add_rmsnorm: h {tuple(h.shape)}, weight {tuple(weight.shape)}, out {tuple(out.shape)}")
        if isinstance(delta, Slabs):
            self._want(delta.tensor, "shares of the product", torch.float32, 3)
            if tuple(delta.tensor.shape[1:]) != (R, H):
                raise KernelError(f"add_rmsnorm: shares {tuple(delta.tensor.shape)} do not match h {tuple(h.shape)}")
            if float(delta_scale) != 1.0:
                raise KernelError("add_rmsnorm: shares of a product are added as they are, not times a factor")
            if rows is not None:
                self._want(rows, "row list", torch.int32, 1)
            M = R if rows is None else rows.shape[0]
            if out.shape[0] != M:
                raise KernelError(f"add_rmsnorm: out has {out.shape[0]} rows, {M} wanted")
            self._check(self.lib.ra_add_slabs_rmsnorm(_ptr(h), _ptr(delta.tensor), delta.tensor.shape[0], R, _ptr(weight),
                                                      float(eps), _ptr(out), _ptr(rows), M, H, _code(out.dtype),
                                                      self._stream()), "add_slabs_rmsnorm")
            return
        if delta is not None:
            self._want(delta, "delta", out.dtype, 2)
            if tuple(delta.shape) != (R, H):
                raise KernelError(f"add_rmsnorm: delta {tuple(delta.shape)} does not match h {tuple(h.shape)}")
        if rows is not None:
            self._want(rows, "row list", torch.int32, 1)
            M = rows.shape[0]
        else:
            M = R
        if out.shape[0] != M:
            raise KernelError(f"add_rmsnorm: out has {out.shape[0]} rows, {M} wanted")
        if float(delta_scale) != 1.0:
            self._check(self.lib.ra_add_scaled_rmsnorm(_ptr(h), _ptr(delta), float(delta_scale), _ptr(weight), float(eps),
                                                       _ptr(out), _ptr(rows), M, H, _code(out.dtype), self._stream()),
                        "add_scaled_rmsnorm")
            return
        self._check(self.lib.ra_add_rmsnorm(_ptr(h), _ptr(delta), _ptr(weight), float(eps), _ptr(out),
                                            _ptr(rows), M, H, _code(out.dtype), self._stream()),
                    "add_rmsnorm")

    def residual_add(self, h, delta, scale=1.0):
        self._want(h, "residual stream", torch.float32)
        self._want(delta, "delta")
        if h.shape != delta.shape:
            raise KernelError(f"residual_add: {tuple(h.shape)} += {tuple(delta.shape)}")
        if float(scale) != 1.0:
            h.add_(delta, alpha=float(scale))            # (32-bit: the sum is formed in h's type)
            return
        self._check(self.lib.ra_residual_add(_ptr(h), _ptr(delta), h.numel(), _code(delta.dtype),
                                             self._stream()), "residual_add")

    def stream_pair_rows(self, h, delta, delta_scale, h0, out):
        """h += delta_scale * delta (delta may be None); out [T, 2H] = [h | h0] in out's type."""
        self._want(h, "residual stream", torch.float32, 2)
        self._want(h0, "first stream", torch.float32, 2)
        self._want(out, "rows", dims=2)
        T, H = h.shape
        if h0.shape != h.shape or tuple(out.shape) != (T, 2 * H):
            raise KernelError(f"stream_pair_rows: h {tuple(h.shape)}, h0 {tuple(h0.shape)}, out {tuple(out.shape)}")
        if delta is not None:
            self._want(delta, "delta", out.dtype, 2)
            if delta.shape != h.shape:
                raise KernelError(f"stream_pair_rows: delta {tuple(delta.shape)} does not match h {tuple(h.shape)}")
        self._check(self.lib.ra_stream_pair_rows(_ptr(h), _ptr(delta), float(delta_scale), _ptr(h0), _ptr(out), T, H,
                                                 _code(out.dtype), self._stream()), "stream_pair_rows")

    def head_rmsnorm(self, x, weight, eps):
        self._want(x, "heads", dims=3)
        self._want(weight, "head norm weight", torch.float32, 1)
        if weight.shape[0] != x.shape[2]:
            raise KernelError(f"head_rmsnorm: weight {tuple(weight.shape)} for heads {tuple(x.shape)}")
        self._check(self.lib.ra_head_rmsnorm(_ptr(x), _ptr(weight), float(eps), x.shape[0] * x.shape[1],
                                             x.shape[2], _code(x.dtype), self._stream()), "head_rmsnorm")

    def rope(self, x, positions, cos, sin, rotary_dim):
        self._want(x, "heads", dims=3)
        self._want(positions, "positions", torch.int32, 1)
        self._want(cos, "cos table", torch.float32, 2)
        self._want(sin, "sin table", torch.float32, 2)
        T, heads, D = x.shape
        R = int(rotary_dim)
        if positions.shape[0] != T or R % 2 or R > D or cos.shape[1] != R // 2 or sin.shape != cos.shape:
            raise KernelError(f"rope: x {tuple(x.shape)}, rotary_dim {R}, tables {tuple(cos.shape)}")
        self._check(self.lib.ra_rope(_ptr(x), _ptr(positions), _ptr(cos), _ptr(sin), T, heads, D, R,
                                     _code(x.dtype), self._stream()), "rope")

    def split_heads(self, qkv, n_q, n_kv, D, q, k, v):
        self._want(qkv, "qkv", dims=2)
        T = qkv.shape[0]
        for t, name, heads in ((q, "q", n_q), (k, "k", n_kv), (v, "v", n_kv)):
            self._want(t, name, qkv.dtype, 3)
            if tuple(t.shape) != (T, heads, D):
                raise KernelError(f"split_heads: {name} is {tuple(t.shape)}, wanted {(T, heads, D)}")
        if qkv.shape[1] != (n_q + 2 * n_kv) * D:
            raise KernelError(f"split_heads: qkv width {qkv.shape[1]} is not {(n_q + 2 * n_kv) * D}")
        self._check(self.lib.ra_split_heads(_ptr(qkv), _ptr(q), _ptr(k), _ptr(v), T, n_q * D, n_kv * D,
                                            _code(qkv.dtype), self._stream()), "split_heads")

    def _pool_rows(self, k_pool, v_pool, n_kv, D, dtype):
        """Checks the pools of one cache layer, [pages, kv heads, rows in a page, D], and returns the
        number of token rows they hold (pages x page size)."""
        for t, name in ((k_pool, "k pool"), (v_pool, "v pool")):
            self._want(t, name, dtype, 4)
            if t.shape[1] != n_kv or t.shape[3] != D:
                raise KernelError(f"{name} {tuple(t.shape)} does not hold {n_kv} heads of {D}")
        if k_pool.shape != v_pool.shape:
            raise KernelError("k pool and v pool differ in shape")
        if k_pool.shape[0] * k_pool.shape[1] * k_pool.shape[2] >= 2 ** 31:
            raise KernelError(f"k pool {tuple(k_pool.shape)}: the kernels count head rows in 32 bits")
        return k_pool.shape[0] * k_pool.shape[2]

    def kv_write(self, k, v, k_pool, v_pool, slot_mapping):
        self._want(k, "k", dims=3)
        self._want(v, "v", k.dtype, 3)
        self._want(slot_mapping, "slot mapping", torch.int32, 1)
        T, n_kv, D = k.shape
        rows = self._pool_rows(k_pool, v_pool, n_kv, D, k.dtype)
        if v.shape != k.shape or slot_mapping.shape[0] != T:
            raise KernelError(f"kv_write: k {tuple(k.shape)}, v {tuple(v.shape)}, slots {tuple(slot_mapping.shape)}")
        self._check(self.lib.ra_kv_write(_ptr(k), _ptr(v), _ptr(k_pool), _ptr(v_pool), _ptr(slot_mapping),
                                         T, n_kv, D, k_pool.shape[2], rows, _code(k.dtype), self._stream()), "kv_write")

    def qkv_prepare(self, qkv, n_q, n_kv, D, w_q, w_k, eps, positions, cos, sin, rotary_dim, q_out,
                    k_pool, v_pool, slot_mapping):
        self._want(qkv, "qkv", dims=2)
        self._want(q_out, "q", qkv.dtype, 3)
        self._want(positions, "positions", torch.int32, 1)
        self._want(slot_mapping, "slot mapping", torch.int32, 1)
        T = qkv.shape[0]
        R = int(rotary_dim)
        if qkv.shape[1] != (n_q + 2 * n_kv) * D or tuple(q_out.shape) != (T, n_q, D):
            raise KernelError(f"qkv_prepare: qkv {tuple(qkv.shape)}, q {tuple(q_out.shape)}")
        if positions.shape[0] != T or slot_mapping.shape[0] != T:
            raise KernelError("qkv_prepare: positions/slot mapping do not match the token count")
        if (w_q is None) != (w_k is None):
            raise KernelError("qkv_prepare: q and k norm weights come together")
        if w_q is not None:
            for w in (w_q, w_k):
                self._want(w, "head norm weight", torch.float32, 1)
                if w.shape[0] != D:
                    raise KernelError(f"qkv_prepare: norm weight {tuple(w.shape)} for head size {D}")
        if R:
            self._want(cos, "cos table", torch.float32, 2)
            self._want(sin, "sin table", torch.float32, 2)
            if R % 2 or R > D or cos.shape[1] != R // 2 or sin.shape != cos.shape:
                raise KernelError(f"qkv_prepare: rotary_dim {R}, tables {tuple(cos.shape)}, head size {D}")
        if D > 512 or R // 2 > 256 or D - R > 256:
            raise KernelError(f"qkv_prepare: head size {D} (rotary {R}) is beyond the kernel's 512")
        rows = 0
        if k_pool is not None:
            rows = self._pool_rows(k_pool, v_pool, n_kv, D, qkv.dtype)
        self._check(self.lib.ra_qkv_prepare(
            _ptr(qkv), T, n_q, n_kv, D, _ptr(w_q), _ptr(w_k), float(eps), _ptr(positions),
            _ptr(cos) if R else None, _ptr(sin) if R else None, R, _ptr(q_out), _ptr(k_pool),
            _ptr(v_pool), _ptr(slot_mapping), k_pool.shape[2] if k_pool is not None else 0, rows, _code(qkv.dtype),
            self._stream()), "qkv_prepare")

    def silu_mul(self, gu, out, bias=None):
        """out = silu(gate) * up of rows [gate | up]; with bias (fp32 [2 I]) the two halves get theirs first."""
        self._want(gu, "gate-up", dims=2)
        self._want(out, "silu-mul output", gu.dtype, 2)
        T, I = out.shape
        if tuple(gu.shape) != (T, 2 * I):
            raise KernelError(f"silu_mul: gate-up {tuple(gu.shape)}, out {tuple(out.shape)}")
        if bias is not None:
            self._want(bias, "gate-up bias", torch.float32, 1)
            if bias.shape[0] != 2 * I:
                raise KernelError(f"silu_mul: bias {tuple(bias.shape)} for {2 * I} columns")
            self._check(self.lib.ra_silu_mul_bias(_ptr(gu), _ptr(bias), _ptr(out), T, I, _code(gu.dtype), self._stream()),
                        "silu_mul_bias")
            return
        self._check(self.lib.ra_silu_mul(_ptr(gu), _ptr(out), T, I, _code(gu.dtype), self._stream()),
                    "silu_mul")

    # ------------------------------------------------------------------ parts beside the usual ones
    def _want_rows(self, t, name, dtype=None):
        """A matrix whose rows may be a column slice of a wider one: rows apart by stride(0), elements side by side."""
        if t.device != self.device:
            raise KernelError(f"{name} is on {t.device}, kernels run on {self.device}")
        if t.dim() != 2 or (t.shape[1] > 1 and t.stride(1) != 1) or (t.shape[0] > 1 and t.stride(0) < t.shape[1]):
            raise KernelError(f"{name} must be rows of elements side by side, got shape {tuple(t.shape)} strides {t.stride()}")
        if dtype is not None and t.dtype != dtype:
            raise KernelError(f"{name} must be {dtype}, got {t.dtype}")
        return t.stride(0) if t.shape[0] > 1 else max(t.shape[1], t.stride(0))

    def relu_sq(self, x):
        """x <- max(x, 0)^2 in place."""
        self._want(x, "activations")
        self._check(self.lib.ra_relu_sq(_ptr(x), x.numel(), _code(x.dtype), self._stream()), "relu_sq")
        return x

    def add_bias(self, x, bias):
        """x [rows, N] += bias [N] (32-bit) in place."""
        self._want(x, "rows", dims=2)
        self._want(bias, "bias", torch.float32, 1)
        if bias.shape[0] != x.shape[1]:
            raise KernelError(f"add_bias: rows {tuple(x.shape)}, bias {tuple(bias.shape)}")
        self._check(self.lib.ra_add_bias(_ptr(x), _ptr(bias), x.shape[0], x.shape[1], _code(x.dtype), self._stream()),
                    "add_bias")
        return x

    def add_rmsnorm_pair(self, h, a, b, w1, eps1, out1, w2, eps2, out2):
        """h (fp32 [T, H]) += a + b in place (each may be None), then two RMS norms of the same rows with weights of
        their own: out1 = rmsnorm(h) w1, out2 = rmsnorm(h) w2 (both in the compute dtype)."""
        self._want(h, "residual stream", torch.float32, 2)
        T, H = h.shape
        self._want(out1, "first norm output", dims=2)
        self._want(out2, "second norm output", out1.dtype, 2)
        for t, name in ((a, "first delta"), (b, "second delta")):
            if t is not None:
                self._want(t, name, out1.dtype, 2)
                if tuple(t.shape) != (T, H):
                    raise KernelError(f"add_rmsnorm_pair: {name} {tuple(t.shape)} for a stream {tuple(h.shape)}")
        for w in (w1, w2):
            self._want(w, "norm weight", torch.float32, 1)
            if w.shape[0] != H:
                raise KernelError(f"add_rmsnorm_pair: norm weight {tuple(w.shape)} for rows of {H}")
        if tuple(out1.shape) != (T, H) or tuple(out2.shape) != (T, H):
            raise KernelError(f"add_rmsnorm_pair: outputs {tuple(out1.shape)}, {tuple(out2.shape)} for a stream {tuple(h.shape)}")
        self._check(self.lib.ra_add_rmsnorm_pair(_ptr(h), _ptr(a), _ptr(b), _ptr(w1), float(eps1), _ptr(out1), _ptr(w2),
                                                 float(eps2), _ptr(out2), T, H, _code(out1.dtype), self._stream()),
                    "add_rmsnorm_pair")

    def gated_rows(self, gu, out, activation="silu", limit=0.0, slope=1.702):
        """gu [T, >= 2 I] (gate columns first; possibly a column slice of wider rows; out's type or fp32) -> out [T, I] =
        silu(gate) * up or, "clamped", g sigmoid(slope g) (u + 1) with g = min(gate, limit), u = clamp(up, -limit, limit)."""
        ld = self._want_rows(gu, "gate-up rows")
        self._want(out, "activation output", dims=2)
        T, I = out.shape
        if activation not in ("silu", "clamped") or (activation == "clamped" and not limit > 0):
            raise KernelError(f"gated_rows: activation {activation!r} with limit {limit}")
        if gu.shape[0] != T or gu.shape[1] < 2 * I or gu.dtype not in (out.dtype, torch.float32):
            raise KernelError(f"gated_rows: gu {tuple(gu.shape)} {gu.dtype}, out {tuple(out.shape)} {out.dtype}")
        self._check(self.lib.ra_gated_rows(_ptr(gu), _code(gu.dtype), ld, _ptr(out), T, I, 1 if activation == "clamped" else 0,
                                           float(limit), float(slope), _code(out.dtype), self._stream()), "gated_rows")
        return out

    def clamped_mul(self, gu, out, limit, slope=1.702):
        return self.gated_rows(gu, out, "clamped", limit, slope)

    def gate_rows(self, o, gate):
        """o [T, N] *= sigmoid(gate) in place, element by element in 32-bit; both possibly column slices of wider rows."""
        ld_o = self._want_rows(o, "rows to gate")
        ld_g = self._want_rows(gate, "gates", o.dtype)
        if gate.shape != o.shape:
            raise KernelError(f"gate_rows: rows {tuple(o.shape)}, gates {tuple(gate.shape)}")
        self._check(self.lib.ra_gate_rows(_ptr(o), ld_o, _ptr(gate), ld_g, o.shape[0], o.shape[1], _code(o.dtype),
                                          self._stream()), "gate_rows")
        return o

    def qkv_rows_prepare(self, qkv, n_q, n_kv, D, w_q, w_k, q_size, k_size, eps, positions, cos, sin, rotary_dim, q_out,
                         k_pool, v_pool, slot_mapping):
        """q/k/v preparation of an attention whose norms run over the whole query and key projections: rows of qkv
        (possibly a column slice of wider rows) are [n_q | n_kv | n_kv] heads of D; the query part is divided by
        sqrt(sum of its squares / q_size + eps) and weighed (w_q fp32 [n_q D]), the key part by k_size likewise (w_k fp32
        [n_kv D]; elements beyond a head's true width must be zeros), then the first rotary_dim elements of every q and k
        head turn by the position (element i with i + rotary_dim / 2). q to q_out [T, n_q, D], k and v to the pools' rows
        that slot_mapping names (pools None: nothing is written)."""
        ld_qkv = self._want_rows(qkv, "qkv")
        self._want(q_out, "q", qkv.dtype, 3)
        self._want(positions, "positions", torch.int32, 1)
        T, R = qkv.shape[0], int(rotary_dim)
        if qkv.shape[1] != (n_q + 2 * n_kv) * D or tuple(q_out.shape) != (T, n_q, D) or positions.shape[0] != T \
                or not 1 <= q_size <= n_q * D or not 1 <= k_size <= n_kv * D:
            raise KernelError(f"qkv_rows_prepare: qkv {tuple(qkv.shape)}, q {tuple(q_out.shape)}, {T} tokens, norms over "
                              f"{q_size} and {k_size}")
        for w, n in ((w_q, n_q), (w_k, n_kv)):
            self._want(w, "norm weight", torch.float32, 1)
            if w.shape[0] != n * D:
                raise KernelError(f"qkv_rows_prepare: norm weight {tuple(w.shape)} for {n} heads of {D}")
        if R:
            self._want(cos, "cos table", torch.float32, 2)
            self._want(sin, "sin table", torch.float32, 2)
            if R % 2 or R > D or cos.shape[1] != R // 2 or sin.shape != cos.shape:
                raise KernelError(f"qkv_rows_prepare: rotary_dim {R}, tables {tuple(cos.shape)}, head size {D}")
        P, pool_rows = 1, 0
        if k_pool is not None:
            self._want(slot_mapping, "slot mapping", torch.int32, 1)
            if slot_mapping.shape[0] != T:
                raise KernelError("qkv_rows_prepare: slot mapping does not match the token count")
            pool_rows = self._pool_rows(k_pool, v_pool, n_kv, D, qkv.dtype)
            P = k_pool.shape[2]
        self._check(self.lib.ra_qkv_rows_prepare(
            _ptr(qkv), ld_qkv, T, n_q, n_kv, D, _ptr(w_q), _ptr(w_k), int(q_size), int(k_size), float(eps), _ptr(positions),
            _ptr(cos) if R else None, _ptr(sin) if R else None, R, _ptr(q_out), _ptr(k_pool), _ptr(v_pool),
            _ptr(slot_mapping) if k_pool is not None else None, P, pool_rows, _code(qkv.dtype), self._stream()),
            "qkv_rows_prepare")

    def qkv_blend_prepare(self, qkv, n_q, n_kv, D, bias, positions, cos, sin, rotary_dim, q_out, k_pool, v_pool,
                          slot_mapping, first=None, blend=None, w_q=None, w_k=None, norm_dim=None, eps=0.0):
        """q/k/v preparation of an attention: rows of qkv (possibly a column slice of wider rows) are [n_q | n_kv | n_kv]
        heads of D; the fp32 bias (one entry per column; None: none) is added, with w_q and w_k (fp32 [D]) every q and k
        head is divided by the root mean square of its first norm_dim (None: all) elements and weighed (what a head has
        beyond norm_dim must be zeros), the first rotary_dim elements of every q and k head turn by the position
        (element i with i + rotary_dim / 2), q goes to q_out [T, n_q, D], k and v to the pools' rows that slot_mapping
        names (pools None: nothing is written). first (fp32 [T, n_kv Dv], Dv <= D a head's true value width) with
        blend None: receives the first Dv elements of every head of the biased v; with blend lambda:
        v <- (1 - lambda) v + lambda first before it is stored."""
        ld_qkv = self._want_rows(qkv, "qkv")
        self._want(q_out, "q", qkv.dtype, 3)
        self._want(positions, "positions", torch.int32, 1)
        T, R = qkv.shape[0], int(rotary_dim)
        if qkv.shape[1] != (n_q + 2 * n_kv) * D or tuple(q_out.shape) != (T, n_q, D) or positions.shape[0] != T:
            raise KernelError(f"qkv_blend_prepare: qkv {tuple(qkv.shape)}, q {tuple(q_out.shape)}, {T} tokens")
        if bias is not None:
            self._want(bias, "bias", torch.float32, 1)
            if bias.shape[0] != qkv.shape[1]:
                raise KernelError(f"qkv_blend_prepare: bias {tuple(bias.shape)} for {qkv.shape[1]} columns")
        if (w_q is None) != (w_k is None):
            raise KernelError("qkv_blend_prepare: q and k norm weights come together")
        norm_dim = D if norm_dim is None else int(norm_dim)
        if not 1 <= norm_dim <= D:
            raise KernelError(f"qkv_blend_prepare: norm over {norm_dim} elements of heads of {D}")
        for w in (w_q, w_k) if w_q is not None else ():
            self._want(w, "head norm weight", torch.float32, 1)
            if w.shape[0] != D:
                raise KernelError(f"qkv_blend_prepare: norm weight {tuple(w.shape)} for head size {D}")
        if R:
            self._want(cos, "cos table", torch.float32, 2)
            self._want(sin, "sin table", torch.float32, 2)
            if R % 2 or R > D or cos.shape[1] != R // 2 or sin.shape != cos.shape:
                raise KernelError(f"qkv_blend_prepare: rotary_dim {R}, tables {tuple(cos.shape)}, head size {D}")
        mode, Dv = 0, D
        if first is not None:
            self._want(first, "first values", torch.float32, 2)
            Dv = first.shape[1] // n_kv
            if first.shape[0] != T or first.shape[1] != n_kv * Dv or not 1 <= Dv <= D:
                raise KernelError(f"qkv_blend_prepare: first values {tuple(first.shape)} for {T} tokens of {n_kv} x {D}")
            mode = 1 if blend is None else 2
        elif blend is not None:
            raise KernelError("qkv_blend_prepare: a blend weight without the values to blend with")
        P, pool_rows = 1, 0
        if k_pool is not None:
            self._want(slot_mapping, "slot mapping", torch.int32, 1)
            if slot_mapping.shape[0] != T:
                raise KernelError("qkv_blend_prepare: slot mapping does not match the token count")
            pool_rows = self._pool_rows(k_pool, v_pool, n_kv, D, qkv.dtype)
            P = k_pool.shape[2]
        self._check(self.lib.ra_qkv_blend_prepare(
            _ptr(qkv), ld_qkv, T, n_q, n_kv, D, _ptr(bias), _ptr(w_q), _ptr(w_k), norm_dim, float(eps), _ptr(positions),
            _ptr(cos) if R else None, _ptr(sin) if R else None,
            R, _ptr(q_out), _ptr(k_pool), _ptr(v_pool), _ptr(slot_mapping) if k_pool is not None else None, P, pool_rows,
            _ptr(first), Dv, mode, float(blend or 0.0), _code(qkv.dtype), self._stream()), "qkv_blend_prepare")

    def causal_conv(self, x, w, tail, step, out, add_input=False, silu=False, bias=None, in_bias=None):
        """out = act(conv(x)) or act(x + conv(x)): a causal convolution over time on each channel, the last
        taps-1 inputs of every request kept in tail [slots, taps-1, C] between steps (rows by the step's
        slot_ids). x: [T, C], possibly a column slice of wider rows; w: fp32 [C, taps], last column the
        current row's; out: [T, C] rows, not x. bias (fp32 [C]): added to the filter's sum; in_bias (fp32 [C]): added to
        every input first, rounded to x's type (the zeros before a request's start stay zeros)."""
        ld_x = self._want_rows(x, "conv input")
        ld_out = self._want_rows(out, "conv output", x.dtype)
        self._want(w, "conv weight", torch.float32, 2)
        self._want(tail, "conv tail", x.dtype, 3)
        T, C = x.shape
        taps = w.shape[1]
        if tuple(out.shape) != (T, C) or w.shape[0] != C or tuple(tail.shape[1:]) != (taps - 1, C) or T != step.n_tokens:
            raise KernelError(f"causal_conv: x {tuple(x.shape)}, w {tuple(w.shape)}, tail {tuple(tail.shape)}, "
                              f"out {tuple(out.shape)}, step of {step.n_tokens}")
        if not 1 <= taps <= 17:
            raise KernelError(f"causal_conv: {taps} taps, the kernel takes 1 to 17")
        if max(step.slot_ids_host, default=0) >= tail.shape[0]:
            raise KernelError("causal_conv: a request's slot lies beyond the tail's rows")
        if out.data_ptr() == x.data_ptr():
            raise KernelError("causal_conv: the output must not be the input")
        if bias is not None or in_bias is not None:
            for b in (bias, in_bias):
                if b is not None:
                    self._want(b, "conv bias", torch.float32, 1)
                    if b.shape[0] != C:
                        raise KernelError(f"causal_conv: bias {tuple(b.shape)} for {C} channels")
            self._check(self.lib.ra_causal_conv_bias(
                _ptr(x), ld_x, _ptr(in_bias), _ptr(w), _ptr(bias), _ptr(tail), _ptr(step.cu_q), _ptr(step.slot_ids), _ptr(out), ld_out,
                step.n_seqs, step.max_q_len, C, taps, (1 if add_input else 0) | (2 if silu else 0), _code(x.dtype),
                self._stream()), "causal_conv")
            return out
        self._check(self.lib.ra_causal_conv(
            _ptr(x), ld_x, _ptr(w), _ptr(tail), _ptr(step.cu_q), _ptr(step.slot_ids), _ptr(out), ld_out, step.n_seqs,
            step.max_q_len, C, taps, (1 if add_input else 0) | (2 if silu else 0), _code(x.dtype), self._stream()),
            "causal_conv")
        return out

    def delta_rule_fits(self, D, V):
        return bool(self.lib.ra_delta_rule_fits(int(D), int(V)))

    def delta_rule(self, qkv, beta, ag, a_log, dt_bias, norm_w, eps, state, step, out, H, G, D, V):
        """The gated delta rule with a decay per key channel over the step's rows, with what surrounds it in
        32-bit (unit q and k, sigmoid of beta, softplus and exponentials of the decay, the norm of the read-out
        and its gate). qkv: [T, 2 G D + H V] after the short convolution; beta: [T, H] before the sigmoid;
        ag: [T, H D + H V], the decay's and the output gate's projections; each may be a column slice of wider
        rows. state: fp32 [slots, H, V, D] (S column by column), updated in place; out: [T, H V]."""
        ld_qkv = self._want_rows(qkv, "delta-rule q/k/v")
        ld_b = self._want_rows(beta, "delta-rule beta", qkv.dtype)
        ld_ag = self._want_rows(ag, "delta-rule decay and gate projections", qkv.dtype)
        self._want(out, "delta-rule output", qkv.dtype, 2)
        self._want(state, "delta-rule state", torch.float32, 4)
        T = qkv.shape[0]
        for t, name, shape in ((a_log, "A_log", (H,)), (dt_bias, "dt_bias", (H * D,)), (norm_w, "norm weight", (V,))):
            self._want(t, name, torch.float32)
            if tuple(t.shape) != shape:
                raise KernelError(f"delta_rule: {name} is {tuple(t.shape)}, wanted {shape}")
        if qkv.shape[1] != 2 * G * D + H * V or tuple(out.shape) != (T, H * V) or tuple(beta.shape) != (T, H) \
                or tuple(ag.shape) != (T, H * D + H * V) or T != step.n_tokens or tuple(state.shape[1:]) != (H, V, D) or H % G:
            raise KernelError(f"delta_rule: qkv {tuple(qkv.shape)}, beta {tuple(beta.shape)}, ag {tuple(ag.shape)}, "
                              f"out {tuple(out.shape)}, state {tuple(state.shape)}, {H} heads over {G} of {D} x {V}, "
                              f"step of {step.n_tokens}")
        if max(step.slot_ids_host, default=0) >= state.shape[0]:
            raise KernelError("delta_rule: a request's slot lies beyond the state's rows")
        if not self.delta_rule_fits(D, V):
            raise KernelError(f"delta_rule: heads of {D} x {V} are beyond the kernel")
        o_raw = torch.empty(T, H * V, dtype=torch.float32, device=self.device)
        self._check(self.lib.ra_delta_rule(
            _ptr(qkv), ld_qkv, _ptr(beta), ld_b, _ptr(ag), ld_ag, _ptr(a_log), _ptr(dt_bias), _ptr(norm_w), float(eps),
            _ptr(state), _ptr(step.cu_q), _ptr(step.slot_ids), _ptr(o_raw), _ptr(out), step.n_seqs, T,
            max(1, int(step.max_q_len)), H, G, D, V,
            _code(qkv.dtype), self._stream()), "delta_rule")
        return out

    def delta_rule_head(self, qkv, beta, a, gate, a_log, dt_bias, norm_w, eps, state, step, out, H, G, D, V):
        """The gated delta rule with one decay per head and token, g = exp(-exp(a_log) softplus(a + dt_bias)), and what
        surrounds it in 32-bit (unit q and k, q times D^-1/2, sigmoid of beta); out = rmsnorm_V(o) * norm_w * silu(gate).
        qkv: [T, 2 G D + H V] after the short convolution; beta, a: [T, H]; gate: [T, H V]; each may be a column slice of
        wider rows. state: fp32 [slots, H, V, D] (S column by column), updated in place; out: [T, H V]."""
        ld_qkv = self._want_rows(qkv, "delta-rule q/k/v")
        ld_b = self._want_rows(beta, "delta-rule beta", qkv.dtype)
        ld_a = self._want_rows(a, "delta-rule decay projection", qkv.dtype)
        ld_g = self._want_rows(gate, "output gate", qkv.dtype)
        self._want(out, "delta-rule output", qkv.dtype, 2)
        self._want(state, "delta-rule state", torch.float32, 4)
        T = qkv.shape[0]
        for t, name, shape in ((a_log, "A_log", (H,)), (dt_bias, "dt_bias", (H,)), (norm_w, "norm weight", (V,))):
            self._want(t, name, torch.float32)
            if tuple(t.shape) != shape:
                raise KernelError(f"delta_rule_head: {name} is {tuple(t.shape)}, wanted {shape}")
        if qkv.shape[1] != 2 * G * D + H * V or tuple(out.shape) != (T, H * V) or tuple(beta.shape) != (T, H) \
                or tuple(a.shape) != (T, H) or tuple(gate.shape) != (T, H * V) or T != step.n_tokens \
                or tuple(state.shape[1:]) != (H, V, D) or H % G:
            raise KernelError(f"delta_rule_head: qkv {tuple(qkv.shape)}, beta {tuple(beta.shape)}, a {tuple(a.shape)}, "
                              f"gate {tuple(gate.shape)}, out {tuple(out.shape)}, state {tuple(state.shape)}, {H} heads over "
                              f"{G} of {D} x {V}, step of {step.n_tokens}")
        if max(step.slot_ids_host, default=0) >= state.shape[0]:
            raise KernelError("delta_rule_head: a request's slot lies beyond the state's rows")
        if not self.delta_rule_fits(D, V):
            raise KernelError(f"delta_rule_head: heads of {D} x {V} are beyond the kernel")
        o_raw = torch.empty(T, H * V, dtype=torch.float32, device=self.device)
        self._check(self.lib.ra_delta_rule_head(
            _ptr(qkv), ld_qkv, _ptr(beta), ld_b, _ptr(a), ld_a, _ptr(gate), ld_g, _ptr(a_log), _ptr(dt_bias), _ptr(norm_w),
            float(eps), _ptr(state), _ptr(step.cu_q), _ptr(step.slot_ids), _ptr(o_raw), _ptr(out), step.n_seqs, T,
            max(1, int(step.max_q_len)), H, G, D, V, _code(qkv.dtype), self._stream()), "delta_rule_head")
        return out

    def channel_recurrence(self, u, w_gates, gate_bias, rate, y, y_bias, state, step, out, out_scale=1.0):
        """A gated linear recurrence per channel over the step's rows: r, i = sigmoid(W u + bias) with a matrix per block
        of neighbouring channels, a = exp(rate r), S <- a S + sqrt(1 - a^2) i u, out = S gelu_tanh(y + y_bias) * out_scale,
        all but u, y and out in 32-bit. u: [T, width] contiguous; w_gates: [blocks, 2, width / blocks, width / blocks]
        (gate r first; rows are outputs); gate_bias: fp32 [2, width]; rate, y_bias: fp32 [width]; y: [T, width], possibly a
        column slice; state: fp32 [slots, width], updated in place; out: [T, >= width] rows, possibly a column slice (the
        columns beyond width become zeros)."""
        self._want(u, "recurrence input", dims=2)
        self._want(w_gates, "gate weights", u.dtype, 4)
        ld_y = self._want_rows(y, "output branch", u.dtype)
        ld_out = self._want_rows(out, "recurrence output", u.dtype)
        self._want(state, "recurrence state", torch.float32, 2)
        T, width = u.shape
        blocks = w_gates.shape[0]
        for t, name, shape in ((gate_bias, "gate bias", (2, width)), (rate, "rate", (width,)), (y_bias, "output bias", (width,))):
            self._want(t, name, torch.float32)
            if tuple(t.shape) != shape:
                raise KernelError(f"channel_recurrence: {name} is {tuple(t.shape)}, wanted {shape}")
        bw = width // blocks
        if width % blocks or tuple(w_gates.shape) != (blocks, 2, bw, bw) or tuple(y.shape) != (T, width) \
                or out.shape[0] != T or out.shape[1] < width or state.shape[1] != width or T != step.n_tokens:
            raise KernelError(f"channel_recurrence: u {tuple(u.shape)}, gates {tuple(w_gates.shape)}, y {tuple(y.shape)}, "
                              f"out {tuple(out.shape)}, state {tuple(state.shape)}, step of {step.n_tokens}")
        if max(step.slot_ids_host, default=0) >= state.shape[0]:
            raise KernelError("channel_recurrence: a request's slot lies beyond the state's rows")
        longest = max(1, int(step.max_q_len))
        # (decays and inputs of every row, and the summaries of the chunks of long requests)
        floats = 2 * T * width
        chunk = self.lib.ra_channel_recurrence_chunk(longest)
        if longest > chunk:
            floats += 2 * (T // chunk + step.n_seqs + 1) * width
        scratch = torch.empty(floats, dtype=torch.float32, device=self.device)
        self._check(self.lib.ra_channel_recurrence(
            _ptr(u), _ptr(w_gates), _ptr(gate_bias), _ptr(rate), _ptr(y), ld_y, _ptr(y_bias), _ptr(state), _ptr(step.cu_q),
            _ptr(step.slot_ids), _ptr(scratch), float(out_scale), _ptr(out), ld_out, out.shape[1], step.n_seqs, T, longest,
            width, blocks, _code(u.dtype), self._stream()), "channel_recurrence")
        return out

    # ------------------------------------------------------------------ layer norm behind a sublayer
    def layer_norm_add(self, h, y, weight, eps, out=None):
        """h (fp32 [T, H]) += (y - mean) / sqrt(variance + eps) * weight, row by row, in 32-bit; out (None: not wanted)
        receives the new rows of h in y's type."""
        self._want(h, "residual stream", torch.float32, 2)
        self._want(y, "sublayer output", dims=2)
        self._want(weight, "norm weight", torch.float32, 1)
        T, H = h.shape
        if tuple(y.shape) != (T, H) or weight.shape[0] != H:
            raise KernelError(f"layer_norm_add: h {tuple(h.shape)}, y {tuple(y.shape)}, weight {tuple(weight.shape)}")
        if out is not None:
            self._want(out, "stream rows", y.dtype, 2)
            if tuple(out.shape) != (T, H):
                raise KernelError(f"layer_norm_add: rows {tuple(out.shape)} for a stream {tuple(h.shape)}")
        self._check(self.lib.ra_layer_norm_add(_ptr(h), _ptr(y), _ptr(weight), float(eps), _ptr(out), T, H, _code(y.dtype),
                                               self._stream()), "layer_norm_add")

    def layer_norm(self, h, weight, eps, out, rows=None, bias=None, first=None, second=None):
        """out[i] = (g[r] - mean) / sqrt(variance + eps) * weight + bias with r = rows[i] (int32; None: r = i), where g is h
        (fp32 [T, H]) plus, in 32-bit, first [T, H] and second (rows [T, H] or RowSums), each None or in out's type. Without
        a list of rows h becomes g; with one it stays as it is."""
        self._want(h, "residual stream", torch.float32, 2)
        self._want(weight, "norm weight", torch.float32, 1)
        self._want(out, "norm output", dims=2)
        T, H = h.shape
        M = T
        if rows is not None:
            self._want(rows, "row list", torch.int32, 1)
            M = rows.shape[0]
        if weight.shape[0] != H or tuple(out.shape) != (M, H):
            raise KernelError(f"layer_norm: h {tuple(h.shape)}, weight {tuple(weight.shape)}, out {tuple(out.shape)}")
        if bias is not None:
            self._want(bias, "norm bias", torch.float32, 1)
            if bias.shape[0] != H:
                raise KernelError(f"layer_norm: bias {tuple(bias.shape)} for rows of {H}")
        if first is not None:
            self._want(first, "first delta", out.dtype, 2)
            if first.shape != h.shape:
                raise KernelError(f"layer_norm: first delta {tuple(first.shape)} for a stream {tuple(h.shape)}")
        b, nb, wb, extra, logit, ld_logit = None, 1, None, None, None, 0
        if isinstance(second, RowSums):
            b, nb, wb, extra, logit = second.rows, second.count, second.weights, second.extra, second.logits
            self._want(b, "rows to sum", out.dtype, 2)
            if tuple(b.shape) != (T * nb, H):
                raise KernelError(f"layer_norm: {tuple(b.shape)} rows for sums of {nb} into a stream {tuple(h.shape)}")
            if wb is not None:
                self._want(wb, "factors", torch.float32, 2)
                if tuple(wb.shape) != (T, nb):
                    raise KernelError(f"layer_norm: factors {tuple(wb.shape)} for {T} x {nb} rows")
            if extra is not None:
                self._want(extra, "further term", out.dtype, 2)
                ld_logit = self._want_rows(logit, "gate logits of the further term", torch.float32)
                if extra.shape != h.shape or tuple(logit.shape) != (T, 1):
                    raise KernelError(f"layer_norm: further term {tuple(extra.shape)}, its logits {tuple(logit.shape)}")
        elif second is not None:
            b = second
            self._want(b, "second delta", out.dtype, 2)
            if b.shape != h.shape:
                raise KernelError(f"layer_norm: second delta {tuple(b.shape)} for a stream {tuple(h.shape)}")
        self._check(self.lib.ra_stream_layer_norm(_ptr(h), _ptr(first), _ptr(b), int(nb), _ptr(wb), _ptr(extra), _ptr(logit),
                                                  ld_logit, _ptr(weight), _ptr(bias), float(eps), _ptr(out), _ptr(rows), M, H,
                                                  _code(out.dtype), self._stream()), "stream_layer_norm")

    def stream_rows(self, h, out):
        """out = the rows of h (fp32) in out's type."""
        self._want(h, "residual stream", torch.float32, 2)
        self._want(out, "stream rows", dims=2)
        if out.shape != h.shape:
            raise KernelError(f"stream_rows: h {tuple(h.shape)}, out {tuple(out.shape)}")
        self._check(self.lib.ra_stream_rows(_ptr(h), _ptr(out), h.numel(), _code(out.dtype), self._stream()), "stream_rows")

    def softcap(self, z, cap):
        """z <- cap * tanh(z / cap) in place (fp32)."""
        self._want(z, "logits", torch.float32)
        if not float(cap) > 0:
            raise KernelError(f"softcap: {cap} must be positive")
        self._check(self.lib.ra_softcap(_ptr(z), float(cap), z.numel(), self._stream()), "softcap")
        return z

    def outer_rule(self, qkv, a, gate, decay_bias, tau, norm_w, eps, state, step, out, H, D, V):
        """The gated outer-product memory of a linear attention over the step's rows: S <- diag(alpha) S + k v^T,
        o = S^T q with alpha = sigmoid(a + decay_bias)^(1/tau), q times D^-1/2; out = rmsnorm_V(o) * norm_w * silu(gate).
        qkv: [T, 2 H D + H V]; a: [T, H D]; gate: [T, H V]; each may be a column slice of wider rows. state: fp32
        [slots, H, V, D] (S column by column), updated in place; out: [T, H V]."""
        ld_qkv = self._want_rows(qkv, "linear-attention q/k/v")
        ld_a = self._want_rows(a, "decay logits", qkv.dtype)
        ld_g = self._want_rows(gate, "output gate", qkv.dtype)
        self._want(out, "linear-attention output", qkv.dtype, 2)
        self._want(state, "linear-attention state", torch.float32, 4)
        T = qkv.shape[0]
        for t, name, shape in ((decay_bias, "decay bias", (H * D,)), (norm_w, "norm weight", (V,))):
            self._want(t, name, torch.float32)
            if tuple(t.shape) != shape:
                raise KernelError(f"outer_rule: {name} is {tuple(t.shape)}, wanted {shape}")
        if qkv.shape[1] != 2 * H * D + H * V or tuple(out.shape) != (T, H * V) or tuple(a.shape) != (T, H * D) \
                or tuple(gate.shape) != (T, H * V) or T != step.n_tokens or tuple(state.shape[1:]) != (H, V, D):
            raise KernelError(f"outer_rule: qkv {tuple(qkv.shape)}, a {tuple(a.shape)}, gate {tuple(gate.shape)}, "
                              f"out {tuple(out.shape)}, state {tuple(state.shape)}, {H} heads of {D} x {V}, "
                              f"step of {step.n_tokens}")
        if max(step.slot_ids_host, default=0) >= state.shape[0]:
            raise KernelError("outer_rule: a request's slot lies beyond the state's rows")
        if not self.delta_rule_fits(D, V) or not float(tau) > 0:
            raise KernelError(f"outer_rule: heads of {D} x {V} (tau {tau}) are beyond the kernel")
        o_raw = torch.empty(T, H * V, dtype=torch.float32, device=self.device)
        self._check(self.lib.ra_outer_rule(
            _ptr(qkv), ld_qkv, _ptr(a), ld_a, _ptr(gate), ld_g, _ptr(decay_bias), 1.0 / float(tau), _ptr(norm_w), float(eps),
            _ptr(state), _ptr(step.cu_q), _ptr(step.slot_ids), _ptr(o_raw), _ptr(out), step.n_seqs, T,
            max(1, int(step.max_q_len)), H, D, V, _code(qkv.dtype), self._stream()), "outer_rule")
        return out

    def scalar_rule(self, qkv, dt, a_log, dt_bias, skip, gate, norm_w, norm_groups, eps, state, step, out, H, G, D, V):
        """The memory of a state-space layer with one decay per head and token over the step's rows:
        delta = softplus(dt + dt_bias); S <- exp(-exp(a_log) delta) S + delta k v^T; o = S^T q + skip v (head h reads
        q and k of group h // (H / G)); out = rmsnorm over each of norm_groups equal parts of (o * silu(gate)), times
        norm_w. qkv: [T, 2 G D + H V] rows [q | k | v]; dt: [T, H]; gate: [T, H V]; each may be a column slice of wider
        rows. state: fp32 [slots, H, V, D] (S column by column), updated in place; out: [T, H V]."""
        ld_qkv = self._want_rows(qkv, "state-space q/k/v")
        ld_dt = self._want_rows(dt, "step sizes", qkv.dtype)
        ld_g = self._want_rows(gate, "output gate", qkv.dtype)
        self._want(out, "state-space output", qkv.dtype, 2)
        self._want(state, "state", torch.float32, 4)
        T = qkv.shape[0]
        for t, name, shape in ((a_log, "A_log", (H,)), (dt_bias, "dt_bias", (H,)), (skip, "skip", (H,)),
                               (norm_w, "norm weight", (H * V,))):
            self._want(t, name, torch.float32)
            if tuple(t.shape) != shape:
                raise KernelError(f"scalar_rule: {name} is {tuple(t.shape)}, wanted {shape}")
        if qkv.shape[1] != 2 * G * D + H * V or tuple(out.shape) != (T, H * V) or tuple(dt.shape) != (T, H) \
                or tuple(gate.shape) != (T, H * V) or T != step.n_tokens or tuple(state.shape[1:]) != (H, V, D) or H % G \
                or norm_groups < 1 or (H * V) % norm_groups:
            raise KernelError(f"scalar_rule: qkv {tuple(qkv.shape)}, dt {tuple(dt.shape)}, gate {tuple(gate.shape)}, "
                              f"out {tuple(out.shape)}, state {tuple(state.shape)}, {H} heads over {G} of {D} x {V}, "
                              f"{norm_groups} norm parts, step of {step.n_tokens}")
        if max(step.slot_ids_host, default=0) >= state.shape[0]:
            raise KernelError("scalar_rule: a request's slot lies beyond the state's rows")
        if not self.delta_rule_fits(D, V):
            raise KernelError(f"scalar_rule: heads of {D} x {V} are beyond the kernel")
        o_raw = torch.empty(T, H * V, dtype=torch.float32, device=self.device)
        self._check(self.lib.ra_scalar_rule(
            _ptr(qkv), ld_qkv, _ptr(dt), ld_dt, _ptr(gate), ld_g, _ptr(a_log), _ptr(dt_bias), _ptr(skip), _ptr(norm_w),
            int(norm_groups), float(eps), _ptr(state), _ptr(step.cu_q), _ptr(step.slot_ids), _ptr(o_raw), _ptr(out),
            step.n_seqs, T, max(1, int(step.max_q_len)), H, G, D, V, _code(qkv.dtype), self._stream()), "scalar_rule")
        return out

    def token_side(self, h, delta, token_ids, table, offset, gate, proj, weight, eps):
        """h += delta, then h += rmsnorm(proj (gelu_tanh(gate h) * table[token][offset:offset+S])) * weight,
        row by row, in place. delta may be None."""
        self._want(h, "residual stream", torch.float32, 2)
        T, H = h.shape
        self._want(token_ids, "token ids", torch.int32, 1)
        self._want(gate, "side gate", dims=2)
        S = gate.shape[0]
        self._want(proj, "side projection", gate.dtype, 2)
        self._want(table, "side table", gate.dtype, 2)
        self._want(weight, "side norm weight", torch.float32, 1)
        if delta is not None:
            self._want(delta, "delta", gate.dtype, 2)
        if tuple(gate.shape) != (S, H) or tuple(proj.shape) != (H, S) or weight.shape[0] != H or token_ids.shape[0] != T \
                or (delta is not None and tuple(delta.shape) != (T, H)) or offset < 0 or offset + S > table.shape[1]:
            raise KernelError(f"token_side: h {tuple(h.shape)}, gate {tuple(gate.shape)}, proj {tuple(proj.shape)}, "
                              f"table {tuple(table.shape)} at {offset}")
        if S > 512 or H > 8192:
            raise KernelError(f"token_side: {S} side channels (at most 512) for rows of {H} (at most 8192)")
        self._check(self.lib.ra_token_side(_ptr(h), _ptr(delta), _ptr(token_ids), _ptr(table), table.shape[1], int(offset),
                                           _ptr(gate), _ptr(proj), _ptr(weight), float(eps), T, H, S,
                                           _code(gate.dtype), self._stream()), "token_side")

    def qk_prepare(self, qk, n_q, n_kv, D, bias, positions, cos, sin, rotary_dim, q_out, k_pool, v_pool, slot_mapping):
        """q/k preparation of an attention whose values are its keys as projected: bias, rotation of the first
        rotary_dim elements, q to q_out, the rotated k to the key pool and the unrotated k to the value pool."""
        self._want(qk, "qk", dims=2)
        self._want(q_out, "q", qk.dtype, 3)
        self._want(positions, "positions", torch.int32, 1)
        self._want(slot_mapping, "slot mapping", torch.int32, 1)
        T = qk.shape[0]
        R = int(rotary_dim)
        if qk.shape[1] != (n_q + n_kv) * D or tuple(q_out.shape) != (T, n_q, D) or positions.shape[0] != T \
                or slot_mapping.shape[0] != T:
            raise KernelError(f"qk_prepare: qk {tuple(qk.shape)}, q {tuple(q_out.shape)}, {T} tokens")
        if bias is not None:
            self._want(bias, "bias", torch.float32, 1)
            if bias.shape[0] != qk.shape[1]:
                raise KernelError(f"qk_prepare: bias {tuple(bias.shape)} for rows of {qk.shape[1]}")
        if R:
            self._want(cos, "cos table", torch.float32, 2)
            self._want(sin, "sin table", torch.float32, 2)
            if R % 2 or R > D or cos.shape[1] != R // 2 or sin.shape != cos.shape:
                raise KernelError(f"qk_prepare: rotary_dim {R}, tables {tuple(cos.shape)}, head size {D}")
        rows = 0
        if k_pool is not None:
            rows = self._pool_rows(k_pool, v_pool, n_kv, D, qk.dtype)
        self._check(self.lib.ra_qk_prepare(
            _ptr(qk), T, n_q, n_kv, D, _ptr(bias), _ptr(positions), _ptr(cos) if R else None, _ptr(sin) if R else None, R,
            _ptr(q_out), _ptr(k_pool), _ptr(v_pool), _ptr(slot_mapping), k_pool.shape[2] if k_pool is not None else 0,
            rows, _code(qk.dtype), self._stream()), "qk_prepare")

    # ------------------------------------------------------------------ matrix products
    # Ways to form y = x @ w^T from bfloat16 operands. Which is fastest depends on the shape in ways no
    # rule captures (the library streams one weight at 5.6 TB/s and the next at 2): route_* give the
    # rule's choice, tune_products replaces it where a measurement at load time says otherwise.
    ROW_STEPS = (1, 2, 4, 8, 12, 16, 24, 32, 48, 64)     # row counts at which products are measured
    # ... and beyond them the products for the residual stream only: with a few hundred rows (portions of
    # prompts beside decoded tokens) the library gives a product with few result columns and many of K too
    # few workgroups, and a batch over pieces of K is up to twice as fast (measured on MI355X, 512 rows:
    # 8B down 84 -> 55 µs, 32B down 272 -> 122 µs)
    ROW_STEPS_RESIDUAL = (96, 128, 192, 256, 384, 512, 640, 768, 1024, 1536, 2048, 3072, 4096)

    def _rows_step(self, M, residual=False):
        for r in self.ROW_STEPS + (self.ROW_STEPS_RESIDUAL if residual else ()):
            if M <= r:
                return r
        return 0                                          # more rows than are ever measured: the library

    SPLITS = (2, 4, 8)            # pieces of K that a product for the residual stream may be cut into

    def route_linear(self, M, N, K, out_dtype):
        """How linear() forms a bfloat16 product of M rows: the measured choice if there is one, else the rule.
        out_dtype "residual": the product whose result goes into the residual stream (linear_residual), bfloat16
        rows or, "split<n>", n shares of 32-bit sums from the library's batched product over n pieces of K."""
        hit = self.product_plan.get((self._rows_step(M, out_dtype == "residual"), N, K, False, out_dtype))
        if hit is not None:
            return hit
        if out_dtype == "residual":
            # measured on MI355X (8B shape, down: N 4,096, K 12,288): at 17 to 64 rows the library gives one
            # workgroup to each tile of the result and leaves half the chip idle; four pieces of K as a
            # batch take 24 µs against 29 to 38
            if 16 < M <= 64 and K >= 8192 and N * 2 <= K and K % 32 == 0 and self._library_bmm_fp32:
                return "split4"
            out_dtype = torch.bfloat16
        if out_dtype in (torch.bfloat16, torch.float32) and self.use_sweep(M, N, K, False):
            return "sweep"
        if out_dtype in (torch.bfloat16, torch.float32) and self.use_resident(M, N, K, False):
            return "resident512" if M <= 8 else "resident256"
        if self.use_skinny(M, N, K, out_dtype):
            return "skinny"
        if not self.own_gemm and (out_dtype == torch.bfloat16 or self._library_fp32_out):
            return "library"
        return "mfma" if K % 8 == 0 else "plain"

    def route_gated(self, M, I, K):
        hit = self.product_plan.get((self._rows_step(M), I, K, True, torch.bfloat16))
        if hit is not None:
            return hit
        if self.use_sweep(M, I, K, True):
            return "sweep"
        if self.use_resident(M, I, K, True):
            return "resident512" if M <= 8 else "resident256"
        if 0 < M <= self.gated_skinny_rows and K % 8 == 0:
            return "skinny"
        return "two"

    def _linear_by(self, how, x, w, out_dtype):
        M, K = x.shape
        N = w.shape[0]
        if how == "library":
            if out_dtype == torch.bfloat16:
                return torch.matmul(x, w.t())          # library product, as the reference's F.linear
            return torch.mm(x, w.t(), out_dtype=torch.float32)   # bf16 operands, 32-bit sums and results
        y = torch.empty(M, N, dtype=out_dtype, device=self.device)
        if how == "sweep":
            self._check(self.lib.ra_gemm_sweep_bf16(_ptr(x), _ptr(w), _ptr(y), M, N, K, 0, _code(out_dtype),
                                                    self.cu_count, self._stream()), "gemm_sweep")
        elif how.startswith("resident"):
            self._check(self.lib.ra_gemm_resident_bf16(_ptr(x), _ptr(w), _ptr(y), M, N, K, 0, _code(out_dtype),
                                                       int(how[8:]), self._stream()), "gemm_resident")
        elif how == "skinny":
            self._check(self.lib.ra_gemm_skinny_bf16(_ptr(x), _ptr(w), _ptr(y), M, N, K, _code(out_dtype),
                                                     self.skinny_max_grid, self._stream()), "gemm_skinny")
        elif how == "mfma":
            self._check(self.lib.ra_gemm_mfma_bf16(_ptr(x), _ptr(w), _ptr(y), M, N, K, _code(out_dtype),
                                                   self._stream()), "gemm_mfma")
        else:
            self._check(self.lib.ra_gemm_nt(_ptr(x), _ptr(w), _ptr(y), M, N, K, _code(x.dtype),
                                            _code(out_dtype), self._stream()), "gemm_nt")
        return y

    # ---- a norm finished inside the products around it (ScaledRows)
    def can_defer_norm(self, M, w_last, w_first, gated_first):
        """Whether, for M rows, the product by w_last [H, K1] can add its result into the residual stream
        and leave the rows of the norm that follows unfinished (linear_add_norm), and the product by
        w_first ([N, H], or [2N, H] gated) can finish them: both must be products that the sweep forms."""
        if not self.defer_norms or M < 1 or M > 16:
            return False
        for w in (w_last, w_first):
            if w.dtype != torch.bfloat16 or w.dim() != 2 or w.device != self.device:
                return False
        H = w_last.shape[0]
        if w_first.shape[1] != H or H < self.cu_count or (gated_first and w_first.shape[0] % 2):
            return False
        if self.lib.ra_gemm_sweep_workgroups(H, self.cu_count) > 256:      # shares of a row's sum that the next product adds up
            return False
        if not (self.lib.ra_gemm_sweep_fits(M, w_last.shape[1]) and self.lib.ra_gemm_sweep_fits(M, H)):
            return False
        # measured at load (tune_norm_pairs) where it was; else yes
        hit = self._defer.get((self._rows_step(M), tuple(w_last.shape), tuple(w_first.shape), bool(gated_first)))
        return True if hit is None else hit

    def tune_norm_pairs(self, pairs, max_rows=16):
        """Measures, for every shape among ``pairs`` and every row count of ROW_STEPS up to 16, whether the
        norm between two products is faster finished inside them (which ties both to the sweep) or as a
        kernel of its own between the fastest ways to form them, and notes it for can_defer_norm.
        pairs: (w_last [H, K1], norm weight [H] fp32, eps, w_first, gated) as the model has them."""
        groups = {}
        for w_last, wn, eps, w_first, gated in pairs:
            if w_last.dtype != torch.bfloat16 or w_first.dtype != torch.bfloat16 or w_last.device != self.device:
                continue
            groups.setdefault((tuple(w_last.shape), tuple(w_first.shape), bool(gated)), []).append((w_last, wn, eps, w_first))
        for (s_last, s_first, gated), members in groups.items():
            for rows in self.ROW_STEPS:
                if rows > 16 or (rows > max(1, max_rows) and rows != self._rows_step(max_rows)):
                    continue
                key = (rows, s_last, s_first, gated)
                if key in _NORM_PAIRS_MEASURED:
                    self._defer[key] = _NORM_PAIRS_MEASURED[key]
                    continue
                self._defer.pop(key, None)
                if not self.can_defer_norm(rows, members[0][0], members[0][3], gated):
                    continue
                _NORM_PAIRS_MEASURED[key] = self._defer[key] = self._measure_norm_pair(rows, members[:16], gated)

    def _measure_norm_pair(self, rows, members, gated):
        H, K1 = members[0][0].shape
        x = torch.randn(rows, K1, device=self.device, dtype=torch.float32).to(torch.bfloat16)
        h = torch.randn(rows, H, device=self.device, dtype=torch.float32)
        out = torch.empty(rows, H, dtype=torch.bfloat16, device=self.device)
        finish = self.linear_silu_mul if gated else self.linear

        def inside(m):
            w_last, wn, eps, w_first = m
            return finish(self.linear_add_norm(x, w_last, h, wn, eps), w_first)

        def apart(m):
            w_last, wn, eps, w_first = m
            self.add_rmsnorm(h, self.linear_residual(x, w_last), wn, eps, out)
            return finish(out, w_first)
        launches = max(4, min(16, len(members)))
        t_in = self._time_over(inside, members, launches)
        h.normal_()
        t_out = self._time_over(apart, members, launches)
        return t_in <= t_out

    def _sweep_norm(self, x, w, gated, out_dtype, rows_in=None, h=None, w_next=None):
        """The sweeping product with a row scale from rows_in (ScaledRows) and, with h, the residual epilogue."""
        M, K = x.shape
        N = w.shape[0] // 2 if gated else w.shape[0]
        if not self.lib.ra_gemm_sweep_fits(M, K) or M > 32:
            raise KernelError(f"rows with an unfinished norm need the sweeping product, which does not take {M} x {K}")
        out = torch.empty(M, N, dtype=out_dtype, device=self.device)
        psq_in = n_in = cols = None
        eps = 0.0
        if rows_in is not None:
            self._want(rows_in.partials, "partial sums of squares", torch.float32, 2)
            if rows_in.partials.shape[0] != M:
                raise KernelError(f"partial sums for {rows_in.partials.shape[0]} rows, x has {M}")
            psq_in, n_in, cols, eps = rows_in.partials, rows_in.partials.shape[1], rows_in.size, rows_in.eps
        psq_out = None
        if h is not None:
            self._want(h, "residual stream", torch.float32, 2)
            self._want(w_next, "norm weight", torch.float32, 1)
            if tuple(h.shape) != (M, N) or w_next.shape[0] != N or gated or out_dtype != torch.bfloat16 or M > 16:
                raise KernelError(f"linear_add_norm: x {tuple(x.shape)}, weight {tuple(w.shape)}, h {tuple(h.shape)}")
            psq_out = torch.empty(M, self.lib.ra_gemm_sweep_workgroups(N, self.cu_count), dtype=torch.float32,
                                  device=self.device)
        self._check(self.lib.ra_gemm_sweep_norm_bf16(
            _ptr(x), _ptr(w), _ptr(out), M, N, K, 1 if gated else 0, _code(out_dtype), self.cu_count,
            _ptr(psq_in), n_in or 0, cols or 0, float(eps), _ptr(h), _ptr(w_next), _ptr(psq_out), self._stream()),
            "gemm_sweep_norm")
        return out, psq_out

    def linear_add_norm(self, x, w, h, norm_weight, eps):
        """h += x @ w^T (the result rounded to the compute dtype first, as a stored result would be), and
        the rows of RMSNorm(h) with this weight and eps left unfinished: ScaledRows for linear() or
        linear_silu_mul(). x: plain rows or ScaledRows."""
        rows_in = x if isinstance(x, ScaledRows) else None
        xt = x.tensor if rows_in is not None else x
        self._want(xt, "x", torch.bfloat16, 2)
        self._want(w, "weight", torch.bfloat16, 2)
        if w.shape[1] != xt.shape[1]:
            raise KernelError(f"linear_add_norm: x {tuple(xt.shape)} times weight {tuple(w.shape)}^T")
        xw, psq = self._sweep_norm(xt, w, False, torch.bfloat16, rows_in, h, norm_weight)
        return ScaledRows(xw, psq, w.shape[0], eps)

    def _split_product(self, x, w, pieces):
        """x @ w^T as `pieces` shares [pieces, M, N] fp32, share i from columns i*K/pieces .. of K: one batched
        library product over strided views of x and w (nothing is copied)."""
        M, K = x.shape
        N = w.shape[0]
        xs = x.view(M, pieces, K // pieces).transpose(0, 1)
        wv = w.view(N, pieces, K // pieces).permute(1, 2, 0)
        return Slabs(torch.bmm(xs, wv, out_dtype=torch.float32))

    def linear_residual(self, x, w):
        """x @ w^T for the residual stream: bfloat16 (or float32) rows as linear() gives them, or Slabs
        where cutting K into pieces is faster; what takes the result must take both (the norm part does)."""
        if isinstance(x, ScaledRows) or x.dtype != torch.bfloat16:
            return self.linear(x, w)
        self._want(x, "x", dims=2)
        self._want(w, "weight", x.dtype, 2)
        M, K = x.shape
        if w.shape[1] != K:
            raise KernelError(f"linear: x {tuple(x.shape)} times weight {tuple(w.shape)}^T")
        if M == 0:
            return self.linear(x, w)
        how = self.route_linear(M, w.shape[0], K, "residual")
        if how.startswith("split"):
            return self._split_product(x, w, int(how[5:]))
        return self._linear_by(how, x, w, torch.bfloat16)

    def linear(self, x, w, out_dtype=None):
        """y = x @ w^T, x [M, K] (or ScaledRows: rows whose norm this product finishes), w [N, K]."""
        if isinstance(x, ScaledRows):
            self._want(x.tensor, "x", torch.bfloat16, 2)
            self._want(w, "weight", torch.bfloat16, 2)
            if w.shape[1] != x.tensor.shape[1]:
                raise KernelError(f"linear: x {tuple(x.tensor.shape)} times weight {tuple(w.shape)}^T")
            return self._sweep_norm(x.tensor, w, False, out_dtype or torch.bfloat16, x)[0]
        self._want(x, "x", dims=2)
        self._want(w, "weight", x.dtype, 2)
        M, K = x.shape
        N = w.shape[0]
        if w.shape[1] != K:
            raise KernelError(f"linear: x {tuple(x.shape)} times weight {tuple(w.shape)}^T")
        out_dtype = out_dtype or x.dtype
        if x.dtype == torch.float32 and out_dtype == torch.float32 and M > 16 and self._library_fp32_exact \
                and not self.own_gemm:
            return torch.matmul(x, w.t())          # the library's float32 product: checked above to be 32-bit
        if M == 0 or x.dtype != torch.bfloat16:
            return self._linear_by("plain", x, w, out_dtype)      # float32: 32-bit FMA products, W streamed once
        return self._linear_by(self.route_linear(M, N, K, out_dtype), x, w, out_dtype)

    def _gated_by(self, how, x, w_gate_up):
        M, K = x.shape
        I = w_gate_up.shape[0] // 2
        out = torch.empty(M, I, dtype=x.dtype, device=self.device)
        if how == "sweep":
            self._check(self.lib.ra_gemm_sweep_bf16(_ptr(x), _ptr(w_gate_up), _ptr(out), M, I, K, 1, _code(x.dtype),
                                                    self.cu_count, self._stream()), "gemm_sweep_gated")
        elif how.startswith("resident"):
            self._check(self.lib.ra_gemm_resident_bf16(_ptr(x), _ptr(w_gate_up), _ptr(out), M, I, K, 1,
                                                       _code(x.dtype), int(how[8:]), self._stream()),
                        "gemm_resident_gated")
        elif how == "skinny":
            self._check(self.lib.ra_gemm_skinny_gated_bf16(_ptr(x), _ptr(w_gate_up), _ptr(out), M, I, K,
                                                           self._stream()), "gemm_skinny_gated")
        else:
            self.silu_mul(self.linear(x, w_gate_up), out)
        return out

    def linear_silu_mul(self, x, w_gate_up):
        """silu(x @ Wg^T) * (x @ Wu^T) for w_gate_up = [Wg; Wu]: one kernel for few rows, else two."""
        if isinstance(x, ScaledRows):
            self._want(x.tensor, "x", torch.bfloat16, 2)
            self._want(w_gate_up, "gate-up weight", torch.bfloat16, 2)
            if w_gate_up.shape[1] != x.tensor.shape[1] or w_gate_up.shape[0] % 2:
                raise KernelError(f"linear_silu_mul: x {tuple(x.tensor.shape)}, weight {tuple(w_gate_up.shape)}")
            return self._sweep_norm(x.tensor, w_gate_up, True, torch.bfloat16, x)[0]
        self._want(x, "x", dims=2)
        self._want(w_gate_up, "gate-up weight", x.dtype, 2)
        M, K = x.shape
        I = w_gate_up.shape[0] // 2
        if w_gate_up.shape[1] != K or w_gate_up.shape[0] != 2 * I:
            raise KernelError(f"linear_silu_mul: x {tuple(x.shape)}, weight {tuple(w_gate_up.shape)}")
        how = self.route_gated(M, I, K) if x.dtype == torch.bfloat16 and M > 0 else "two"
        return self._gated_by(how, x, w_gate_up)

    def _candidates(self, M, N, K, gated, out_dtype):
        """The ways that can form this product at all."""
        residual = out_dtype == "residual"
        if residual:
            out_dtype = torch.bfloat16
        if gated:
            c = ["two"]
            if M <= 16 and K % 8 == 0:
                c.append("skinny")
        else:
            c = ["library"] if out_dtype == torch.bfloat16 or self._library_fp32_out else []
            if M <= 64 and K % 8 == 0:
                c.append("skinny")
        if self.lib.ra_gemm_resident_fits(M, K, 1 if gated else 0):
            c += ["resident256", "resident512"]
        if self.lib.ra_gemm_sweep_fits(M, K):
            c.append("sweep")
        if residual and self._library_bmm_fp32 and M > 16:
            c += [f"split{n}" for n in self.SPLITS if K % (8 * n) == 0]
        return c

    def tune_products(self, products, max_rows=64, margin=0.93, max_rows_residual=0):
        """Measures, for every shape among ``products`` and every row count of ROW_STEPS up to max_rows,
        the ways to form the product, and notes the fastest in product_plan where it beats the rule's
        choice by more than the margin (so that noise does not move a choice to and fro).

        products: (weight [N, K] bfloat16, gated, out_dtype) of the model's projections. The weights
        of one shape are taken in turn, as a decode step reads them: from memory, not from a cache
        that a repeated product on one weight would sit in. A few milliseconds per shape and row count."""
        groups = {}
        for w, gated, out_dtype in products:
            if w.dtype != torch.bfloat16 or w.dim() != 2 or w.device != self.device:
                continue
            N = w.shape[0] // 2 if gated else w.shape[0]
            groups.setdefault((N, w.shape[1], bool(gated), out_dtype or torch.bfloat16), []).append(w)
        for (N, K, gated, out_dtype), ws in groups.items():
            seen, uniq = set(), []
            for w in ws:                                  # tied weights are listed once
                if w.data_ptr() not in seen:
                    seen.add(w.data_ptr())
                    uniq.append(w)
            launches = max(4, min(16, len(uniq)))
            steps = self.ROW_STEPS
            if out_dtype == "residual" and max_rows_residual > self.ROW_STEPS[-1]:
                top = self._rows_step(max_rows_residual, True) or self.ROW_STEPS_RESIDUAL[-1]
                steps = steps + tuple(r for r in self.ROW_STEPS_RESIDUAL if r <= top)
            for rows in steps:
                if rows <= self.ROW_STEPS[-1] and rows > max(1, max_rows) and rows != self._rows_step(max_rows):
                    continue
                key = (rows, N, K, gated, out_dtype)
                if key not in self._measured:
                    # (products of many rows take long enough to be timed over a few launches)
                    few = launches if rows <= self.ROW_STEPS[-1] else max(4, min(launches, 4096 // rows))
                    self._measured[key] = self._measure(key, uniq, few, margin)
                if self._measured[key] is not None:
                    self.product_plan[key] = self._measured[key]

    def _measure(self, key, weights, launches, margin):
        """The way that forms this product clearly faster than the rule's, or None."""
        rows, N, K, gated, out_dtype = key
        cands = self._candidates(rows, N, K, gated, out_dtype)
        saved, self.product_plan = self.product_plan, {}          # the rule's choice, and "two" by the rule's product
        try:
            rule = self.route_gated(rows, N, K) if gated else self.route_linear(rows, N, K, out_dtype)
            if len(cands) < 2 or rule not in cands:
                return None
            x = torch.randn(rows, K, device=self.device, dtype=torch.float32).to(torch.bfloat16)
            if out_dtype == "residual":
                # with the residual add and norm that takes the result: shares cost it more than one result does
                h = torch.zeros(rows, N, device=self.device, dtype=torch.float32)
                wn = torch.ones(N, device=self.device, dtype=torch.float32)
                normed = torch.empty(rows, N, device=self.device, dtype=torch.bfloat16)
            runs = {}
            for how in cands:
                if gated:
                    runs[how] = lambda w, how=how: self._gated_by(how, x, w)
                elif how.startswith("split"):
                    runs[how] = lambda w, how=how: self.add_rmsnorm(h, self._split_product(x, w, int(how[5:])), wn, 1e-6, normed)
                elif out_dtype == "residual":
                    runs[how] = lambda w, how=how: self.add_rmsnorm(h, self._linear_by(how, x, w, torch.bfloat16), wn, 1e-6, normed)
                else:
                    runs[how] = lambda w, how=how: self._linear_by(how, x, w, out_dtype)
            times = self._time_ways(runs, weights, launches)
        finally:
            self.product_plan = saved
        self._times[key] = dict(times)
        best = min(times, key=times.get)
        return best if best != rule and times[best] < margin * times[rule] else None

    def _time_ways(self, runs, weights, launches, rounds=3):
        """Seconds per call of every way in ``runs`` (name -> run(w)), the weights taken in turn: one captured
        graph per way, and the ways timed in turn, round after round, each way's fastest round counting. So a
        clock that is still rising, or falls under load, meets every way alike, and the choice between two
        ways that are close does not follow the order in which they were measured."""
        import time
        graphs = {}
        for how, run in runs.items():
            run(weights[0])
            torch.cuda.synchronize(self.device)
            graph = torch.cuda.CUDAGraph()
            with torch.cuda.graph(graph):
                for i in range(launches):
                    run(weights[i % len(weights)])
            graph.replay()
            graphs[how] = graph
        torch.cuda.synchronize(self.device)
        best = {how: float("inf") for how in runs}
        for _ in range(rounds):
            for how, graph in graphs.items():
                t0 = time.perf_counter()
                graph.replay()
                torch.cuda.synchronize(self.device)
                best[how] = min(best[how], time.perf_counter() - t0)
        return {how: t / launches for how, t in best.items()}

    def _time_over(self, run, weights, launches):
        """Seconds per call of run(w), the weights taken in turn, launched from one captured graph."""
        import time
        run(weights[0])
        torch.cuda.synchronize(self.device)
        graph = torch.cuda.CUDAGraph()
        with torch.cuda.graph(graph):
            for i in range(launches):
                run(weights[i % len(weights)])
        graph.replay()
        torch.cuda.synchronize(self.device)
        best = float("inf")
        for _ in range(3):
            t0 = time.perf_counter()
            graph.replay()
            torch.cuda.synchronize(self.device)
            best = min(best, time.perf_counter() - t0)
        return best / launches

    # ------------------------------------------------------------------ attention
    MAX_HEAD_DIM = 512

    def check_attention_sizes(self, n_q, n_kv, D, dtype):
        """Raises for head counts and sizes that no attention kernel here takes (asked when a model is built)."""
        if D > self.MAX_HEAD_DIM or D < 1:
            raise KernelError(f"attention: head size {D} is beyond the kernels' {self.MAX_HEAD_DIM}")
        if n_kv < 1 or n_q % n_kv:
            raise KernelError(f"attention: {n_q} query heads over {n_kv} kv heads")
        _code(dtype)

    def prefill_tile_rows(self, D, dtype):
        """Rows per q tile of the lists that attention() reads from step.prefill_tiles for requests with
        more than one token (a tuple; the first is the one it needs, the others it uses when they are
        there), or None where the kernel that serves this head size takes no list."""
        if dtype == torch.bfloat16 and D % 16 == 0 and D <= 256:
            rows = int(self.lib.ra_attention_prefill_tile_rows(D))
            return (rows,) if rows == 64 else (rows, 64)
        return None

    def attention(self, q, out, k_pool, v_pool, step, group, scale, window=0, head_scale=None, softcap=0.0,
                  keep_first=0, sink=False, sink_logit=None, out_scale=1.0, fine_weights=False):
        """Attention of the step's queries over the paged cache. Optional: head_scale (fp32, one factor per query
        head on the scale), softcap c (score -> c tanh(score / c)), keep_first n (keys at positions below n
        stay visible whatever the window), sink (one more key of score 0 without a value in the softmax),
        sink_logit (fp32, one per query head: that key's score, neither scaled nor capped), out_scale (a factor on the
        result), fine_weights (bfloat16: the weights enter the product with the values with 16 bits of mantissa in
        place of 8). out: [T, n_q, D], tokens possibly further apart than n_q D (columns of wider rows)."""
        self._want(q, "q", dims=3)
        T, n_q, D = q.shape
        if out.device != self.device or out.dtype != q.dtype or out.dim() != 3 or (D > 1 and out.stride(2) != 1) or \
                (n_q > 1 and out.stride(1) != D) or (T > 1 and out.stride(0) < n_q * D):
            raise KernelError(f"attention: output {tuple(out.shape)} with strides {out.stride()} of {out.dtype} on {out.device}")
        ld_out = out.stride(0) if T > 1 else max(n_q * D, out.stride(0))
        g = step.groups[group]
        n_kv = k_pool.shape[1]
        self._pool_rows(k_pool, v_pool, n_kv, D, q.dtype)
        if out.shape != q.shape or T != step.n_tokens:
            raise KernelError(f"attention: q {tuple(q.shape)}, out {tuple(out.shape)}, step of {step.n_tokens}")
        if n_q % n_kv:
            raise KernelError(f"attention: {n_q} query heads over {n_kv} kv heads")
        self.check_attention_sizes(n_q, n_kv, D, q.dtype)
        P = k_pool.shape[2]
        window = int(window)
        tabs = (_ptr(g.page_table), _ptr(g.cu_pages), _ptr(g.kv_start), _ptr(step.cu_q), _ptr(step.q_start))
        softcap, keep_first, sink = float(softcap or 0.0), int(keep_first or 0), bool(sink)
        if head_scale is not None:
            self._want(head_scale, "head scale", torch.float32, 1)
            if head_scale.shape[0] != n_q:
                raise KernelError(f"attention: head scale {tuple(head_scale.shape)} for {n_q} heads")
        out_scale = float(out_scale)
        if sink_logit is not None:
            self._want(sink_logit, "sink logits", torch.float32, 1)
            if sink_logit.shape[0] != n_q:
                raise KernelError(f"attention: sink logits {tuple(sink_logit.shape)} for {n_q} heads")
            sink = True
        fine_weights = bool(fine_weights)
        if q.dtype == torch.bfloat16 and D % 16 == 0 and D <= 256 and (ld_out % 4 or out.data_ptr() % 8):
            raise KernelError(f"attention: output rows {ld_out} elements apart, or not aligned to four elements")
        extras = head_scale is not None or softcap > 0.0 or keep_first > 0 or sink or out_scale != 1.0 or fine_weights \
            or ld_out != n_q * D
        fast_decode = q.dtype == torch.bfloat16 and step.n_decode > 0 and D % 16 == 0 and D <= 256
        fast_prefill = q.dtype == torch.bfloat16 and bool(step.prefill_tiles) and D % 16 == 0 and D <= 256 and \
            (fast_decode or step.n_decode == 0)

        def decode_part():
            S, max_splits, merge = self._decode_splits(step, n_q, n_kv, D, window)
            if keep_first > 0 and window > 0:
                max_splits += 1                  # the kept keys below the window are a split of their own
            nd = step.n_decode
            part_acc = part_ml = None
            if not merge:
                part_acc = torch.empty(nd, n_q, max_splits, D, dtype=torch.float32, device=self.device)
                part_ml = torch.empty(nd, n_q, max_splits, 2, dtype=torch.float32, device=self.device)
            if extras:
                self._check(self.lib.ra_attention_decode_extras_bf16(
                    _ptr(q), _ptr(out), _ptr(part_acc), _ptr(part_ml), _ptr(k_pool), _ptr(v_pool), *tabs,
                    _ptr(step.decode_segs), nd, n_q, n_kv, D, P, float(scale), window, S, max_splits,
                    1 if merge else 0, _ptr(head_scale), softcap, keep_first, 1 if sink else 0, _ptr(sink_logit), out_scale,
                    ld_out, 1 if fine_weights else 0, self._stream()), "attention_decode_extras_bf16")
                return
            self._check(self.lib.ra_attention_decode_bf16(
                _ptr(q), _ptr(out), _ptr(part_acc), _ptr(part_ml), _ptr(k_pool), _ptr(v_pool), *tabs,
                _ptr(step.decode_segs), nd, n_q, n_kv, D, P, float(scale), window, S, max_splits,
                1 if merge else 0, self._stream()), "attention_decode_bf16")

        def prefill_part():
            rows = self.lib.ra_attention_prefill_tile_rows(D)
            tiles = step.prefill_tiles.get(rows)
            if tiles is None:
                raise KernelError(f"attention: the step lists no q tiles of {rows} rows (head size {D})")
            # Few tiles (a portion of 512 rows is four or five of 128 rows: 128 to 160 workgroups with 32
            # heads) leave CUs idle: tiles of 64 rows, one group of rows per wave and two groups of waves a
            # tile, make twice the workgroups of less than half the work each (measured at 32 heads of 128:
            # 512 rows over 4,096 keys 78 µs against 109, 300 rows at 1,500 beside 212 from scratch 36
            # against 50; from 1,024 rows on slower)
            small = step.prefill_tiles.get(64) if rows == 128 else None
            small_split = 0
            if small is not None and self.prefill_small_tiles and 2 * small.shape[0] * n_q <= 3 * self.cu_count:
                rows, tiles, small_split = 64, small, 2
            split = self.prefill_key_split or small_split or self._prefill_key_split(step, rows, tiles.shape[0] * n_q)
            self._check(self.lib.ra_attention_prefill_bf16(
                _ptr(q), _ptr(out), _ptr(k_pool), _ptr(v_pool), *tabs, _ptr(tiles), tiles.shape[0], rows,
                split, n_q, n_kv, D, P, float(scale), window, _ptr(head_scale), softcap, keep_first,
                1 if sink else 0, _ptr(sink_logit), out_scale, ld_out, 1 if fine_weights else 0, self._stream()),
                "attention_prefill_bf16")

        def plain_part(toks, n_tok):
            self._check(self.lib.ra_attention_plain(
                _ptr(q), _ptr(out), _ptr(k_pool), _ptr(v_pool), *tabs, _ptr(toks), step.n_seqs, n_tok,
                n_q, n_kv, D, P, float(scale), window, _code(q.dtype), _ptr(head_scale), softcap, keep_first,
                1 if sink else 0, _ptr(sink_logit), out_scale, ld_out, self._stream()), "attention_plain")

        if fast_decode and fast_prefill and step.n_prefill_tokens > 0:
            # A step of prompt portions beside decoded tokens: the two kernels work on different rows of q and
            # out, one is bound by memory and the other by the matrix cores and the latency inside its waves,
            # so they run side by side on two streams (never while a graph is being captured: such steps are
            # not captured anyway, and a fork and join inside a graph costs more than it gives).
            if self.overlap_attention and not torch.cuda.is_current_stream_capturing():
                main = torch.cuda.current_stream(self.device)
                if self._side_stream is None:
                    self._side_stream = torch.cuda.Stream(self.device)      # (default priority, like every stream here)
                side = self._side_stream
                side.wait_stream(main)               # q and the new keys and values are written
                with torch.cuda.stream(side):
                    prefill_part()
                decode_part()
                main.wait_stream(side)               # what follows reads both kernels' rows of out
            else:
                decode_part()
                prefill_part()
            return
        if fast_decode:
            decode_part()
            if step.n_prefill_tokens == 0:
                return
            toks, n_tok = step.prefill_toks, step.n_prefill_tokens
        else:
            toks, n_tok = None, T
        if fast_prefill:
            prefill_part()
            return
        plain_part(toks, n_tok)

    def _decode_splits(self, step, n_q, n_kv, D, window):
        """Keys per split of the decode attention, the most splits a request has, and whether a
        request's splits are the waves of one workgroup that merges them itself (no partial sums
        in memory, no merge kernel). Measured on MI355X: that is 3 to 11 % faster when the
        (request, kv head) pairs are a whole number of rounds over the CUs (batch 32, 64, 96, 128 with
        8 kv heads) or at least three rounds (batch 100 of uneven lengths: 208 against 221 µs), and
        slower otherwise (batch 40, 48, 72: 5 to 15 %): a workgroup of eight waves fills a CU's LDS, and
        a last round that is far from full leaves most of the chip idle."""
        longest = step.max_decode_seq_len
        # what the choice is based on: the step's own numbers, or the class its runner names (then a step run
        # eagerly and its replay from a graph choose alike and sum in the same order)
        rule = getattr(step, "decode_rule", None)
        n_rule, l_rule = rule if rule else (step.n_decode, longest)
        S = self.decode_split_tokens
        groups = n_rule * n_kv * -(-(n_q // n_kv) // 16)
        waves = self.lib.ra_attention_decode_merge_waves(D)
        if S <= 0 and window == 0 and waves >= 2 and l_rule > 64 and self.decode_merge_round > 0 \
                and (groups % self.decode_merge_round == 0 or groups >= 3 * self.decode_merge_round):
            # (the kernel cuts every request into W even splits of its own length)
            # Waves of such a workgroup (measured, 8 kv heads of 128, batch 32 to 128, contexts of 2,048 and
            # 8,192, even and uneven lengths): with fewer waves more workgroups share a CU and one's start and
            # merge run while another reads. Two are 3 to 9 % faster from two rounds of pairs on with contexts
            # up to 4,096 (and 2 % slower with longer, uneven ones), four up to 5 % faster below two rounds.
            want = self.decode_merge_waves
            if want <= 0:
                want = 4 if groups < 2 * self.decode_merge_round else (2 if l_rule <= 4096 else 8)
            W = min(want, waves, -(-l_rule // 64))
            return 64, max(W, 2), True
        if S <= 0:
            # about two thousand waves in all (eight per CU) fill the chip; fewer, longer
            # splits spend less on starting up and on the merge (measured from 1 to 128 requests)
            # (a few hundred waves do not fill it: then a wave takes one pass of 64 keys and all of a
            # request's loads are on their way at once; batch 1 over 2,048 keys 10.0 against 10.8 µs, batch 2
            # 11.8 against 12.4, from about a thousand waves on 15.4 against 14.8)
            chunks = n_rule * n_kv * ((l_rule + 63) // 64)
            S = 64 * max(1 if chunks <= 640 else 2, -(-chunks // 2048), -(-l_rule // 4096))     # and at most 64 splits a request
            if rule or getattr(step, "decode_len_is_bound", False):
                # the lengths lie somewhere below the bound (a graph's context bucket): splits
                # of at most an eighth of it keep the work of a request even
                S = min(S, max(128 if S > 64 else 64, l_rule // 8 // 64 * 64))
        max_splits = (longest - 1) // S + 1
        if window > 0:                       # a window spans at most this many splits
            max_splits = min(max_splits, (window + S - 2) // S + 1)
        return S, max_splits, False

    def attention_qkv(self, qkv, out, k_pool, v_pool, step, group, scale, window, n_q, n_kv, D,
                      w_q, w_k, eps, cos, sin, rotary_dim):
        """Attention of a step in which every request brings one token, straight from the q/k/v
        projection: the decode kernel norms and rotates q and k itself and writes k and v into
        the cache, which saves the preparation kernel. Returns False, having done nothing, when
        the step or the sizes are not such (then qkv_prepare and attention do the work)."""
        if qkv.dtype != torch.bfloat16 or step.n_decode != step.n_seqs or step.n_prefill_tokens != 0:
            return False
        R = int(rotary_dim)
        if D % 64 or D > 256 or R not in (0, D) or (w_q is None) != (w_k is None):
            return False
        self._want(qkv, "qkv", torch.bfloat16, 2)
        self._want(out, "attention output", torch.bfloat16, 3)
        T = qkv.shape[0]
        g = step.groups[group]
        self._pool_rows(k_pool, v_pool, n_kv, D, torch.bfloat16)
        if qkv.shape[1] != (n_q + 2 * n_kv) * D or tuple(out.shape) != (T, n_q, D) or T != step.n_tokens or n_q % n_kv:
            raise KernelError(f"attention_qkv: qkv {tuple(qkv.shape)}, out {tuple(out.shape)}, "
                              f"{n_q} heads over {n_kv} of {D}, step of {step.n_tokens}")
        if w_q is not None:
            for w in (w_q, w_k):
                self._want(w, "head norm weight", torch.float32, 1)
                if w.shape[0] != D:
                    raise KernelError(f"attention_qkv: norm weight {tuple(w.shape)} for head size {D}")
        if R:
            self._want(cos, "cos table", torch.float32, 2)
            self._want(sin, "sin table", torch.float32, 2)
            if cos.shape[1] != D // 2 or sin.shape != cos.shape:
                raise KernelError(f"attention_qkv: tables {tuple(cos.shape)} for head size {D}")
        P = k_pool.shape[2]
        window = int(window)
        S, max_splits, merge = self._decode_splits(step, n_q, n_kv, D, window)
        nd = step.n_decode
        part_acc = part_ml = None
        if not merge:
            part_acc = torch.empty(nd, n_q, max_splits, D, dtype=torch.float32, device=self.device)
            part_ml = torch.empty(nd, n_q, max_splits, 2, dtype=torch.float32, device=self.device)
        self._check(self.lib.ra_attention_decode_fused_bf16(
            _ptr(qkv), _ptr(out), _ptr(part_acc), _ptr(part_ml), _ptr(k_pool), _ptr(v_pool),
            # (no cu_q: every request brings one token, checked above, so request i is row i)
            _ptr(g.page_table), _ptr(g.cu_pages), _ptr(g.kv_start), None, _ptr(step.q_start),
            None, nd, n_q, n_kv, D, P, float(scale), window, S, max_splits,
            _ptr(w_q), _ptr(w_k), float(eps), _ptr(cos) if R else None, _ptr(sin) if R else None,
            1 if merge else 0, self._stream()), "attention_decode_fused_bf16")
        return True

    @staticmethod
    def _prefill_key_split(step, rows, n_workgroups):
        """Whether two groups of waves should share each q tile's keys (measured on MI355X): yes
        while the workgroups do not fill the chip, and up to three per CU when the longest tile
        reads far more keys than the average one, since then the longest tile decides the time."""
        if n_workgroups <= 256:
            return 2
        if n_workgroups > 768:
            return 1
        ends = [s + min(off + rows, q) for q, s in zip(step.q_lens, step.q_starts) if q != 1
                for off in range(0, q, rows)]
        return 2 if max(ends) * len(ends) >= 1.4 * sum(ends) else 1

    # ------------------------------------------------------------------ differential attention
    def check_attention_diff_sizes(self, n_q, n_kv, D, Dv, dtype):
        """Raises for sizes that no differential attention kernel here takes (asked when a model is built)."""
        if n_kv < 1 or n_q % n_kv or n_q > 65535:
            raise KernelError(f"differential attention: {n_q} query heads over {n_kv} kv heads")
        if not self.lib.ra_attention_diff_plain_fits(int(D), int(Dv)):
            raise KernelError(f"differential attention: maps of {D} with values of {Dv} are beyond the kernels")
        _code(dtype)

    def _pools_two_widths(self, k_pool, v_pool, n_kv, Dk, Dv, dtype):
        for t, name, width in ((k_pool, "k pool", Dk), (v_pool, "v pool", Dv)):
            self._want(t, name, dtype, 4)
            if t.shape[1] != n_kv or t.shape[3] != width:
                raise KernelError(f"{name} {tuple(t.shape)} does not hold {n_kv} heads of {width}")
        if k_pool.shape[:3] != v_pool.shape[:3]:
            raise KernelError("k pool and v pool differ in pages, heads or rows")
        if k_pool.shape[0] * k_pool.shape[1] * k_pool.shape[2] >= 2 ** 31:
            raise KernelError(f"k pool {tuple(k_pool.shape)}: the kernels count head rows in 32 bits")
        return k_pool.shape[0] * k_pool.shape[2]

    def maps_qkv_prepare(self, qkv, n_q, n_kv, maps, D, Dv, positions, cos, sin, rotary_dim, interleaved, q_out,
                         k_pool, v_pool, slot_mapping):
        """q/k/v preparation of an attention with several score maps per head: rows of qkv are
        [n_q * maps * D | n_kv * maps * D | n_kv * Dv]; the first rotary_dim elements of every map of q and k are
        rotated (pairs 2i, 2i + 1 when interleaved, else i, i + rotary_dim / 2); q to q_out [T, n_q, maps * D],
        k and v to the rows of the pools that slot_mapping names (pools None: nothing is written)."""
        self._want(qkv, "qkv", dims=2)
        self._want(q_out, "q", qkv.dtype, 3)
        self._want(positions, "positions", torch.int32, 1)
        T, R = qkv.shape[0], int(rotary_dim)
        if qkv.shape[1] != (n_q + n_kv) * maps * D + n_kv * Dv or tuple(q_out.shape) != (T, n_q, maps * D) \
                or positions.shape[0] != T:
            raise KernelError(f"maps_qkv_prepare: qkv {tuple(qkv.shape)}, q {tuple(q_out.shape)}, {T} tokens")
        if R:
            self._want(cos, "cos table", torch.float32, 2)
            self._want(sin, "sin table", torch.float32, 2)
            if R % 2 or R > D or cos.shape[1] != R // 2 or sin.shape != cos.shape:
                raise KernelError(f"maps_qkv_prepare: rotary_dim {R}, tables {tuple(cos.shape)}, map size {D}")
        P = 1
        if k_pool is not None:
            self._want(slot_mapping, "slot mapping", torch.int32, 1)
            if slot_mapping.shape[0] != T:
                raise KernelError("maps_qkv_prepare: slot mapping does not match the token count")
            self._pools_two_widths(k_pool, v_pool, n_kv, maps * D, Dv, qkv.dtype)
            P = k_pool.shape[2]
        self._check(self.lib.ra_maps_qkv_prepare(
            _ptr(qkv), T, n_q, n_kv, maps, D, Dv, _ptr(positions), _ptr(cos) if R else None, _ptr(sin) if R else None,
            R, 1 if interleaved else 0, _ptr(q_out), _ptr(k_pool), _ptr(v_pool),
            _ptr(slot_mapping) if k_pool is not None else None, P, _code(qkv.dtype), self._stream()), "maps_qkv_prepare")

    def diff_prefill_tile_rows(self, D, Dv, dtype):
        """Rows per q tile of the lists that attention_diff reads from step.prefill_tiles, or None where the
        kernel that serves these sizes takes no list."""
        if dtype == torch.bfloat16 and self.lib.ra_attention_diff_mfma_fits(int(D), int(Dv)):
            return (64,)
        return None

    def attention_diff(self, q, out, k_pool, v_pool, step, group, scale, lam, eps, out_scale, window=0, chunk=0):
        """Differential attention of the step's queries over the paged cache: q [T, n_q, 2 D] (two maps a head),
        key pool rows [2 D], value pool rows [Dv], out [T, n_q, Dv] = norm(a1 - lam a2) * out_scale."""
        self._want(q, "q", dims=3)
        self._want(out, "attention output", q.dtype, 3)
        T, n_q, D2 = q.shape
        Dv = out.shape[2]
        g = step.groups[group]
        n_kv = k_pool.shape[1]
        if D2 % 2 or tuple(out.shape[:2]) != (T, n_q) or T != step.n_tokens:
            raise KernelError(f"attention_diff: q {tuple(q.shape)}, out {tuple(out.shape)}, step of {step.n_tokens}")
        self._pools_two_widths(k_pool, v_pool, n_kv, D2, Dv, q.dtype)
        self.check_attention_diff_sizes(n_q, n_kv, D2 // 2, Dv, q.dtype)
        P = k_pool.shape[2]
        tabs = (_ptr(g.page_table), _ptr(g.cu_pages), _ptr(g.kv_start), _ptr(step.cu_q), _ptr(step.q_start))
        consts = (float(scale), int(window), int(chunk), float(lam), float(eps), float(out_scale))

        if q.dtype == torch.bfloat16 and scale > 0 and self.lib.ra_attention_diff_mfma_fits(D2 // 2, Dv):
            # the matrix-core kernel, tile by tile: the q tiles of the requests with two or more new tokens, and
            # one tile of one row for every request that brings a single token
            lists = []
            if step.n_prefill_tokens > 0:
                tiles = step.prefill_tiles.get(64) if getattr(step, "prefill_tiles", None) else None
                if tiles is None:
                    raise KernelError("attention_diff: the step lists no q tiles of 64 rows")
                lists.append((tiles, 1, 0))
            if step.n_decode > 0:
                if step.decode_segs is None:             # every request brings one token: request i is tile (i, 0)
                    if step.n_decode > self._unit_tiles.shape[0]:
                        self._unit_tiles = self._make_unit_tiles(2 * step.n_decode)
                    tiles = self._unit_tiles[:step.n_decode]
                else:
                    tiles = torch.stack([step.decode_segs, torch.zeros_like(step.decode_segs)], dim=1).contiguous()
                # (one kv head's group of query heads as the rows of one workgroup, where it fits a tile of rows)
                pack = 1 if n_q // n_kv <= 16 else 0
                lists.append((tiles, self._diff_decode_splits(step, n_kv if pack else n_q, int(window), int(chunk)), pack))
            for tiles, splits, pack in lists:
                part = None
                if splits > 1:
                    part = torch.empty(tiles.shape[0] * n_q * splits * 2 * (Dv + 2), dtype=torch.float32, device=self.device)
                self._check(self.lib.ra_attention_diff_mfma_bf16(
                    _ptr(q), _ptr(out), _ptr(k_pool), _ptr(v_pool), *tabs, _ptr(tiles), tiles.shape[0], n_q, n_kv,
                    D2 // 2, Dv, P, *consts, splits, _ptr(part), pack, self._stream()), "attention_diff_mfma_bf16")
            return
        # float32, and sizes the matrix-core kernel does not take: the plain kernel over all rows of the step
        self._check(self.lib.ra_attention_diff_plain(
            _ptr(q), _ptr(out), _ptr(k_pool), _ptr(v_pool), *tabs, None, 0, step.n_seqs, T, n_q, n_kv, D2 // 2, Dv, P,
            *consts, _code(q.dtype), self._stream()), "attention_diff_plain")

    def _diff_decode_splits(self, step, n_heads, window, chunk, per_cu=8, least=4):
        """Workgroups that share the keys of a request that brings one token: enough of them to fill the chip
        (about `per_cu` a CU), at least `least` blocks of 64 keys each. Decided by the step's class (the batch size and
        context bucket of the graph that serves or would serve it) where the runner names one, so that a step run
        eagerly and its replay from a graph sum in the same order."""
        rule = getattr(step, "decode_rule", None)
        n, longest = rule if rule else (step.n_decode, getattr(step, "max_decode_seq_len", 0))
        keys = longest
        if window > 0:
            keys = min(keys, window)
        if chunk > 0:
            keys = min(keys, chunk)
        blocks = -(-max(int(keys), 1) // 64)
        want = -(-per_cu * self.cu_count // max(1, n * n_heads))
        return int(max(1, min(64, want, blocks // least)))

    # ------------------------------------------------------------------ attention over a latent row per token
    def check_attention_latent_sizes(self, n_heads, C, R, dtype):
        """Raises for sizes that no latent attention kernel here takes (asked when a model is built)."""
        if n_heads < 1 or not self.lib.ra_attention_latent_plain_fits(int(C), int(R)):
            raise KernelError(f"latent attention: {n_heads} heads over rows of {C} + {R} are beyond the kernels")
        _code(dtype)

    def latent_kv_prepare(self, z, Q, C, R, wq_norm, wkv_norm, eps, positions, cos, sin, rotary_dim, cq_out,
                          k_pool, v_pool, slot_mapping, q=None, qq_out=None):
        """From the rows z = [a: Q | b: C | r: R | ...]: cq_out = rmsnorm(a) wq_norm (Q 0: no such part, both None);
        rmsnorm(b) wkv_norm to the value pool's rows and r, its first rotary_dim elements turned by the position (element i
        with i + rotary_dim / 2), to the key pool's rows that slot_mapping names (pools None: not written). With q (rows
        [T, H (D + R)], possibly a column slice of wider rows) and qq_out [T, H, C + R] also latent_q_prepare's rotated
        part, qq_out[t, h, C:] = q[t, h, D:] turned, by the same kernel."""
        ld = self._want_rows(z, "latent rows")
        self._want(positions, "positions", torch.int32, 1)
        self._want(wkv_norm, "latent norm weight", torch.float32, 1)
        T, rot = z.shape[0], int(rotary_dim)
        if Q:
            self._want(cq_out, "query latent", z.dtype, 2)
            self._want(wq_norm, "query latent norm weight", torch.float32, 1)
            if tuple(cq_out.shape) != (T, Q) or wq_norm.shape[0] != Q:
                raise KernelError(f"latent_kv_prepare: cq {tuple(cq_out.shape)}, its norm {tuple(wq_norm.shape)} for {Q}")
        if z.shape[1] < Q + C + R or positions.shape[0] != T or wkv_norm.shape[0] != C:
            raise KernelError(f"latent_kv_prepare: z {tuple(z.shape)} for {Q} + {C} + {R}")
        if rot:
            self._want(cos, "cos table", torch.float32, 2)
            self._want(sin, "sin table", torch.float32, 2)
            if rot % 2 or rot > R or cos.shape[1] != rot // 2 or sin.shape != cos.shape:
                raise KernelError(f"latent_kv_prepare: rotary_dim {rot}, tables {tuple(cos.shape)}, key part {R}")
        ld_q, Hn, D = 0, 0, 0
        if q is not None:
            ld_q = self._want_rows(q, "query rows", z.dtype)
            self._want(qq_out, "prepared q", z.dtype, 3)
            Hn = qq_out.shape[1]
            D = q.shape[1] // Hn - R
            if qq_out.shape[0] != T or qq_out.shape[2] != C + R or D < 0 or tuple(q.shape) != (T, Hn * (D + R)):
                raise KernelError(f"latent_kv_prepare: q {tuple(q.shape)}, prepared q {tuple(qq_out.shape)}")
        P = 1
        if k_pool is not None:
            self._want(slot_mapping, "slot mapping", torch.int32, 1)
            if slot_mapping.shape[0] != T:
                raise KernelError("latent_kv_prepare: slot mapping does not match the token count")
            self._pools_two_widths(k_pool, v_pool, 1, R, C, z.dtype)
            P = k_pool.shape[2]
            k_pool = k_pool if R else None               # (no rotated part: the key pool's rows are empty)
        self._check(self.lib.ra_latent_kv_prepare(
            _ptr(z), ld, T, int(Q), int(C), int(R), _ptr(wq_norm) if Q else None, _ptr(wkv_norm), float(eps), _ptr(positions),
            _ptr(cos) if rot else None, _ptr(sin) if rot else None, rot, _ptr(cq_out) if Q else None, _ptr(k_pool), _ptr(v_pool),
            _ptr(slot_mapping) if v_pool is not None else None, P, _ptr(q), ld_q, Hn, D, _ptr(qq_out) if q is not None else None,
            _code(z.dtype), self._stream()), "latent_kv_prepare")

    def latent_q_prepare(self, q, q_lat, D, R, positions, cos, sin, rotary_dim, qq_out):
        """qq_out [T, H, C + R] = [q_lat[h, t] | q[t, h, D:] with its first rotary_dim elements turned]; q [T, H (D + R)],
        q_lat [H, T, C] (None: the first C elements are there already)."""
        self._want(q, "q", dims=2)
        self._want(qq_out, "prepared q", q.dtype, 3)
        self._want(positions, "positions", torch.int32, 1)
        T, Hn, CR = qq_out.shape
        C, rot = CR - R, int(rotary_dim)
        if q_lat is not None:
            self._want(q_lat, "q over the latent", q.dtype, 3)
            if tuple(q_lat.shape) != (Hn, T, C):
                raise KernelError(f"latent_q_prepare: q_lat {tuple(q_lat.shape)}, out {tuple(qq_out.shape)}")
        if tuple(q.shape) != (T, Hn * (D + R)) or C < 1 or positions.shape[0] != T:
            raise KernelError(f"latent_q_prepare: q {tuple(q.shape)}, out {tuple(qq_out.shape)}")
        if rot:
            self._want(cos, "cos table", torch.float32, 2)
            self._want(sin, "sin table", torch.float32, 2)
            if rot % 2 or rot > R or cos.shape[1] != rot // 2 or sin.shape != cos.shape:
                raise KernelError(f"latent_q_prepare: rotary_dim {rot}, tables {tuple(cos.shape)}, rotated part {R}")
        self._check(self.lib.ra_latent_q_prepare(
            _ptr(q), _ptr(q_lat), T, Hn, int(D), int(R), C, _ptr(positions), _ptr(cos) if rot else None,
            _ptr(sin) if rot else None, rot, _ptr(qq_out), _code(q.dtype), self._stream()), "latent_q_prepare")

    def attention_latent(self, qq, out, k_pool, v_pool, step, group, scale, sink=None, window=0):
        """Attention of the step's queries qq [T, H, C + R] over the rows [c | kr] that the value pool (rows of C)
        and the key pool (rows of R) hold for every token; softmax with exp(sink[h]) in its denominator (sink None:
        none); out [H, T, C] = sum_j p_j c_j. window w > 0: the query at position i reads the keys j with
        0 <= i - j < w. The key pool's rows may be empty (R = 0)."""
        self._want(qq, "q", dims=3)
        self._want(out, "attention output", qq.dtype, 3)
        T, Hn, CR = qq.shape
        C, R = v_pool.shape[3], k_pool.shape[3]
        g = step.groups[group]
        if CR != C + R or tuple(out.shape) != (Hn, T, C) or T != step.n_tokens:
            raise KernelError(f"attention_latent: q {tuple(qq.shape)}, out {tuple(out.shape)}, rows of {C} + {R}, "
                              f"step of {step.n_tokens}")
        self._pools_two_widths(k_pool, v_pool, 1, R, C, qq.dtype)
        self.check_attention_latent_sizes(Hn, C, R, qq.dtype)
        if sink is not None:
            self._want(sink, "sink", torch.float32, 1)
            if sink.shape[0] != Hn:
                raise KernelError(f"attention_latent: sink {tuple(sink.shape)} for {Hn} heads")
        P = k_pool.shape[2]
        window = int(window or 0)
        if window < 0:
            raise KernelError(f"attention_latent: window {window}")
        tabs = (_ptr(g.page_table), _ptr(g.cu_pages), _ptr(g.kv_start), _ptr(step.cu_q), _ptr(step.q_start))
        if qq.dtype == torch.bfloat16 and scale > 0 and self.lib.ra_attention_latent_mfma_fits(C, R, Hn):
            # the matrix-core kernel, tile by tile: the q tiles of the requests with two or more new tokens (64 / heads
            # tokens a tile), and one tile for every request that brings a single token
            lists = []
            if step.n_prefill_tokens > 0:
                rows = int(self.lib.ra_attention_latent_mfma_tile_tokens(Hn))
                tiles = step.prefill_tiles.get(rows) if getattr(step, "prefill_tiles", None) else None
                if tiles is None:
                    raise KernelError(f"attention_latent: the step lists no q tiles of {rows} rows")
                lists.append((tiles, 1))
            if step.n_decode > 0:
                if step.decode_segs is None:             # every request brings one token: request i is tile (i, 0)
                    if step.n_decode > self._unit_tiles.shape[0]:
                        self._unit_tiles = self._make_unit_tiles(2 * step.n_decode)
                    tiles = self._unit_tiles[:step.n_decode]
                else:
                    tiles = torch.stack([step.decode_segs, torch.zeros_like(step.decode_segs)], dim=1).contiguous()
                # A block of 64 keys is 6.7 µs of one workgroup's time whatever the heads, and a workgroup's tile of long
                # rows fills half a CU's LDS: one workgroup a CU, down to one block each (measured with rows of 512 + 64
                # at 16 and 32 heads: 2,048 keys, batch 1 23 µs against 39 with four blocks at least, batch 8 26 against
                # 40; batch 64 73 with one workgroup a CU against 80 with two and 93 with four; 8,192 keys 38 against 121,
                # 50 against 124, 266 against 277)
                lists.append((tiles, self._diff_decode_splits(step, 1, window, 0, 1 if C + R >= 320 else 2, 1)))
            for tiles, splits in lists:
                part = None
                if splits > 1:
                    part = torch.empty(tiles.shape[0] * Hn * splits * (C + 2), dtype=torch.float32, device=self.device)
                self._check(self.lib.ra_attention_latent_mfma_window_bf16(
                    _ptr(qq), _ptr(out), _ptr(k_pool), _ptr(v_pool), *tabs, _ptr(tiles), tiles.shape[0], T, Hn, C, R, P,
                    float(scale), _ptr(sink), splits, _ptr(part), window, self._stream()), "attention_latent_mfma_bf16")
            return
        # float32, and sizes the matrix-core kernel does not take: the plain kernel over all rows of the step
        self._check(self.lib.ra_attention_latent_plain_window(
            _ptr(qq), _ptr(out), _ptr(k_pool), _ptr(v_pool), *tabs, None, step.n_seqs, T, T, Hn, C, R, P, float(scale),
            _ptr(sink), 1 if step.all_decode else 0, window, _code(qq.dtype), self._stream()), "attention_latent_plain")

    def latent_prefill_tile_rows(self, n_heads, C, R, dtype):
        """Rows (tokens) per q tile of the lists that attention_latent reads from step.prefill_tiles, or None where
        the kernel that serves these sizes takes no list."""
        if dtype == torch.bfloat16 and self.lib.ra_attention_latent_mfma_fits(int(C), int(R), int(n_heads)):
            return (int(self.lib.ra_attention_latent_mfma_tile_tokens(int(n_heads))),)
        return None

    # ------------------------------------------------------------------ routed experts
    MAX_EXPERTS = 1024

    def check_moe_sizes(self, experts, top, groups, keep):
        if not 1 <= experts <= self.MAX_EXPERTS or not 1 <= top <= min(64, experts) or groups < 1 or experts % groups \
                or not 1 <= keep <= groups or keep * (experts // groups) < top:
            raise KernelError(f"routed experts: {experts} experts, top {top}, {groups} groups of which {keep} stay "
                              f"are beyond the kernels (at most {self.MAX_EXPERTS} experts, top 64)")

    def moe_route(self, z, bias, top, groups, keep, norm_eps, law="sigmoid_groups"):
        """Router logits z [T, E] (32-bit) -> (ids int32 [T, top], weights fp32 [T, top]). law "softmax_top": the
        largest z + bias are taken and weighed by the softmax over them alone. law "softmax_groups": the choice is made
        on s = softmax(z) over all experts, a group scores its largest s, the weights are the chosen s as they are. law
        "sigmoid_raw": as "sigmoid_groups", but the weights are the chosen s as they are."""
        laws = {"sigmoid_groups": 0, "softmax_top": 1, "softmax_groups": 2, "sigmoid_raw": 3}
        if law not in laws:
            raise KernelError(f"moe_route: no router law {law!r}")
        ld_z = self._want_rows(z, "router logits", torch.float32)
        T, E = z.shape
        self.check_moe_sizes(E, top, groups, keep)
        if bias is not None:
            self._want(bias, "router correction", torch.float32, 1)
            if bias.shape[0] != E:
                raise KernelError(f"moe_route: correction {tuple(bias.shape)} for {E} experts")
        ids = torch.empty(T, top, dtype=torch.int32, device=self.device)
        weights = torch.empty(T, top, dtype=torch.float32, device=self.device)
        self._check(self.lib.ra_moe_route_law(_ptr(z), ld_z, _ptr(bias), T, E, int(top), int(groups), int(keep), float(norm_eps),
                                              _ptr(ids), _ptr(weights),
                                              laws[law], self._stream()),
                    "moe_route")
        return ids, weights

    def moe_experts(self, x, ids, weights, w_gate_up, w_down, activation="silu", limit=0.0, slope=1.702, extra=None,
                    extra_logits=None, weigh="output", combine=True):
        """sum_k weights[t, k] * down_e(silu(gate_e x_t) * up_e x_t), e = ids[t, k]; w_gate_up [E, 2I, H] (gate
        rows first), w_down [E, H, I]. The pairs are grouped by expert on the device. activation "clamped": an
        expert is down(g sigmoid(slope g) (u + 1)) with g = min(gate x, limit), u = clamp(up x, -limit, limit).
        extra [T, H] with extra_logits [T, 1] (possibly a column of wider rows): one more term of every token's sum,
        extra[t] * sigmoid(extra_logits[t]), added last in the same 32-bit sum (extra_logits in x's type or fp32).
        weigh "input": a weight multiplies what its expert reads, down_e(act(gate_e (w x), up_e (w x))), and the sum is a
        plain one. combine False: the sum is not formed; returns RowSums (extra_logits must then be fp32) for whatever forms
        the stream next."""
        if weigh not in ("output", "input"):
            raise KernelError(f"moe_experts: weigh {weigh!r}: 'output' or 'input'")
        if activation not in ("silu", "clamped") or (activation == "clamped" and not limit > 0):
            raise KernelError(f"moe_experts: activation {activation!r} with limit {limit}")
        act = 1 if activation == "clamped" else 0
        self._want(x, "rows", dims=2)
        self._want(ids, "expert ids", torch.int32, 2)
        self._want(weights, "expert weights", torch.float32, 2)
        self._want(w_gate_up, "gate-up matrices", x.dtype, 3)
        self._want(w_down, "down matrices", x.dtype, 3)
        T, H = x.shape
        E, I2, _ = w_gate_up.shape
        top, I = ids.shape[1], I2 // 2
        if tuple(ids.shape) != (T, top) or weights.shape != ids.shape or w_gate_up.shape[2] != H or I2 % 2 \
                or tuple(w_down.shape) != (E, H, I):
            raise KernelError(f"moe_experts: x {tuple(x.shape)}, ids {tuple(ids.shape)}, gate-up {tuple(w_gate_up.shape)}, "
                              f"down {tuple(w_down.shape)}")
        n_pairs, code = T * top, _code(x.dtype)
        ld_logits = 0
        if (extra is None) != (extra_logits is None):
            raise KernelError("moe_experts: a further term needs its rows and its gate logits")
        if extra is not None:
            self._want(extra, "further term", x.dtype, 2)
            ld_logits = self._want_rows(extra_logits, "gate logits of the further term")
            if extra_logits.dtype not in (x.dtype, torch.float32) or (not combine and extra_logits.dtype != torch.float32):
                raise KernelError(f"moe_experts: gate logits of the further term in {extra_logits.dtype}")
            if tuple(extra.shape) != (T, H) or tuple(extra_logits.shape) != (T, 1):
                raise KernelError(f"moe_experts: further term {tuple(extra.shape)}, its logits {tuple(extra_logits.shape)}")
        if n_pairs == 0:
            return torch.empty(T, H, dtype=x.dtype, device=self.device)
        mid = torch.empty(n_pairs, I, dtype=x.dtype, device=self.device)
        y = torch.empty(n_pairs, H, dtype=x.dtype, device=self.device)

        def plan(rows):
            # (every expert may end in a tile that is not full)
            max_tiles = min(n_pairs, n_pairs // rows + E)
            order = torch.empty(n_pairs, dtype=torch.int32, device=self.device)
            tiles = torch.empty(max_tiles, 3, dtype=torch.int32, device=self.device)
            meta = torch.empty(1, dtype=torch.int32, device=self.device)
            self._check(self.lib.ra_moe_plan(_ptr(ids), n_pairs, E, rows, _ptr(order), _ptr(tiles), _ptr(meta),
                                             self._stream()), "moe_plan")
            return order, tiles, meta, max_tiles, rows

        # the two products may take tiles of different heights (their K differ): a plan each where they do
        rows_up, rows_down = (int(self.lib.ra_moe_tile_rows(n_pairs, E, K, code)) for K in (H, I))
        up = plan(rows_up)
        down = up if rows_down == rows_up else plan(rows_down)
        order, tiles, meta, max_tiles, rows = up
        self._check(self.lib.ra_moe_product_act(_ptr(x), _ptr(w_gate_up), _ptr(mid), _ptr(order), _ptr(tiles), _ptr(meta),
                                                max_tiles, rows, I, H, top, 1, act, float(limit), float(slope),
                                                _ptr(weights) if weigh == "input" else None, code,
                                                self._stream()), "moe_product (gate-up)")
        order, tiles, meta, max_tiles, rows = down
        self._check(self.lib.ra_moe_product(_ptr(mid), _ptr(w_down), _ptr(y), _ptr(order), _ptr(tiles), _ptr(meta),
                                            max_tiles, rows, H, I, 1, 0, code, self._stream()), "moe_product (down)")
        sums = RowSums(y, top, weights if weigh == "output" else None, extra, extra_logits)
        return self.row_sums(sums) if combine else sums

    def row_sums(self, sums):
        """The rows [T, H] of RowSums (32-bit sums in their order, rounded to the rows' type)."""
        y, top, extra = sums.rows, sums.count, sums.extra
        T, H, code = y.shape[0] // top, y.shape[1], _code(y.dtype)
        out = torch.empty(T, H, dtype=y.dtype, device=self.device)
        logits_code = _code(sums.logits.dtype) if extra is not None else code
        ld_logits = self._want_rows(sums.logits, "gate logits of the further term") if extra is not None else 0
        self._check(self.lib.ra_moe_combine_extra(_ptr(y), _ptr(sums.weights), _ptr(out), T, top, H, _ptr(extra),
                                                  _ptr(sums.logits), logits_code, ld_logits, code, self._stream()), "moe_combine")
        return out

    # ------------------------------------------------------------------ measurement
    def stream_read(self, t, workgroups=0):
        """Reads every byte of tensor t once with a plain read-only kernel (one workgroup per CU unless
        given); returns the words it folded them into. For measuring the machine's read rate."""
        self._want(t, "tensor to read")
        n = t.numel() * t.element_size()
        if n == 0 or n % 16 or t.data_ptr() % 16:
            raise KernelError(f"stream_read: {n} bytes at {t.data_ptr():#x} are no whole 16-byte pieces")
        g = int(workgroups) or self.cu_count
        out = torch.empty(g, dtype=torch.int32, device=self.device)
        self._check(self.lib.ra_stream_read(_ptr(t), n, _ptr(out), g, self._stream()), "stream_read")
        return out

    # ------------------------------------------------------------------ sampling
    def sample(self, logits, temperature, top_k, top_p, u, path=None):
        """Tokens and their raw log-probabilities: int32 [m, 2] (token, float bits of logprob).
        path (int32 [m], optional) is told how each row's thresholds were found: 0 none were needed,
        1 from the list of the row's largest logits, 2 by passes over the whole row."""
        self._want(logits, "logits", torch.float32, 2)
        M, V = logits.shape
        for t, name, dt in ((temperature, "temperature", torch.float32), (top_k, "top_k", torch.int32),
                            (top_p, "top_p", torch.float32), (u, "uniforms", torch.float32)):
            self._want(t, name, dt, 1)
            if t.shape[0] != M:
                raise KernelError(f"sample: {name} has {t.shape[0]} entries for {M} rows")
        out = torch.empty(M, 2, dtype=torch.int32, device=self.device)
        if path is not None:
            self._want(path, "path", torch.int32, 1)
            if path.shape[0] != M:
                raise KernelError(f"sample: path has {path.shape[0]} entries for {M} rows")
        self._check(self.lib.ra_sample_traced(_ptr(logits), M, V, _ptr(temperature), _ptr(top_k), _ptr(top_p),
                                              _ptr(u), _ptr(out), _ptr(path), self._stream()), "sample")
        return out
