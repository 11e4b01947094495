"""Operator API of the TimeViper hot path, bound to the gfx950 kernels.

Each function keeps the NAME and ARGUMENT MEANING of the third-party operator
the reference calls (SURVEY.md §8b "inner boundary"), so `NemotronHMamba2Mixer`
and friends read like the reference's:

    causal_conv1d_fn / causal_conv1d_update      modeling_nano.py:619-624 / :495-501
    mamba_chunk_scan_combined                    modeling_nano.py:639-653
    selective_state_update                       modeling_nano.py:528-539
    rmsnorm_fn                                   modeling_nano.py:372-380
    flash_attn_func / _flash_attention_forward   modeling_nano.py:1198-1209
    flash_attn_varlen_qkvpacked_func             flash_attention_class.py:59-66
    scaled_dot_product_attention                 cross_attention.py:310-317

torch is plumbing only (device memory, current stream).  There is no CPU or
eager fallback: tensors must live on the GPU and the HIP library must be built.
"""
from __future__ import annotations

import math
import os
from typing import Optional

import torch

from . import _capi
from ._capi import TV_BF16, TV_F16, TV_F32, TimeViperHipError, check

_DT = {torch.float32: TV_F32, torch.bfloat16: TV_BF16, torch.float16: TV_F16}


def _dt(t: torch.Tensor) -> int:
    try:
        return _DT[t.dtype]
    except KeyError:
        raise TimeViperHipError(f"unsupported dtype {t.dtype}") from None


def _gpu(*ts: Optional[torch.Tensor]) -> None:
    cur = None
    for t in ts:
        if t is None:
            continue
        if not t.is_cuda:
            raise TimeViperHipError(
                "timeviper_amd kernels run on the GPU only (got a CPU tensor); "
                "there is no CPU fallback in the product path"
            )
        # the launch goes to the CURRENT device's stream (`_stream`): a tensor of another device
        # would hand that stream foreign pointers.  One process drives one GPU here.
        if cur is None:
            cur = torch.cuda.current_device()
        if t.device.index != cur:
            raise TimeViperHipError(
                f"tensor on cuda:{t.device.index} but the current device is cuda:{cur}: "
                "call torch.cuda.set_device() (one process per GPU)")


def _stream() -> int:
    return torch.cuda.current_stream().cuda_stream


def _p(t: Optional[torch.Tensor]) -> Optional[int]:
    return None if t is None else t.data_ptr()


def _rows2d(t: torch.Tensor) -> torch.Tensor:
    """View (..., D) as (rows, D) with one row stride, copying only if needed."""
    if t.stride(-1) != 1:
        t = t.contiguous()
    if t.dim() == 2:
        return t
    try:
        return t.view(-1, t.shape[-1])
    except RuntimeError:
        return t.reshape(-1, t.shape[-1])


# --------------------------------------------------------------------- conv1d
def causal_conv1d_fn(x, weight, bias=None, seq_idx=None, initial_states=None,
                     return_final_states=False, final_states_out=None, activation=None,
                     halo=None):
    """x: (B, C, L) — the reference passes the transposed view of a (B, L, C)
    tensor, which is exactly the channels-last layout the kernel wants.
    weight (C, K), bias (C).  Returns (B, C, L) (again a transposed view).
    `halo` (B, K-1, C): rows preceding this shard (sequence sharding)."""
    if seq_idx is not None or initial_states is not None or return_final_states:
        raise TimeViperHipError("causal_conv1d_fn: seq_idx/initial_states/final_states unsupported")
    if activation not in (None, "silu", "swish"):
        raise TimeViperHipError(f"causal_conv1d_fn: activation {activation!r}")
    _gpu(x, weight, bias, halo)
    B, Cc, L = x.shape
    xl = x.transpose(1, 2)  # (B, L, C)
    if xl.stride(2) != 1:
        xl = xl.contiguous()
    K = weight.shape[-1]
    w = weight.reshape(Cc, K).to(x.dtype).contiguous()
    b = None if bias is None else bias.to(x.dtype).contiguous()
    if halo is not None:
        halo = halo.to(x.dtype).contiguous()
        assert halo.shape == (B, K - 1, Cc)
    y = torch.empty((B, L, Cc), dtype=x.dtype, device=x.device)
    check(_capi.lib().tv_causal_conv1d_fwd(
        _p(xl), _p(w), _p(b), _p(halo), _p(y), B, L, Cc, K, xl.stride(0), xl.stride(1),
        y.stride(0), y.stride(1), _dt(x), int(activation in ("silu", "swish")), _stream()),
        "tv_causal_conv1d_fwd")
    return y.transpose(1, 2)


def causal_conv1d_xbc(xBC, weight, bias, d_inner: int, ngroups: int, dstate: int,
                      activation="silu", halo=None, return_cb: bool = False):
    """Mamba-2 mixer variant of causal_conv1d_fn + the [x | B | C] split of
    modeling_nano.py:628-636 in one pass.  xBC (B, L, d_inner + 2*G*N) (any row stride).
    Returns x (B, L, d_inner) and B, C as (B, L, G, N) VIEWS of group-major (B, G, L, N)
    storage — the layout the scan kernel streams best.
    `return_cb`: also return the causal C.B^T fragments of every (chunk, group) for
    `mamba_chunk_scan_combined(..., cb=...)` (an opaque bf16 tensor; None where the scan would
    not use them: other dtypes / d_state), computed while the B / C tiles are on the chip."""
    _gpu(xBC, weight, bias, halo)
    Bsz, L, Cc = xBC.shape
    assert Cc == d_inner + 2 * ngroups * dstate
    if xBC.stride(2) != 1:
        xBC = xBC.contiguous()
    K = weight.shape[-1]
    w = weight.reshape(Cc, K).to(xBC.dtype).contiguous()
    b = None if bias is None else bias.to(xBC.dtype).contiguous()
    if halo is not None:
        halo = halo.to(xBC.dtype).contiguous()
    yx = torch.empty((Bsz, L, d_inner), dtype=xBC.dtype, device=xBC.device)
    yb = torch.empty((Bsz, ngroups, L, dstate), dtype=xBC.dtype, device=xBC.device)
    yc = torch.empty((Bsz, ngroups, L, dstate), dtype=xBC.dtype, device=xBC.device)
    lib = _capi.lib()
    if return_cb and xBC.dtype == torch.bfloat16 and dstate == 128 and L > 0:
        cb = torch.empty(lib.tv_ssd_cb_bytes(Bsz, L, ngroups) // 2, dtype=torch.bfloat16, device=xBC.device)
        check(lib.tv_causal_conv1d_xbc_cb_fwd(
            _p(xBC), _p(w), _p(b), _p(halo), _p(yx), _p(yb), _p(yc), _p(cb), Bsz, L, d_inner, ngroups, dstate,
            K, xBC.stride(0), xBC.stride(1), _dt(xBC), int(activation in ("silu", "swish")), _stream()),
            "tv_causal_conv1d_xbc_cb_fwd")
        return yx, yb.transpose(1, 2), yc.transpose(1, 2), cb
    check(lib.tv_causal_conv1d_xbc_fwd(
        _p(xBC), _p(w), _p(b), _p(halo), _p(yx), _p(yb), _p(yc), Bsz, L, d_inner, ngroups, dstate,
        K, xBC.stride(0), xBC.stride(1), _dt(xBC), int(activation in ("silu", "swish")), _stream()),
        "tv_causal_conv1d_xbc_fwd")
    if return_cb:
        return yx, yb.transpose(1, 2), yc.transpose(1, 2), None
    return yx, yb.transpose(1, 2), yc.transpose(1, 2)


def causal_conv1d_update(x, conv_state, weight, bias=None, activation=None):
    """x (B, C); conv_state (B, C, K) updated in place; returns (B, C)."""
    _gpu(x, conv_state, weight, bias)
    B, Cc = x.shape
    K = weight.shape[-1]
    if not conv_state.is_contiguous() or conv_state.dtype != x.dtype:
        raise TimeViperHipError("causal_conv1d_update: conv_state must be contiguous, x.dtype")
    xc = x.contiguous()
    w = weight.reshape(Cc, K).to(x.dtype).contiguous()
    b = None if bias is None else bias.to(x.dtype).contiguous()
    y = torch.empty_like(xc)
    check(_capi.lib().tv_causal_conv1d_update(
        _p(xc), _p(conv_state), _p(w), _p(b), _p(y), B, Cc, K, _dt(x),
        int(activation in ("silu", "swish")), _stream()), "tv_causal_conv1d_update")
    return y


# ---------------------------------------------------------------------- norms
def rms_norm(x, weight, eps, residual=None, return_sum=False):
    """NemotronHRMSNorm (modeling_nano.py:897-903); with `residual`, normalises
    s = x + residual (rounded to x.dtype like the reference's bf16 add, :966) and
    can return s too."""
    _gpu(x, weight, residual)
    x2 = _rows2d(x)
    r2 = None if residual is None else _rows2d(residual)
    y = torch.empty(x2.shape, dtype=x.dtype, device=x.device)
    s = torch.empty_like(y) if (return_sum and residual is not None) else None
    w = weight if weight.dtype in (torch.float32, x.dtype) else weight.to(torch.float32)
    w = w.contiguous()
    check(_capi.lib().tv_rmsnorm_fwd(
        _p(x2), _p(r2), _p(w), _p(s), _p(y), x2.shape[0], x2.shape[1], x2.stride(0),
        0 if r2 is None else r2.stride(0), 0 if s is None else s.stride(0), y.stride(0),
        float(eps), _dt(x), _dt(w), _stream()), "tv_rmsnorm_fwd")
    y = y.view(x.shape)
    if return_sum:
        return y, (s.view(x.shape) if s is not None else x)
    return y


def layer_norm(x, weight, bias, eps, residual=None, return_sum=False, row_bias=None):
    """nn.LayerNorm over the last dim, optionally of s = x + residual (rounded to x.dtype),
    returning s too — the fused form of a pre-norm ViT block's residual add + norm.
    `row_bias` (D,) fp32: a constant row added to every s before the statistics (not to the
    returned sum): the projection biases a caller carries beside a stream its GEMMs accumulate into."""
    _gpu(x, weight, bias, residual, row_bias)
    x2 = _rows2d(x)
    r2 = None if residual is None else _rows2d(residual)
    y = torch.empty(x2.shape, dtype=x.dtype, device=x.device)
    s = torch.empty_like(y) if (return_sum and residual is not None) else None
    w = weight.to(x.dtype).contiguous()
    b = None if bias is None else bias.to(x.dtype).contiguous()
    rb = None if row_bias is None else row_bias.to(torch.float32).contiguous()
    check(_capi.lib().tv_layernorm_fwd(
        _p(x2), _p(r2), _p(w), _p(b), _p(rb), _p(s), _p(y), x2.shape[0], x2.shape[1], x2.stride(0),
        0 if r2 is None else r2.stride(0), 0 if s is None else s.stride(0), y.stride(0), float(eps),
        _dt(x), _stream()), "tv_layernorm_fwd")
    y = y.view(x.shape)
    if return_sum:
        return y, (s.view(x.shape) if s is not None else x)
    return y


def gelu(x, inplace=False):
    """exact (erf) GELU, elementwise."""
    _gpu(x)
    xc = x if x.is_contiguous() else x.contiguous()
    y = xc if inplace else torch.empty_like(xc)
    check(_capi.lib().tv_gelu_fwd(_p(xc), _p(y), xc.numel(), _dt(xc), _stream()), "tv_gelu_fwd")
    return y


def relu2(x, inplace=False):
    """square(relu(x)) — NemotronHMLP's activation (modeling_nano.py:993-994), elementwise."""
    _gpu(x)
    xc = x if x.is_contiguous() else x.contiguous()
    y = xc if inplace else torch.empty_like(xc)
    check(_capi.lib().tv_relu2_fwd(_p(xc), _p(y), xc.numel(), _dt(xc), _stream()), "tv_relu2_fwd")
    return y


def rmsnorm_fn(x, weight, bias=None, z=None, eps=1e-6, group_size=None,
               norm_before_gate=True, upcast=True):
    """mamba_ssm.ops.triton.layernorm_gated.rmsnorm_fn as the reference calls it
    (norm_before_gate=False): y = w * u * rsqrt(mean_group(u^2)+eps), u = x*silu(z)."""
    if bias is not None:
        raise TimeViperHipError("rmsnorm_fn: bias unsupported (reference passes None)")
    if z is not None and norm_before_gate:
        raise TimeViperHipError("rmsnorm_fn: only norm_before_gate=False is on the path")
    _gpu(x, weight, z)
    x2 = _rows2d(x)
    z2 = None if z is None else _rows2d(z)
    D = x2.shape[1]
    gs = D if group_size is None else int(group_size)
    y = torch.empty(x2.shape, dtype=x.dtype, device=x.device)
    w = weight if weight.dtype in (torch.float32, x.dtype) else weight.to(torch.float32)
    w = w.contiguous()
    check(_capi.lib().tv_rmsnorm_gated_fwd(
        _p(x2), _p(z2), _p(w), _p(y), x2.shape[0], D, gs, x2.stride(0),
        0 if z2 is None else z2.stride(0), y.stride(0), float(eps), _dt(x), _dt(w), _stream()),
        "tv_rmsnorm_gated_fwd")
    return y.view(x.shape)


# ------------------------------------------------------------------- linears with fused epilogues
GEMM_BIAS, GEMM_BIAS_GELU, GEMM_ACCUM = 0, 1, 2


def linear_fused(x, weight, bias=None, epilogue: int = GEMM_BIAS, out=None):
    """F.linear(x, weight, bias) on the hand-written bf16 GEMM (csrc/gemm.hip) with the epilogue fused:
    GEMM_BIAS (plain), GEMM_BIAS_GELU (exact GELU of the bf16-rounded result: the timm Mlp's fc1 + act) or
    GEMM_ACCUM (out += x @ weight.T, `out` required, bias ignored).  x (..., K) bf16 with dense rows,
    weight (N, K) bf16; K % 128 == 0, N % 4 == 0."""
    _gpu(x, weight, bias, out)
    if x.dtype != torch.bfloat16 or weight.dtype != torch.bfloat16:
        raise TimeViperHipError("linear_fused: bf16 only")
    x2 = _rows2d(x)
    N, Kd = weight.shape
    if weight.stride(1) != 1:
        weight = weight.contiguous()
    if epilogue == GEMM_ACCUM:
        if out is None:
            raise TimeViperHipError("linear_fused: GEMM_ACCUM needs `out`")
        bias = None
    if out is None:
        out = torch.empty(x.shape[:-1] + (N,), dtype=x.dtype, device=x.device)
    o2 = out.view(-1, N) if out.dim() != 2 else out
    if o2.stride(1) != 1 or o2.shape[0] != x2.shape[0]:
        raise TimeViperHipError("linear_fused: `out` must be (rows, N) with a contiguous last dim")
    bd = TV_F32
    if bias is not None:
        if bias.dtype not in (torch.float32, torch.bfloat16):
            bias = bias.float()
        bias = bias.contiguous()
        bd = _dt(bias)
    check(_capi.lib().tv_gemm_bf16_fwd(_p(x2), _p(weight), _p(bias), _p(o2), x2.shape[0], N, Kd, x2.stride(0),
                                       weight.stride(0), o2.stride(0), int(epilogue), bd, _stream()),
          "tv_gemm_bf16_fwd")
    return out


def param_key(params):
    """Cache key for tensors derived from parameters (stacked / padded / fp32 copies): storage, version counter, dtype
    and device of each.  Tensors created under `torch.inference_mode()` track no version ("Inference tensors do not
    track version counter"): they count as version 0 — such a model must not be written in place after its first forward.
    Note that writes through `.data` never bump the counter either: reload weights with `load_state_dict` / `copy_`."""
    key = []
    for p in params:
        try:
            v = p._version
        except RuntimeError:
            v = 0
        key.append((p.data_ptr(), v, p.dtype, p.device))
    return tuple(key)


def gemm_set_persist(mode: int = -1, grid: int = 0) -> None:
    """Which of the two GEMM kernels `linear_fused` runs on: -1 automatic (the persistent kernel from 4 tiles per
    compute unit on), 0 the per-tile kernel only, 1 the persistent kernel wherever the shape allows; `grid`:
    work-groups of the persistent kernel (0 = one per compute unit; tests use 8 so that small problems still give
    every work-group several tiles)."""
    _capi.lib().tv_gemm_set_persist(int(mode), int(grid))


# zero-padded inference copies of weights (model/vit/siglip.py): storage address -> (useful rows, useful columns), so that a
# FLOP count (bench.py) can leave the padding out whatever view of the copy a GEMM receives
PADDED_USEFUL: dict = {}


def gemm_set_drip(mode: int = -1) -> None:
    """The 256 x 192-tile persistent GEMM (csrc/gemm_drip.hip): -1 automatic (first choice wherever the shape allows and
    every compute unit gets a few tiles), 0 never, 1 wherever the shape allows (tests on small grids)."""
    _capi.lib().tv_gemm_set_drip(int(mode))


# ------------------------------------------------------------------- SSD scan
def _row_view(t: torch.Tensor, inner: int):
    """(B, L, ...) tensor whose trailing dims are contiguous with `inner`
    elements per row: return (tensor, stride_b, stride_l) without copying when
    the rows are dense (slices of a wider projection keep their row stride)."""
    ok = t.stride(-1) == 1
    exp = 1
    for d in range(t.dim() - 1, 1, -1):
        ok = ok and t.stride(d) == exp
        exp *= t.shape[d]
    if not ok:
        t = t.contiguous()
    return t, t.stride(0), t.stride(1)


def mamba_chunk_scan_combined(x, dt, A, B, C, chunk_size=None, D=None, z=None, dt_bias=None,
                              initial_states=None, seq_idx=None, cu_seqlens=None,
                              dt_softplus=False, dt_limit=(0.0, float("inf")),
                              return_final_states=False, return_varlen_states=False,
                              group_map="block", return_total_decay=False, cb=None):
    """x (B,L,H,P), dt (B,L,H), A (H), B/C (B,L,G,N), D (H), dt_bias (H),
    initial_states (B,H,P,N).  Returns y (B,L,H,P) [, final_states (B,H,P,N) fp32]
    [, total_decay (B,H) fp32].  `chunk_size` is accepted for signature parity
    and ignored (the result is chunk-invariant).  `group_map`: "block"
    (h // (H/G), GPU reference) or "tile" (h % G, reference CPU quirk).
    `cb`: the C.B^T fragments `causal_conv1d_xbc(..., return_cb=True)` returned for these B / C."""
    if z is not None or seq_idx is not None or cu_seqlens is not None or return_varlen_states:
        raise TimeViperHipError("mamba_chunk_scan_combined: z/seq_idx/cu_seqlens unsupported")
    if D is not None and D.dim() != 1:
        raise TimeViperHipError("mamba_chunk_scan_combined: D must be (nheads,)")
    _gpu(x, dt, A, B, C, D, dt_bias, initial_states)
    Bsz, L, H, P = x.shape
    G, N = B.shape[2], B.shape[3]
    if dt.dtype != x.dtype:
        dt = dt.to(x.dtype)
    if B.dtype != x.dtype:
        B = B.to(x.dtype)
    if C.dtype != x.dtype:
        C = C.to(x.dtype)
    x, xsb, xsl = _row_view(x, H * P)
    dt, dsb, dsl = _row_view(dt, H)
    # B/C: any (B, L, G, N) view with contiguous N (token-major rows or group-major storage)
    if B.stride(3) != 1:
        B = B.contiguous()
    if C.stride(3) != 1:
        C = C.contiguous()
    bsb, bsl, bsg = B.stride(0), B.stride(1), B.stride(2)
    csb, csl, csg = C.stride(0), C.stride(1), C.stride(2)
    f32 = lambda t: None if t is None else t.to(torch.float32).contiguous()
    A, D, dt_bias, initial_states = f32(A), f32(D), f32(dt_bias), f32(initial_states)
    y = torch.empty((Bsz, L, H, P), dtype=x.dtype, device=x.device)
    final = torch.empty((Bsz, H, P, N), dtype=torch.float32, device=x.device) \
        if return_final_states else None
    decay = torch.empty((Bsz, H), dtype=torch.float32, device=x.device) \
        if return_total_decay else None
    lib = _capi.lib()
    ws_bytes = lib.tv_ssd_scan_workspace_bytes(Bsz, L, H, P, G, N, _dt(x))
    ws = torch.empty(max(ws_bytes, 16), dtype=torch.uint8, device=x.device)
    if cb is not None:
        _gpu(cb)
        if cb.dtype != torch.bfloat16 or cb.numel() * 2 != lib.tv_ssd_cb_bytes(Bsz, L, G) or not cb.is_contiguous():
            raise TimeViperHipError("mamba_chunk_scan_combined: cb is not the C.B^T buffer of these shapes")
    check(lib.tv_ssd_scan_cb_fwd(
        _p(x), _p(dt), _p(A), _p(B), _p(C), _p(cb), _p(D), _p(dt_bias), _p(initial_states), _p(y),
        _p(final), _p(decay), Bsz, L, H, P, G, N, xsb, xsl, dsb, dsl, bsb, bsl, bsg, csb, csl, csg,
        y.stride(0), y.stride(1), _dt(x), int(bool(dt_softplus)), float(dt_limit[0]),
        float(min(dt_limit[1], 3.0e38)), {"block": 0, "tile": 1}[group_map], _p(ws), ws_bytes,
        _stream()), "tv_ssd_scan_cb_fwd")
    out = (y,)
    if return_final_states:
        out += (final,)
    if return_total_decay:
        out += (decay,)
    return out[0] if len(out) == 1 else out


def ssd_state_correction(y, dt, A, C, state_in, dt_bias=None, dt_softplus=False,
                         dt_limit=(0.0, float("inf")), group_map="block"):
    """In place: y_t += exp(sum_{j<=t} dt_j A_h) C_t . state_in[h] — completes the outputs of a scan
    that started from a zero state once the state entering it is known (sequence shards, SURVEY
    Appendix A).  y (B,L,H,P), dt (B,L,H) raw, C (B,L,G,N), state_in (B,H,P,N) fp32.  Returns y."""
    _gpu(y, dt, A, C, state_in, dt_bias)
    Bsz, L, H, P = y.shape
    G, N = C.shape[2], C.shape[3]
    assert y.stride(3) == 1 and y.stride(2) == P, "y rows must be dense (H*P elements)"
    if dt.dtype != y.dtype:
        dt = dt.to(y.dtype)
    dt, dsb, dsl = _row_view(dt, H)
    if C.dtype != y.dtype:
        C = C.to(y.dtype)
    if C.stride(3) != 1:
        C = C.contiguous()
    f32 = lambda t: None if t is None else t.to(torch.float32).contiguous()
    A, dt_bias, state_in = f32(A), f32(dt_bias), f32(state_in)
    lib = _capi.lib()
    ws_bytes = lib.tv_ssd_state_correction_workspace_bytes(Bsz, L, H)
    ws = torch.empty(max(ws_bytes, 16), dtype=torch.uint8, device=y.device)
    check(lib.tv_ssd_state_correction(
        _p(y), _p(dt), _p(A), _p(C), _p(dt_bias), _p(state_in), Bsz, L, H, P, G, N,
        y.stride(0), y.stride(1), dsb, dsl, C.stride(0), C.stride(1), C.stride(2), _dt(y),
        int(bool(dt_softplus)), float(dt_limit[0]), float(min(dt_limit[1], 3.0e38)),
        {"block": 0, "tile": 1}[group_map], _p(ws), ws_bytes, _stream()), "tv_ssd_state_correction")
    return y


def selective_state_update(state, x, dt, A, B, C, D=None, z=None, dt_bias=None,
                           dt_softplus=False):
    """Single decode step.  state (B,H,P,N) fp32, in place.  The reference passes
    A/dt/dt_bias/D expanded over (P[,N]) from per-head values (:514-522); the
    kernel takes the per-head values, so expanded views are reduced here."""
    if z is not None:
        raise TimeViperHipError("selective_state_update: z unsupported (reference passes None)")
    _gpu(state, x, dt, A, B, C, D, dt_bias)
    Bsz, H, P = x.shape
    G, N = B.shape[1], B.shape[2]
    if state.dtype != torch.float32 or not state.is_contiguous():
        raise TimeViperHipError("selective_state_update: state must be contiguous fp32")
    head = lambda t, nd: None if t is None else \
        (t if t.dim() == nd else t[(..., *([0] * (t.dim() - nd)))]).to(torch.float32).contiguous()
    A1, D1, b1 = head(A, 1), head(D, 1), head(dt_bias, 1)
    dt1 = (dt if dt.dim() == 2 else dt[..., 0]).to(x.dtype).contiguous()
    xc, Bc, Cc = x.contiguous(), B.to(x.dtype).contiguous(), C.to(x.dtype).contiguous()
    y = torch.empty_like(xc)
    check(_capi.lib().tv_selective_state_update(
        _p(state), _p(xc), _p(dt1), _p(A1), _p(Bc), _p(Cc), _p(D1), _p(b1), _p(y), Bsz, H, P, G,
        N, _dt(x), int(bool(dt_softplus)), _stream()), "tv_selective_state_update")
    return y


def ssd_scan_set_impl(impl: int) -> None:
    """0 auto (= 6 where it applies, else 4, 3; other dtypes / d_state: 8, else 1), 1 generic fp32 token recurrence, 3 MFMA
    slice march on <= 40-column slices of a head, 4 whole-head slice march x sequence segments, 6 head-per-wave march
    (ssd_head.hip), 8 chunk-parallel fp32 form (ssd_chunked.hip); 2 / 5 / 7 (removed kernels) select 3 / 4 / 6.
    Process-global (dev tools and tests)."""
    _capi.lib().tv_ssd_scan_set_impl(int(impl))


def ssd_head_set_asm(on: int) -> None:
    """Head-per-wave march at head_dim 80 x 4 heads per work-group: 1 the generated step (default), 0 the C++ step, -1 default /
    TV_HEAD_ASM.  Process-global (A/B runs and the bit-identity test)."""
    _capi.lib().tv_ssd_head_set_asm(int(on))


def ssd_scan_last_impl() -> int:
    """Kernel family (the numbers of `ssd_scan_set_impl`) the most recent scan call of this process ran on."""
    return int(_capi.lib().tv_ssd_scan_last_impl())


# ------------------------------------------------------------------ attention
def flash_attn_set_variant(variant: int) -> None:
    """0 auto (bf16 ViT frames: the kernel with the generated tile loop, csrc/attention_vit.hpp; else the compiled streaming
    kernel), 5 always the compiled streaming kernel (P's row sums out of the P.V MFMAs), 3 the compiled kernel with the row
    sums on the vector pipe (A/B, tests); include/timeviper_hip.h.  Process-global (dev tools and tests)."""
    _capi.lib().tv_flash_attn_set_variant(int(variant))


_ATTN_FP8 = {"on": False, "min_keys": 4096, "min_queries": 64}


class fp8_attention:
    """Context manager / switch: inside it `flash_attn_func` (and everything built on it) runs the
    QK^T / PV products on the FP8 MFMA path (`tv_flash_attn_fp8_fwd`) — BASELINE config 5.  Off by
    default: the reference's attention arithmetic is bf16.  Key sequences shorter than `min_keys`
    stay on the bf16 kernel: the ViT towers (<= 1 025 keys per frame / tube; measured 2.3 ms fp8
    against 1.5 ms bf16 per 256 SigLIP frames — the quantisation pre-pass and head_dim 72 -> 128
    padding cost more than the MFMAs save); calls with fewer than `min_queries` queries stay there too: the
    decode step (one query against the whole cache: the quantisation pre-pass over the cache would cost
    more than the attention, with per-head scales that differ from the prefill's).  The long causal LM
    attention is where the fp8 matrix rate pays (131 172 tokens, 28/4 x 128: 83 ms against 122 ms).
    The switch is process-global state (like `ssd_scan_set_impl`): right for an evaluation process, not for
    two models with different settings in one process."""

    def __init__(self, on: bool = True, min_keys: int = 4096, min_queries: int = 64):
        self.new = {"on": bool(on), "min_keys": int(min_keys), "min_queries": int(min_queries)}

    def __enter__(self):
        self.old = dict(_ATTN_FP8)
        _ATTN_FP8.update(self.new)
        return self

    def __exit__(self, *exc):
        _ATTN_FP8.update(self.old)


def flash_attn_fp8_func(q, k, v, softmax_scale=None, causal=False, return_lse=False):
    """`flash_attn_func` with e4m3 MFMA operands (per-head scales, fp32 accumulation / softmax)."""
    _gpu(q, k, v)
    B, Lq, Hq, D = q.shape
    Lk, Hkv = k.shape[1], k.shape[2]
    fix = lambda t: t if t.stride(-1) == 1 else t.contiguous()
    q, k, v = fix(q), fix(k), fix(v)
    if D % 8 or D > 128:
        raise TimeViperHipError(f"flash_attn_fp8_func: head_dim {D} must be a multiple of 8, <= 128")
    for t in (q, k, v):
        if any(s % 8 for s in t.stride()[:3]) or t.data_ptr() % 16:
            raise TimeViperHipError("flash_attn_fp8_func: strides must be multiples of 8 elements")
    scale = 1.0 / math.sqrt(D) if softmax_scale is None else float(softmax_scale)
    o = torch.empty((B, Lq, Hq, D), dtype=q.dtype, device=q.device)
    lse = torch.empty((B, Hq, Lq), dtype=torch.float32, device=q.device) if return_lse else None
    lib = _capi.lib()
    ws_bytes = lib.tv_flash_attn_fp8_workspace_bytes(B, Lq, Lk, Hq, Hkv)
    ws = torch.empty(max(ws_bytes, 256), dtype=torch.uint8, device=q.device)
    check(lib.tv_flash_attn_fp8_fwd(
        _p(q), _p(k), _p(v), _p(o), _p(lse), B, Lq, Lk, Hq, Hkv, D,
        q.stride(0), q.stride(1), q.stride(2), k.stride(0), k.stride(1), k.stride(2),
        v.stride(0), v.stride(1), v.stride(2), o.stride(0), o.stride(1), o.stride(2),
        scale, int(bool(causal)), _dt(q), _p(ws), ws_bytes, _stream()), "tv_flash_attn_fp8_fwd")
    return (o, lse) if return_lse else o


def flash_attn_func(q, k, v, dropout_p=0.0, softmax_scale=None, causal=False,
                    return_lse=False):
    """q (B,Lq,Hq,D), k/v (B,Lk,Hkv,D) -> (B,Lq,Hq,D).  GQA without repeat_kv;
    causal mask bottom-right aligned (flash-attn >= 2.1 semantics)."""
    if dropout_p:
        raise TimeViperHipError("flash_attn_func: dropout is not on the inference path")
    _gpu(q, k, v)
    B, Lq, Hq, D = q.shape
    Lk, Hkv = k.shape[1], k.shape[2]
    # (Lq >= 64: a decode step against a long cache stays on the bf16 kernel — the fp8 path would re-quantise and
    # transpose the whole K / V cache for one query, with a scale that differs from the prefill's)
    if _ATTN_FP8["on"] and Lk >= _ATTN_FP8["min_keys"] and Lq >= _ATTN_FP8["min_queries"] and D <= 128 \
            and q.dtype in (torch.bfloat16, torch.float16):
        return flash_attn_fp8_func(q, k, v, softmax_scale, causal, return_lse)
    fix = lambda t: t if t.stride(-1) == 1 else t.contiguous()
    q, k, v = fix(q), fix(k), fix(v)
    if Lq == 1 and _decode_attn_takes(q, k, v):         # a decode step: split-KV kernel (causal or not: one query, last row)
        return flash_attn_decode(q, k, v, softmax_scale=softmax_scale, return_lse=return_lse)
    if D % 8:
        raise TimeViperHipError(f"flash_attn_func: head_dim {D} must be a multiple of 8")
    for t in (q, k, v):
        if any(s % 8 for s in t.stride()[:3]) or t.data_ptr() % 16:
            raise TimeViperHipError("flash_attn_func: strides must be multiples of 8 elements")
    scale = 1.0 / math.sqrt(D) if softmax_scale is None else float(softmax_scale)
    o = torch.empty((B, Lq, Hq, D), dtype=q.dtype, device=q.device)
    lse = torch.empty((B, Hq, Lq), dtype=torch.float32, device=q.device) if return_lse else None
    check(_capi.lib().tv_flash_attn_fwd(
        _p(q), _p(k), _p(v), _p(o), _p(lse), B, Lq, Lk, Hq, Hkv, D,
        q.stride(0), q.stride(1), q.stride(2), k.stride(0), k.stride(1), k.stride(2),
        v.stride(0), v.stride(1), v.stride(2), o.stride(0), o.stride(1), o.stride(2),
        scale, int(bool(causal)), _dt(q), _stream()), "tv_flash_attn_fwd")
    return (o, lse) if return_lse else o


GEMV_NONE, GEMV_RMSNORM, GEMV_RELU2, GEMV_GATED = 0, 1, 2, 3


def gemv_takes(x: torch.Tensor, weight: torch.Tensor) -> bool:
    """Shapes tv_gemv_bf16_fwd is written for: 1..4 rows of bf16 against a bf16 (N, K) weight, f(x) within 128 KiB of LDS."""
    K = x.shape[-1]
    rows = x.numel() // max(K, 1)
    return (x.is_cuda and x.dtype == torch.bfloat16 and weight.dtype == torch.bfloat16 and weight.dim() == 2
            and 1 <= rows <= 4 and K % 8 == 0 and rows * K * 2 <= 128 * 1024 and weight.stride(1) == 1
            and weight.stride(0) % 8 == 0)


def gemv_fused(x, weight, bias=None, prologue=GEMV_NONE, delta=None, sum_out=None, norm_weight=None, eps=0.0,
               gate=None, group_size=0, conv=None):
    """y = f(x) @ weight.T (+ bias) for 1..4 rows — the linear layers of a decode step (torch.nn.Linear at q_len 1) with
    the single-row operator in front of them computed in the kernel's prologue: GEMV_RMSNORM (NemotronHRMSNorm with the
    block's residual add: `delta` is added to x first, the sum goes to `sum_out`), GEMV_RELU2 (the MLP activation),
    GEMV_GATED (MambaRMSNormGated with `gate`), rounding where the stand-alone operators round.
    `conv=(conv_state, weight, bias, row0)`: the outputs [row0, row0 + C) go through `causal_conv1d_update` (width 4,
    SiLU) on conv_state (B, C, 4) before they are stored — the mixer's in_proj -> conv pair as one launch (K < 8192)."""
    _gpu(x, weight, bias, delta, sum_out, norm_weight, gate)
    K = x.shape[-1]
    x2 = _rows2d(x)
    M, N = x2.shape[0], weight.shape[0]
    if weight.shape[1] != K:
        raise TimeViperHipError(f"gemv_fused: weight {tuple(weight.shape)} against rows of {K}")
    # the C ABI carries no weight dtype: anything but dense bf16 rows would be re-interpreted silently
    if (x.dtype != torch.bfloat16 or weight.dtype != torch.bfloat16 or weight.stride(1) != 1 or weight.stride(0) % 8
            or K % 8):
        raise TimeViperHipError("gemv_fused: bf16 x and weight with dense rows of a multiple of 8 elements only "
                                f"(x {x.dtype}, weight {weight.dtype}, strides {tuple(weight.stride())}, K {K})")
    y = torch.empty(x.shape[:-1] + (N,), dtype=x.dtype, device=x.device)
    d2 = None if delta is None else _rows2d(delta)
    g2 = None if gate is None else _rows2d(gate)
    s2 = None if sum_out is None else sum_out.view(-1, K)
    for t in (d2, g2, s2):
        if t is not None and (t.shape != x2.shape or t.dtype != x.dtype):
            raise TimeViperHipError("gemv_fused: delta / gate / sum_out must have x's shape and dtype")
    if bias is not None and (bias.dtype != x.dtype or not bias.is_contiguous()):
        raise TimeViperHipError("gemv_fused: bias must be contiguous, of x's dtype")
    nw_dt = 0
    if norm_weight is not None:
        if not norm_weight.is_contiguous() or norm_weight.numel() != K:
            raise TimeViperHipError("gemv_fused: norm_weight must be a contiguous vector of K entries")
        nw_dt = _dt(norm_weight)
    cst = cw = cb = None
    row0 = nch = 0
    if conv is not None:
        cst, cw, cb, row0 = conv
        _gpu(cst, cw, cb)
        nch = cst.shape[1]
        if (cst.dtype != x.dtype or cw.dtype != x.dtype or not cst.is_contiguous() or not cw.is_contiguous()
                or cst.shape != (M, nch, 4) or cw.shape != (nch, 4) or (cb is not None and (cb.dtype != x.dtype or not cb.is_contiguous()))):
            raise TimeViperHipError("gemv_fused: conv needs a contiguous (rows, C, 4) state and (C, 4) weight of x's dtype")
    check(_capi.lib().tv_gemv_bf16_fwd(
        _p(x2), _p(weight), _p(bias), _p(y), M, N, K, x2.stride(0), weight.stride(0), N, int(prologue),
        _p(d2), 0 if d2 is None else d2.stride(0), _p(s2), 0 if s2 is None else s2.stride(0),
        _p(norm_weight), nw_dt, float(eps), _p(g2), 0 if g2 is None else g2.stride(0), int(group_size),
        _p(cst), _p(cw), _p(cb), int(row0), int(nch), _stream()), "tv_gemv_bf16_fwd")
    return y


def _decode_attn_takes(q, k, v) -> bool:
    """Shapes tv_attn_decode_fwd is written for (the rest stays on tv_flash_attn_fwd with one query row)."""
    return (q.dtype == torch.bfloat16 and q.shape[-1] == 128 and k.shape[1] >= 256
            and os.environ.get("TV_ATTN_DECODE", "1") != "0"
            and all(s % 8 == 0 for t in (q, k, v) for s in t.stride()[:3])
            and all(t.data_ptr() % 16 == 0 for t in (q, k, v)))


def flash_attn_decode(q, k, v, seqlens_k=None, softmax_scale=None, return_lse=False, out=None):
    """One query token per sequence against a K / V cache: q (B, 1, Hq, 128) bf16, k / v (B, Lk, Hkv, 128) ->
    (B, 1, Hq, 128) (the q_len == 1 call of modeling_nano.py:1198-1209).  `seqlens_k`: int32 tensor (B,) ON THE GPU with
    the keys in use per sequence (<= Lk, the capacity of the cache buffers) — the form a captured decode step replays
    with; None: all Lk keys."""
    _gpu(q, k, v, seqlens_k)
    B, Lq, Hq, D = q.shape
    Lk, Hkv = k.shape[1], k.shape[2]
    if Lq != 1:
        raise TimeViperHipError("flash_attn_decode: one query token per sequence")
    if seqlens_k is not None and (seqlens_k.dtype != torch.int32 or seqlens_k.numel() != B or not seqlens_k.is_contiguous()):
        raise TimeViperHipError("flash_attn_decode: seqlens_k must be a contiguous int32 tensor of `batch` entries")
    fix = lambda t: t if t.stride(-1) == 1 else t.contiguous()
    q, k, v = fix(q), fix(k), fix(v)
    scale = 1.0 / math.sqrt(D) if softmax_scale is None else float(softmax_scale)
    o = torch.empty((B, 1, Hq, D), dtype=q.dtype, device=q.device) if out is None else out
    if o.shape != (B, 1, Hq, D) or o.dtype != q.dtype or o.stride(-1) != 1:
        raise TimeViperHipError("flash_attn_decode: out must be (B, 1, Hq, D) of q's dtype with unit last stride")
    lse = torch.empty((B, Hq, 1), dtype=torch.float32, device=q.device) if return_lse else None
    lib = _capi.lib()
    ws = torch.empty((max(int(lib.tv_attn_decode_workspace_bytes(B, Hq, Hkv, Lk)), 16),), dtype=torch.uint8,
                     device=q.device)
    check(lib.tv_attn_decode_fwd(
        _p(q), _p(k), _p(v), _p(o), _p(lse), B, Lk, _p(seqlens_k), Hq, Hkv, D,
        q.stride(0), q.stride(2), k.stride(0), k.stride(1), k.stride(2),
        v.stride(0), v.stride(1), v.stride(2), o.stride(0), o.stride(2),
        scale, _dt(q), _p(ws), ws.numel() * ws.element_size(), _stream()), "tv_attn_decode_fwd")
    return (o, lse) if return_lse else o


def _flash_attention_forward(query_states, key_states, value_states, attention_mask=None,
                             query_length=None, is_causal=True, dropout=0.0, position_ids=None,
                             softmax_scale=None, sliding_window=None, use_top_left_mask=False,
                             **kwargs):
    """transformers' helper as NemotronHFlashAttention2 calls it (:1198-1209)."""
    if attention_mask is not None or sliding_window is not None:
        raise TimeViperHipError("_flash_attention_forward: padding mask / sliding window unsupported")
    causal = is_causal and not (use_top_left_mask and query_states.shape[1] == 1)
    return flash_attn_func(query_states, key_states, value_states, dropout,
                           softmax_scale=softmax_scale, causal=causal)


def scaled_dot_product_attention(query, key, value, attn_mask=None, dropout_p=0.0,
                                 is_causal=False, scale=None):
    """F.scaled_dot_product_attention layout: (B, H, L, D) in and out."""
    if attn_mask is not None:
        raise TimeViperHipError("scaled_dot_product_attention: attn_mask unsupported")
    o = flash_attn_func(query.transpose(1, 2), key.transpose(1, 2), value.transpose(1, 2),
                        dropout_p, softmax_scale=scale, causal=is_causal)
    return o.transpose(1, 2)


def flash_attn_varlen_qkvpacked_func(qkv, cu_seqlens, max_seqlen, dropout_p=0.0,
                                     softmax_scale=None, causal=False, **kwargs):
    """qkv (nnz, 3, H, D), sequences [cu_seqlens[i], cu_seqlens[i+1]) (flash_attention_class.py:59-66, :68-91).
    Equal lengths — what the InternVideo2 ViT produces: every clip has the same token count — are ONE launch over
    a (nseq, len) view; a ragged batch (the `key_padding_mask` / `unpad_input` path of the reference) runs one launch per
    run of consecutive equal-length sequences.  The boundaries are read on the host: one device-to-host copy of
    `cu_seqlens` when it lives on the GPU (the reference's unpad_input synchronises for max_seqlen as well)."""
    nnz, three, H, D = qkv.shape
    assert three == 3
    nseq = cu_seqlens.numel() - 1
    if nseq > 0 and nnz == nseq * max_seqlen:                # equal lengths: no host read
        x = qkv.view(nseq, max_seqlen, 3, H, D)
        o = flash_attn_func(x[:, :, 0], x[:, :, 1], x[:, :, 2], dropout_p, softmax_scale, causal)
        return o.reshape(nnz, H, D)
    cu = [int(v) for v in cu_seqlens.tolist()]
    if cu[0] != 0 or cu[-1] != nnz or any(b < a for a, b in zip(cu, cu[1:])):
        raise TimeViperHipError("flash_attn_varlen_qkvpacked_func: cu_seqlens must rise from 0 to nnz")
    out = torch.empty((nnz, H, D), dtype=qkv.dtype, device=qkv.device)
    i = 0
    while i < nseq:
        n = cu[i + 1] - cu[i]
        j = i + 1
        while j < nseq and cu[j + 1] - cu[j] == n:
            j += 1
        if n > 0:
            x = qkv[cu[i]:cu[j]].view(j - i, n, 3, H, D)
            out[cu[i]:cu[j]] = flash_attn_func(x[:, :, 0], x[:, :, 1], x[:, :, 2], dropout_p, softmax_scale,
                                               causal).reshape((j - i) * n, H, D)
        i = j
    return out


# --------------------------------------------------------------- token ops
def gather_rows(src: torch.Tensor, index: torch.Tensor) -> torch.Tensor:
    """dst[r] = src[index[r]] for a (rows, D) tensor; index int64 on the GPU."""
    _gpu(src, index)
    s2 = _rows2d(src)
    idx = index.to(torch.int64).contiguous()
    out = torch.empty((idx.numel(), s2.shape[1]), dtype=src.dtype, device=src.device)
    check(_capi.lib().tv_gather_rows(_p(s2), _p(idx), _p(out), idx.numel(), s2.shape[1],
                                     s2.stride(0), out.stride(0), _dt(src), _stream()),
          "tv_gather_rows")
    return out


def uniform_keep_indices(n_tokens: int, keep: int, offset: int = 0, device="cuda"):
    """torch.linspace(0, n-1, keep, dtype=long) with CPU semantics, + offset
    (modeling_nano.py:1946-1957), produced on the GPU, bit-exact."""
    out = torch.empty((keep,), dtype=torch.int64, device=device)
    check(_capi.lib().tv_uniform_keep_indices(_p(out), int(n_tokens), int(keep), int(offset),
                                              _stream()), "tv_uniform_keep_indices")
    return out


def dropped_indices(keep_sorted: torch.Tensor, start: int, n: int) -> torch.Tensor:
    """[start, start+n) minus keep_sorted, ascending (modeling_nano.py:1966-1970)."""
    _gpu(keep_sorted)
    ks = keep_sorted.to(torch.int64).contiguous()
    out = torch.empty((n - ks.numel(),), dtype=torch.int64, device=ks.device)
    check(_capi.lib().tv_dropped_indices(_p(ks), ks.numel(), int(start), int(n), _p(out),
                                         _stream()), "tv_dropped_indices")
    return out


def attn_rank_scores(q_row: torch.Tensor, k: torch.Tensor, n_keys: int, vis_start: int,
                     n_vis: int, scale: Optional[float] = None) -> torch.Tensor:
    """Importance of each vision token for pdrop "attn" (modeling_nano.py:1914-1939):
    q_row (Hq, D) = last prompt token's queries, k (L, Hkv, D); softmax over keys
    [0, n_keys) per head in fp32, mean over heads, slice [vis_start, vis_start+n_vis)."""
    _gpu(q_row, k)
    Hq, D = q_row.shape
    L, Hkv, _ = k.shape
    q_row = q_row.contiguous()
    if k.stride(-1) != 1:
        k = k.contiguous()
    scale = 1.0 / math.sqrt(D) if scale is None else float(scale)
    lib = _capi.lib()
    ws_bytes = lib.tv_attn_rank_workspace_bytes(int(n_keys), Hq)
    ws = torch.empty(ws_bytes, dtype=torch.uint8, device=k.device)
    scores = torch.empty((n_vis,), dtype=torch.float32, device=k.device)
    check(lib.tv_attn_rank_scores(_p(q_row), _p(k), _p(scores), int(n_keys), Hq, Hkv, D,
                                  k.stride(0), k.stride(1), int(vis_start), int(n_vis), scale,
                                  _dt(k), _p(ws), ws_bytes, _stream()), "tv_attn_rank_scores")
    return scores


def attn_rank_logits(q_row: torch.Tensor, k: torch.Tensor, scale: Optional[float] = None) -> torch.Tensor:
    """First half of `attn_rank_scores` for a sequence shard: logits (n_keys, Hq) fp32 of this
    rank's keys k (n_keys, Hkv, D) against the broadcast query row, with the reference's roundings."""
    _gpu(q_row, k)
    Hq, D = q_row.shape
    n, Hkv, _ = k.shape
    q_row = q_row.contiguous()
    if k.stride(-1) != 1:
        k = k.contiguous()
    scale = 1.0 / math.sqrt(D) if scale is None else float(scale)
    out = torch.empty((n, Hq), dtype=torch.float32, device=k.device)
    check(_capi.lib().tv_attn_rank_logits(_p(q_row), _p(k), _p(out), int(n), Hq, Hkv, D, k.stride(0),
                                          k.stride(1), scale, _dt(k), _stream()), "tv_attn_rank_logits")
    return out


def attn_rank_scores_from_logits(logits: torch.Tensor, vis_start: int, n_vis: int, dtype) -> torch.Tensor:
    """Second half: softmax over ALL keys per head, mean over heads (roundings in `dtype`, the
    activation dtype), slice [vis_start, vis_start + n_vis).  logits (n_keys, Hq) fp32."""
    _gpu(logits)
    logits = logits.contiguous()
    n, Hq = logits.shape
    ws = torch.empty(2 * Hq, dtype=torch.float32, device=logits.device)
    scores = torch.empty((n_vis,), dtype=torch.float32, device=logits.device)
    check(_capi.lib().tv_attn_rank_scores_from_logits(_p(logits), _p(scores), int(n), Hq, int(vis_start),
                                                      int(n_vis), _DT[dtype], _p(ws), ws.numel() * 4,
                                                      _stream()), "tv_attn_rank_scores_from_logits")
    return scores


# ---------------------------------------------------------------- patch embed
def apply_rotary_pos_emb_(q, k, cos, sin):
    """In-place rotary embedding of q (B, L, Hq, D) and k (B, L, Hkv, D) (views with a
    contiguous head dim) with cos / sin (B, L, D): modeling_qwen2.py:89-113."""
    _gpu(q, k, cos, sin)
    B, L, _, D = q.shape
    cs = cos.to(q.dtype).reshape(B * L, D).contiguous()
    sn = sin.to(q.dtype).reshape(B * L, D).contiguous()
    for t in (q, k):
        assert t.stride(-1) == 1 and (B == 1 or t.stride(0) == L * t.stride(1))
        check(_capi.lib().tv_rope_fwd(_p(t), _p(cs), _p(sn), B * L, t.shape[2], D, t.stride(1),
                                      t.stride(2), _dt(t), _stream()), "tv_rope_fwd")
    return q, k


def silu_mul(gate, up):
    """silu(gate) * up over the last dim (Qwen2MLP, modeling_qwen2.py:78-80)."""
    _gpu(gate, up)
    g2, u2 = _rows2d(gate), _rows2d(up)
    y = torch.empty(g2.shape, dtype=gate.dtype, device=gate.device)
    check(_capi.lib().tv_silu_mul_fwd(_p(g2), _p(u2), _p(y), g2.shape[0], g2.shape[1], g2.stride(0),
                                      u2.stride(0), y.stride(0), _dt(gate), _stream()), "tv_silu_mul_fwd")
    return y.view(gate.shape)


def tome_merge_round(x, size, r: int, heads: int = 16):
    """One ToMe round for every frame (tome.py:14-83): x (F, T, C), size (F, T, 1) or None ->
    (x' (F, T-r, C), size' (F, T-r, 1)); rows = [kept even tokens, descending match score |
    odd tokens with their merged partners], size-weighted average."""
    _gpu(x, size)
    F_, T, Cc = x.shape
    x = x.contiguous()
    sz = None if size is None else size.reshape(F_, T).to(x.dtype).contiguous()
    xo = torch.empty((F_, T - r, Cc), dtype=x.dtype, device=x.device)
    so = torch.empty((F_, T - r, 1), dtype=x.dtype, device=x.device)
    lib = _capi.lib()
    ws_bytes = lib.tv_tome_workspace_bytes(F_, T, Cc, heads)
    ws = torch.empty(max(int(ws_bytes), 16), dtype=torch.uint8, device=x.device)
    check(lib.tv_tome_merge_round(_p(x), _p(sz), _p(xo), _p(so), F_, T, Cc, heads, int(r), _dt(x),
                                  _p(ws), int(ws_bytes), _stream()), "tv_tome_merge_round")
    return xo, so


def patch_embed(pixels, weight, bias=None, pos=None, patch: Optional[int] = None):
    """pixels (F, C, H, W) -> (F, gh*gw, Dout); weight is the Conv2d weight
    (Dout, C, p, p) (or Conv3d (Dout, C, 1, p, p)); pos (gh*gw, Dout) optional."""
    _gpu(pixels, weight, bias, pos)
    F_, Cin, H, W = pixels.shape
    Dout = weight.shape[0]
    p = int(weight.shape[-1]) if patch is None else int(patch)
    pixels = pixels.contiguous()
    w = weight.reshape(Dout, -1).to(pixels.dtype).contiguous()
    assert w.shape[1] == Cin * p * p
    b = None if bias is None else bias.to(pixels.dtype).contiguous()
    ps = None if pos is None else pos.reshape(-1, Dout).to(pixels.dtype).contiguous()
    out = torch.empty((F_, (H // p) * (W // p), Dout), dtype=pixels.dtype, device=pixels.device)
    ws = torch.empty((_capi.lib().tv_patch_embed_workspace_bytes(Dout, Cin, p),), dtype=torch.uint8,
                     device=pixels.device)
    check(_capi.lib().tv_patch_embed_fwd(_p(pixels), _p(w), _p(b), _p(ps), _p(out), F_, Cin, H,
                                         W, p, Dout, _dt(pixels), _p(ws), _stream()),
          "tv_patch_embed_fwd")
    return out


def patch_embed_video(pixels, weight, bias=None, pos=None):
    """Conv3d k=s=(1,p,p) on (B, C, T, H, W) -> (B, T*gh*gw, Dout), token order
    (t, py, px) as vit_scale_clean.py:455-460."""
    _gpu(pixels, weight, bias, pos)
    B, Cin, T, H, W = pixels.shape
    Dout, p = weight.shape[0], int(weight.shape[-1])
    pixels = pixels.contiguous()
    w = weight.reshape(Dout, -1).to(pixels.dtype).contiguous()
    b = None if bias is None else bias.to(pixels.dtype).contiguous()
    ps = None if pos is None else pos.reshape(-1, Dout).to(pixels.dtype).contiguous()
    npatch = (H // p) * (W // p)
    out = torch.empty((B, T * npatch, Dout), dtype=pixels.dtype, device=pixels.device)
    ws = torch.empty((_capi.lib().tv_patch_embed_workspace_bytes(Dout, Cin, p),), dtype=torch.uint8,
                     device=pixels.device)
    check(_capi.lib().tv_patch_embed_strided_fwd(
        _p(pixels), _p(w), _p(b), _p(ps), _p(out), B * T, Cin, H, W, p, Dout, T,
        Cin * T * H * W, H * W, T * H * W, _dt(pixels), _p(ws), _stream()), "tv_patch_embed_strided_fwd")
    return out


# ------------------------------------------------- post-norm models on a 32-bit residual stream
def _vec(t: torch.Tensor, n: int, what: str) -> torch.Tensor:
    if t.numel() != n or not t.is_contiguous():
        raise TimeViperHipError(f"{what}: a contiguous vector of {n} entries is needed, got {tuple(t.shape)}")
    return t


def _i32(t: Optional[torch.Tensor], n: int, what: str) -> None:
    if t is not None and (t.dtype != torch.int32 or t.numel() < n or not t.is_contiguous()):
        raise TimeViperHipError(f"{what}: a contiguous int32 tensor of {n} entries is needed")


def rms_norm_ex(x, weight, eps, weight_offset=0.0, gate=None, residual=None, mult=1.0, out_dtype=None, sum_out=None,
                y2=None, y2_rows=None, need_y=True):
    """n = x / sqrt(mean(x^2) + eps) * (weight_offset + weight) over the last dim [, * sigmoid(gate)].  With `residual` (fp32):
    s = residual + mult * n; returns (y, s) with y = s in `out_dtype` (default: the weight's).  Without: returns n.
    `y2` / `y2_rows`: the result rows are written to rows y2_rows of the 2-D buffer y2 as well (a cache)."""
    _gpu(x, weight, gate, residual, sum_out, y2, y2_rows)
    x2 = _rows2d(x)
    rows, D = x2.shape
    _vec(weight, D, "rms_norm_ex weight")
    yd = out_dtype or weight.dtype
    g2 = None if gate is None else _rows2d(gate)
    r2 = s2 = None
    if gate is not None and (gate.dtype != weight.dtype or g2.shape != x2.shape):
        raise TimeViperHipError("rms_norm_ex: gate must have x's shape and the weight's dtype")
    if residual is not None:
        r2 = _rows2d(residual)
        if residual.dtype != torch.float32 or r2.shape != x2.shape:
            raise TimeViperHipError("rms_norm_ex: the residual is fp32 and has x's shape")
        s2 = torch.empty((rows, D), dtype=torch.float32, device=x.device) if sum_out is None else _rows2d(sum_out)
        if s2.dtype != torch.float32 or s2.shape != x2.shape:
            raise TimeViperHipError("rms_norm_ex: sum_out is fp32 and has x's shape")
    y = torch.empty((rows, D), dtype=yd, device=x.device) if need_y else None
    if y2 is not None:
        _i32(y2_rows, rows, "rms_norm_ex y2_rows")
        if y2.dtype != yd or y2.dim() != 2 or y2.shape[1] != D or y2.stride(1) != 1:
            raise TimeViperHipError("rms_norm_ex: y2 is a (rows, D) buffer of the output dtype")
    st = lambda t: 0 if t is None else t.stride(0)
    check(_capi.lib().tv_rmsnorm_ex_fwd(
        _p(x2), _p(weight), _p(g2), _p(r2), _p(s2), _p(y), _p(y2), _p(y2_rows), st(y2), rows, D, x2.stride(0), st(g2), st(r2), st(s2),
        st(y), float(eps), float(mult), float(weight_offset), _dt(x), _dt(weight), _DT[yd], _stream()), "tv_rmsnorm_ex_fwd")
    y = None if y is None else y.view(x.shape)
    return y if residual is None else (y, s2.view(x.shape))


def moe_combine_norm(expert_out, pos, weights, residual, norm_weight, eps, weight_offset=0.0, mult=1.0, out_dtype=None):
    """u = sum_j weights[:, j] * expert_out[pos[:, j]] (pos < 0: the residual row, an identity expert), then as `rms_norm_ex` with
    this residual.  Returns (y, s)."""
    _gpu(expert_out, pos, weights, residual, norm_weight)
    rows, D = residual.shape
    top = pos.shape[1]
    _i32(pos, rows * top, "moe_combine_norm pos")
    _vec(norm_weight, D, "moe_combine_norm weight")
    if (residual.dtype != torch.float32 or residual.stride(1) != 1 or weights.dtype != torch.float32 or not weights.is_contiguous()
            or weights.shape != pos.shape or expert_out.shape[1] != D or expert_out.stride(1) != 1):
        raise TimeViperHipError("moe_combine_norm: fp32 residual (rows, D), fp32 weights (rows, top), expert rows of D elements")
    yd = out_dtype or norm_weight.dtype
    y = torch.empty((rows, D), dtype=yd, device=residual.device)
    s = torch.empty((rows, D), dtype=torch.float32, device=residual.device)
    check(_capi.lib().tv_moe_combine_norm_fwd(
        _p(expert_out), _p(pos), _p(weights), top, _p(residual), _p(norm_weight), _p(s), _p(y), rows, D, expert_out.stride(0),
        residual.stride(0), s.stride(0), y.stride(0), float(eps), float(mult), float(weight_offset), _dt(expert_out),
        _dt(norm_weight), _DT[yd], _stream()), "tv_moe_combine_norm_fwd")
    return y, s


def embed_scaled(ids, table, scale=1.0, positions=None, plan=None, need_h=True):
    """(fp32 rows, rows in the table's dtype) of `table[ids] * scale`; ids int64 on the GPU.  `positions` (max, D): the row of the
    token's place in its sequence is added (plan: the step's `cache.StepPlan`; its places lie within the table)."""
    _gpu(ids, table, positions)
    flat = ids.reshape(-1).contiguous()
    V, D = table.shape
    if flat.dtype != torch.int64 or not table.is_contiguous():
        raise TimeViperHipError("embed_scaled: int64 ids and a contiguous table")
    x = torch.empty((flat.numel(), D), dtype=torch.float32, device=table.device)
    h = torch.empty((flat.numel(), D), dtype=table.dtype, device=table.device) if need_h else None
    seq = cu = start = None
    if positions is not None:
        seq, cu, start = _plan(plan, flat.numel(), "embed_scaled")[:3]
        if positions.dtype != table.dtype or positions.dim() != 2 or positions.shape[1] != D or not positions.is_contiguous():
            raise TimeViperHipError("embed_scaled: positions (max, D) of the table's dtype")
    check(_capi.lib().tv_embed_scaled_fwd(_p(flat), _p(table), _p(x), _p(h), flat.numel(), D, V, float(scale), _p(positions), _p(seq), _p(cu),
                                          _p(start), 0 if positions is None else positions.shape[0], _dt(table), _stream()),
          "tv_embed_scaled_fwd")
    return x, h


# ------------------------------------------------- parallel layers on a 32-bit residual stream
def _plan(plan, rows, what):
    """(seq, cu, start, slot) of a step's plan for `rows` packed rows"""
    B = len(plan.slots)
    if plan.rows.numel() != rows:
        raise TimeViperHipError(f"{what}: {rows} rows in a step of {plan.rows.numel()}")
    for t, n in ((plan.seq, rows), (plan.cu, B + 1), (plan.start, B), (plan.slot, B)):
        _gpu(t)
        _i32(t, n, what + " plan")
    return plan.seq, plan.cu, plan.start, plan.slot


def _shift_state(state, plan, D, what):
    """(slots, 2, D) fp32 blocks, possibly one layer's slice of a wider state: the distance between two blocks"""
    if (state.dtype != torch.float32 or state.dim() != 3 or state.shape[1:] != (2, D) or state.stride(2) != 1 or state.stride(1) != D
            or max(plan.slots) >= state.shape[0]):
        raise TimeViperHipError(f"{what}: a (slots, 2, {D}) fp32 state with dense blocks")
    return state.stride(0)


def norm_shift(x, gain, eps, pending=None, pending_weight=None, shift=None, state=None, plan=None, need_h=True):
    """x (T, D) fp32 -> (x', h, hs): x' = x + rms(pending) * pending_weight (x itself without `pending`), h = rms(x') * gain (a tensor of one
    element), hs = h + (h_before - h) * shift with the h of the sequence's previous token (`state` (slots, 2, D) fp32, advanced in
    place; None without `shift`).  h and hs have the gain's dtype."""
    _gpu(x, gain, pending, pending_weight, shift, state)
    T, D = x.shape
    if x.dtype != torch.float32 or not x.is_contiguous() or gain.numel() != 1:
        raise TimeViperHipError("norm_shift: dense fp32 rows and a gain of one element")
    xo, ps = None, 0
    if pending is not None:
        if pending.shape != x.shape or pending.dtype != gain.dtype or pending.stride(1) != 1 or pending_weight.dtype != gain.dtype:
            raise TimeViperHipError("norm_shift: pending rows and weight of x's width and the gain's dtype")
        _vec(pending_weight, D, "norm_shift pending weight")
        xo, ps = torch.empty_like(x), pending.stride(0)
    h = torch.empty((T, D), dtype=gain.dtype, device=x.device) if need_h or shift is None else None
    hs, seq, cu, start, slot, sst = None, None, None, None, None, 0
    if shift is not None:
        _vec(shift, D, "norm_shift shift")
        if shift.dtype != gain.dtype:
            raise TimeViperHipError("norm_shift: shift of the gain's dtype")
        hs = torch.empty((T, D), dtype=gain.dtype, device=x.device)
        seq, cu, start, slot = _plan(plan, T, "norm_shift")
        sst = _shift_state(state, plan, D, "norm_shift")
    check(_capi.lib().tv_norm_shift_fwd(
        _p(x), _p(pending), _p(pending_weight), _p(xo), _p(gain), _p(shift), _p(state if shift is not None else None), _p(seq), _p(cu), _p(start), _p(slot),
        _p(h), _p(hs), T, D, ps, sst, float(eps), int(plan is not None and plan.decode), _dt(gain), _stream()), "tv_norm_shift_fwd")
    return x if xo is None else xo, h, hs


def residual_add(x, u):
    """(x + u in fp32, its rounding to u's dtype); x (T, D) fp32"""
    _gpu(x, u)
    if x.dtype != torch.float32 or not x.is_contiguous() or u.shape != x.shape or u.stride(1) != 1:
        raise TimeViperHipError("residual_add: dense fp32 x and u of its shape")
    xo, h = torch.empty_like(x), torch.empty(x.shape, dtype=u.dtype, device=x.device)
    check(_capi.lib().tv_residual_add_fwd(_p(x), _p(u), _p(xo), _p(h), x.shape[0], x.shape[1], u.stride(0), _dt(u), _stream()),
          "tv_residual_add_fwd")
    return xo, h


ACT_SIGMOID, ACT_GELU_TANH = 0, 1


def gated_mul(a, b, act, ids=None, out=None):
    """f(a) * b over rows, f = sigmoid or the tanh form of gelu; `ids` (int64): row r meets b[ids[r]].  `out`: rows to write to."""
    _gpu(a, b, ids, out)
    T, n = a.shape
    o = torch.empty((T, n), dtype=a.dtype, device=a.device) if out is None else out
    if (b.dtype != a.dtype or b.dim() != 2 or b.shape[1] != n or o.shape != a.shape or o.dtype != a.dtype or any(t.stride(1) != 1 for t in (a, b, o))
            or (ids is None and b.shape[0] != T) or (ids is not None and (ids.dtype != torch.int64 or ids.numel() != T or not ids.is_contiguous()))):
        raise TimeViperHipError(f"gated_mul: a {tuple(a.shape)} against b {tuple(b.shape)}")
    check(_capi.lib().tv_gated_mul_fwd(_p(a), _p(b), _p(ids), _p(o), T, n, a.stride(0), b.stride(0), o.stride(0), b.shape[0], int(act), _dt(a),
                                       _stream()), "tv_gated_mul_fwd")
    return o


def scatter_rows(src, rows, dst):
    """dst[rows] = src (rows int32 on the GPU, within dst)"""
    _gpu(src, rows, dst)
    _i32(rows, src.shape[0], "scatter_rows rows")
    if src.dtype != dst.dtype or src.shape[1] != dst.shape[1] or src.stride(1) != 1 or dst.stride(1) != 1:
        raise TimeViperHipError("scatter_rows: rows of one width and dtype")
    check(_capi.lib().tv_scatter_rows(_p(src), _p(rows), _p(dst), src.shape[0], src.shape[1], src.stride(0), dst.stride(0), _dt(src), _stream()),
          "tv_scatter_rows")


# ------------------------------------------------- linear attention with a constant decay per head
def lightning_attention(q, k, v, decay, state, cu_seqlens, slot, nheads, max_len, silu=True, out=None):
    """S_t = decay_h S_(t-1) + k_t v_t^T, o_t = S_t^T q_t for a ragged batch.  q, k (T, H * dk), v (T, H * dv): rows of a
    projection output (any row stride); decay (H) fp32; state (slots, H, dk, dv) fp32, advanced in place for the slots of this
    batch; cu_seqlens (B + 1) / slot (B) int32 on the GPU; max_len: the longest sequence's rows.  `silu`: q, k, v pass through SiLU here.  Returns (T, H * dv)."""
    _gpu(q, k, v, decay, state, cu_seqlens, slot)
    B = slot.numel()
    _i32(cu_seqlens, B + 1, "lightning_attention cu_seqlens")
    _i32(slot, B, "lightning_attention slot")
    T = q.shape[0]
    _, H, dk, dv = state.shape
    if H != nheads or q.shape != (T, H * dk) or k.shape != q.shape or v.shape != (T, H * dv):
        raise TimeViperHipError(f"lightning_attention: q {tuple(q.shape)}, k {tuple(k.shape)}, v {tuple(v.shape)}, state {tuple(state.shape)}")
    if state.dtype != torch.float32 or not state.is_contiguous() or decay.dtype != torch.float32 or k.dtype != q.dtype or v.dtype != q.dtype:
        raise TimeViperHipError("lightning_attention: fp32 contiguous state and decay; q, k, v of one dtype")
    if any(t.stride(1) != 1 for t in (q, k, v)) or not (1 <= max_len <= T) or (max_len == 1 and T != B):
        raise TimeViperHipError("lightning_attention: dense rows; max_len rows in the longest sequence")
    _vec(decay, H, "lightning_attention decay")
    o = torch.empty((T, H * dv), dtype=q.dtype, device=q.device) if out is None else out
    lib = _capi.lib()
    nbytes = int(lib.tv_lightning_workspace_bytes(B, int(max_len), H, dk, dv, _dt(q))) if max_len > 1 else 0
    ws = torch.empty(nbytes, dtype=torch.uint8, device=q.device) if nbytes else None
    check(lib.tv_lightning_fwd(
        _p(q), _p(k), _p(v), _p(decay), _p(state), _p(o), _p(cu_seqlens), _p(slot), B, int(max_len), _p(ws), nbytes, H, dk, dv,
        q.stride(0), k.stride(0), v.stride(0), o.stride(0), int(bool(silu)), _dt(q), _stream()), "tv_lightning_fwd")
    return o


# ------------------------------------------------- attention without shape limits, latent attention
NO_WINDOW = 2 ** 31 - 1


def attention_generic(q, k, v, cu_seqlens, scale, causal=True, sink=None, start=None, slot=None, window=NO_WINDOW, keep_first=0, gate=None,
                      out=None):
    """q (T, Hq, dk) packed rows of B sequences (cu_seqlens (B + 1) int32); k (blocks, Lk, Hkv, dk), v (blocks, Lk, Hkv, dv): sequence b
    reads block slot[b] (default b).  Row i of a sequence sees keys [0, start[b] + i] when causal — with a window, the last `window` of
    them and the first `keep_first`.  gate (T, Hq, dv): the result times sigmoid(gate).  Returns (T, Hq, dv)."""
    _gpu(q, k, v, cu_seqlens, sink, start, slot, gate, out)
    T, Hq, dk = q.shape
    B = cu_seqlens.numel() - 1
    Hkv, dv = k.shape[2], v.shape[3]
    for t, n, what in ((cu_seqlens, B + 1, "cu_seqlens"), (start, B, "start"), (slot, B, "slot")):
        _i32(t, n, "attention_generic " + what)
    if k.dtype != q.dtype or v.dtype != q.dtype or any(t.stride(-1) != 1 for t in (q, k, v)) or k.shape[3] != dk or v.shape[:3] != k.shape[:3]:
        raise TimeViperHipError("attention_generic: q, k, v of one dtype with dense last dims and matching shapes")
    if sink is not None:
        if sink.dtype != torch.float32:
            raise TimeViperHipError("attention_generic: fp32 sinks")
        _vec(sink, Hq, "attention_generic sink")
    o = torch.empty((T, Hq, dv), dtype=q.dtype, device=q.device) if out is None else out
    for t in (o, gate):
        if t is not None and (t.shape != (T, Hq, dv) or t.dtype != q.dtype or t.stride(2) != 1):
            raise TimeViperHipError("attention_generic: gate and out (T, Hq, dv) of q's dtype with dense last dims")
    check(_capi.lib().tv_attn_generic_fwd(
        _p(q), _p(k), _p(v), _p(sink), _p(o), _p(cu_seqlens), _p(start), _p(slot), B, T, Hq, Hkv, dk, dv, q.stride(0), q.stride(1),
        k.stride(0), k.stride(1), k.stride(2), v.stride(0), v.stride(1), v.stride(2), o.stride(0), o.stride(1), float(scale),
        int(bool(causal)), int(window), int(keep_first), _p(gate), 0 if gate is None else gate.stride(0),
        0 if gate is None else gate.stride(1), _dt(q), _stream()), "tv_attn_generic_fwd")
    return o


def _cache_views(cache, kv_heads, dim, vdim):
    """keys (slots, capacity, kv_heads, dim) and values (slots, capacity, kv_heads, vdim) of rows that hold both side by side"""
    slots, cap, W = cache.shape
    if W != kv_heads * (dim + vdim) or not cache.is_contiguous():
        raise TimeViperHipError(f"cache rows of {W} elements for {kv_heads} x ({dim} + {vdim})")
    k, v = cache.split([kv_heads * dim, kv_heads * vdim], dim=2)
    return k.unflatten(2, (kv_heads, dim)), v.unflatten(2, (kv_heads, vdim))


def attention_window(q, cache, plan, kv_heads, scale, window=NO_WINDOW, keep_first=0, gate=None, out=None):
    """Causal attention of a step's packed rows against a slot cache that already holds the step's own keys and values: q (T, H, dk), cache
    (slots, capacity, kv_heads * (dk + dv)), a row = all keys, then all values; the query at position p sees keys (p - window, p]
    and the first `keep_first` of its sequence.  gate (T, H, dv): the result times sigmoid(gate).  out (T, H, dv).  plan: the step's
    `cache.StepPlan`."""
    T, H, dk = q.shape
    dv = cache.shape[2] // kv_heads - dk
    k, v = _cache_views(cache, kv_heads, dk, dv)
    _, cu, start, slot = _plan(plan, T, "attention_window")
    if max(plan.slots) >= cache.shape[0] or max(a + n for a, n in zip(plan.starts, plan.counts)) > cache.shape[1]:
        raise TimeViperHipError("attention_window: the cache does not hold the step's tokens")
    o = torch.empty((T, H, dv), dtype=q.dtype, device=q.device) if out is None else out
    rows8 = lambda t: t is None or (all(s % 4 == 0 for s in t.stride()[:2]) and t.data_ptr() % 8 == 0 and t.stride(2) == 1)
    if not (q.dtype == torch.bfloat16 and cache.dtype == q.dtype and _flash_rows(q) and _flash_rows(k[0]) and _flash_rows(v[0]) and rows8(gate)
            and rows8(o) and scale > 0):
        return attention_generic(q, k, v, cu, scale, start=start, slot=slot, window=window, keep_first=keep_first, gate=gate, out=o)
    _gpu(q, cache, gate, o)
    if H % kv_heads or any(t is not None and (t.shape != (T, H, dv) or t.dtype != q.dtype) for t in (gate, o)):
        raise TimeViperHipError("attention_window: gate and out (T, H, dv) of q's dtype")
    lib, at = _capi.lib(), 0
    for s, n, a in zip(plan.slots, plan.counts, plan.starts):
        sl = slice(at, at + n)
        gb = None if gate is None else gate[sl]
        check(lib.tv_flash_attn_window_fwd(
            _p(q[sl]), _p(k[s]), _p(v[s]), _p(o[sl]), _p(gb), int(window), int(keep_first), dv, n, a + n, H, kv_heads, dk, q.stride(0), q.stride(1),
            k.stride(1), k.stride(2), v.stride(1), v.stride(2), o.stride(0), o.stride(1), 0 if gate is None else gate.stride(0),
            0 if gate is None else gate.stride(1), float(scale), _dt(q), _stream()), "tv_flash_attn_window_fwd")
        at += n
    return o


def attention_window_decode(q, cache, plan, kv_heads, scale, window=NO_WINDOW, keep_first=0, gate=None, fresh=None, out=None):
    """`attention_window` for a step of single tokens: q (B, H, dk), gate (B, H, dv).  fresh (B, kv_heads * (dk + dv)): the step's own cache
    rows, which are written here (without it they are in the cache already).  Key counts are read on the device.  Returns (B, H, dv)
    (`out`: where to)."""
    B, H, dk = q.shape
    dv = cache.shape[2] // kv_heads - dk
    k, v = _cache_views(cache, kv_heads, dk, dv)
    _, cu, start, slot = _plan(plan, B, "attention_window_decode")
    if not plan.decode or max(plan.slots) >= cache.shape[0] or H % kv_heads:
        raise TimeViperHipError("attention_window_decode: one token per sequence, each with a slot of the cache")
    _gpu(q, cache, gate, fresh, out, plan.keys)
    _i32(plan.keys, B, "attention_window_decode keys")
    if fresh is not None and (fresh.shape != (B, cache.shape[2]) or fresh.dtype != cache.dtype or fresh.stride(1) != 1):
        raise TimeViperHipError("attention_window_decode: new rows of the cache's width and dtype")
    dense = lambda t: t is None or (t.stride(2) == 1 and t.stride(1) == t.shape[2])
    ok16 = lambda t: t is None or (t.stride(0) % 8 == 0 and t.data_ptr() % 16 == 0)
    if (q.dtype == torch.bfloat16 and cache.dtype == q.dtype and dk % 8 == 0 and dv % 8 == 0 and max(dk, dv) <= 256 and dense(q) and dense(gate)
            and dense(out) and ok16(q) and ok16(fresh) and ok16(cache)):
        if any(t is not None and (t.shape != (B, H, dv) or t.dtype != q.dtype) for t in (gate, out)):
            raise TimeViperHipError("attention_window_decode: gate and out (B, H, dv) of q's dtype")
        o = torch.empty((B, H, dv), dtype=q.dtype, device=q.device) if out is None else out
        lib, cap = _capi.lib(), cache.shape[1]
        nbytes = int(lib.tv_attn_window_decode_workspace_bytes(B, H, kv_heads, dv, cap, int(window), int(keep_first)))
        ws = torch.empty(nbytes, dtype=torch.uint8, device=q.device) if nbytes else None
        check(lib.tv_attn_window_decode_fwd(
            _p(q), _p(cache), _p(fresh), _p(gate), _p(o), _p(plan.keys), _p(slot), B, H, kv_heads, dk, dv, cap, int(window), int(keep_first),
            q.stride(0), 0 if fresh is None else fresh.stride(0), 0 if gate is None else gate.stride(0), o.stride(0), float(scale), _p(ws), nbytes,
            _stream()), "tv_attn_window_decode_fwd")
        return o
    if fresh is not None:
        scatter_rows(fresh, plan.rows, cache.view(-1, cache.shape[2]))
    return attention_generic(q, k, v, cu, scale, start=start, slot=slot, window=window, keep_first=keep_first, gate=gate, out=out)


def _flash_rows(t: torch.Tensor) -> bool:
    """(rows, heads, dim) operands of tv_flash_attn_sink_fwd"""
    return t.shape[-1] % 8 == 0 and t.shape[-1] <= 128 and t.stride(-1) == 1 and all(s % 8 == 0 for s in t.stride()[:2]) \
        and t.data_ptr() % 16 == 0


def _flash_sink(q, k, v, counts, starts, scale, sink):
    T, Hq, D = q.shape
    Hkv, Dv = k.shape[1], v.shape[2]
    _gpu(q, k, v, sink)
    o = torch.empty((T, Hq, Dv), dtype=q.dtype, device=q.device)
    lib, at, kt = _capi.lib(), 0, 0
    for n, a in zip(counts, starts):
        qb, kb, vb, ob = q[at:at + n], k[kt:kt + a + n], v[kt:kt + a + n], o[at:at + n]
        check(lib.tv_flash_attn_sink_fwd(
            _p(qb), _p(kb), _p(vb), _p(ob), _p(sink), Dv, 1, n, a + n, Hq, Hkv, D, 0, q.stride(0), q.stride(1), 0, k.stride(0), k.stride(1),
            0, v.stride(0), v.stride(1), 0, o.stride(0), o.stride(1), float(scale), _dt(q), _stream()), "tv_flash_attn_sink_fwd")
        at, kt = at + n, kt + a + n
    return o


def attention_sink(q, k, v, cu_q, cu_k, start, counts, starts, scale, sink):
    """Causal attention over a ragged batch with a sink logit per head.  q (T, H, dk): sequence b owns rows [cu_q[b], cu_q[b + 1]);
    k (Tk, H, dk), v (Tk, H, dv): rows [cu_k[b], cu_k[b + 1]), start[b] = the keys in front of the sequence's first query row
    (int32 tensors on the GPU; `counts` / `starts`: the same per sequence on the host).  Returns (T, H, dv)."""
    if q.dtype == torch.bfloat16 and all(_flash_rows(t) for t in (q, k, v)):
        return _flash_sink(q, k, v, counts, starts, scale, sink)
    blocks = lambda t: t.as_strided((t.shape[0], 1) + t.shape[1:], (t.stride(0),) + t.stride())      # a "block" per row: slot = first row
    return attention_generic(q, blocks(k), blocks(v), cu_q, scale, sink=sink, start=start, slot=cu_k[:-1])


def _latent_args(t, w, nheads, what):
    if t.dtype != w.dtype or t.stride(1) != 1 or w.stride(1) != 1 or t.shape[1] % nheads or w.shape[0] % nheads:
        raise TimeViperHipError(f"{what}: operands of one dtype with dense rows, heads contiguous")


def latent_query(q, w_uk, nheads):
    """(B, H * dim), W_uk (H * dim, rank) -> (B, H, rank): the query against the latents themselves."""
    _gpu(q, w_uk)
    _latent_args(q, w_uk, nheads, "latent_query")
    B, rank, dim = q.shape[0], w_uk.shape[1], w_uk.shape[0] // nheads
    if q.shape[1] != nheads * dim:
        raise TimeViperHipError("latent_query: q and W_uk disagree about the head size")
    y = torch.empty((B, nheads, rank), dtype=q.dtype, device=q.device)
    check(_capi.lib().tv_latent_query_fwd(_p(q), _p(w_uk), _p(y), B, nheads, dim, rank, q.stride(0), w_uk.stride(0), y.stride(0), _dt(q),
                                          _stream()), "tv_latent_query_fwd")
    return y


def latent_value(y, w_uv, nheads):
    """(B, H, rank), W_uv (H * vdim, rank) -> (B, H * vdim)."""
    _gpu(y, w_uv)
    B, H, rank = y.shape
    vdim = w_uv.shape[0] // nheads
    if H != nheads or w_uv.shape != (H * vdim, rank) or not y.is_contiguous() or w_uv.stride(1) != 1 or y.dtype != w_uv.dtype:
        raise TimeViperHipError("latent_value: y (B, H, rank) contiguous, W_uv (H * vdim, rank)")
    o = torch.empty((B, H * vdim), dtype=y.dtype, device=y.device)
    check(_capi.lib().tv_latent_value_fwd(_p(y), _p(w_uv), _p(o), B, H, vdim, rank, y.stride(0), w_uv.stride(0), o.stride(0), _dt(y),
                                          _stream()), "tv_latent_value_fwd")
    return o


def latent_decode(q, w_uk, w_uv, latents, keys, slot, nheads, scale, sink, new=None):
    """One token per sequence: q (B, H * dim) against the first keys[b] (int32, on the GPU) rows of latents[slot[b]] (slots, capacity,
    rank) -> (B, H * vdim), what attention over the expanded keys W_uk c and values W_uv c gives.
    `new=(c, norm_weight, eps, rows)`: the step's own down projections (B, rank); their normed rows go to the cache rows `rows` (of
    the (slots * capacity, rank) view) first."""
    _gpu(q, w_uk, w_uv, latents, keys, slot, sink)
    B, R = q.shape[0], latents.shape[2]
    _latent_args(q, w_uk, nheads, "latent_decode")
    dim, vdim = w_uk.shape[0] // nheads, w_uv.shape[0] // nheads
    _i32(keys, B, "latent_decode keys")
    _i32(slot, B, "latent_decode slot")
    if (q.shape[1] != nheads * dim or w_uk.shape[1] != R or w_uv.shape != (nheads * vdim, R) or latents.dtype != q.dtype
            or w_uv.dtype != q.dtype or not latents.is_contiguous()):
        raise TimeViperHipError("latent_decode: q, W_uk, W_uv and the latents disagree")
    if new is not None:
        c, cn, _, rows = new
        _gpu(c, cn, rows)
        _i32(rows, B, "latent_decode rows")
        _vec(cn, R, "latent_decode norm weight")
        if c.shape != (B, R) or c.dtype != q.dtype or cn.dtype != q.dtype or c.stride(1) != 1:
            raise TimeViperHipError("latent_decode: new latents (B, rank) of the model's dtype")
    if (q.dtype == torch.bfloat16 and R % 8 == 0 and R <= 512 and w_uk.is_contiguous() and w_uv.is_contiguous()
            and all(t.data_ptr() % 16 == 0 for t in (w_uk, w_uv, latents))):
        _vec(sink, nheads, "latent_decode sink")
        c, cn, eps, rows = new if new is not None else (None, None, 0.0, None)
        o = torch.empty((B, nheads * vdim), dtype=q.dtype, device=q.device)
        lib = _capi.lib()
        nbytes = int(lib.tv_latent_decode_workspace_bytes(B, nheads, R, latents.shape[1]))
        ws = torch.empty(nbytes, dtype=torch.uint8, device=q.device)
        check(lib.tv_latent_decode_fwd(
            _p(q), _p(w_uk), _p(w_uv), _p(latents), _p(c), _p(cn), float(eps), _p(rows), _p(keys), _p(slot), _p(sink), _p(o), B, nheads,
            dim, vdim, R, latents.shape[1], q.stride(0), 0 if c is None else c.stride(0), o.stride(0), float(scale), _p(ws), nbytes,
            _stream()), "tv_latent_decode_fwd")
        return o
    if new is not None:
        rms_norm_ex(new[0], new[1], new[2], y2=latents.view(-1, R), y2_rows=new[3], need_y=False)
    ql = latent_query(q, w_uk, nheads)
    kv = latents.unsqueeze(2)                                   # one shared key / value head of `rank` dimensions
    cu = torch.arange(B + 1, dtype=torch.int32, device=q.device)
    y = attention_generic(ql, kv, kv, cu, scale, sink=sink, start=keys - 1, slot=slot)
    return latent_value(y, w_uv, nheads)


# ------------------------------------------------- decode-step linear layers of post-norm models
GEMV_POSTNORM, GEMV_NORMGATE = 4, 5


def gemv_post_takes(rows: int, width: int, dtype) -> bool:
    """Shapes of tv_gemv_post_fwd with a norm prologue: 1..4 bf16 rows of up to 8 192 elements."""
    return dtype == torch.bfloat16 and 1 <= rows <= 4 and width % 8 == 0 and width <= 8192 and rows * width * 2 <= 128 * 1024


def gemv_post(x, weight, prologue=GEMV_NONE, residual=None, norm_weight=None, eps=0.0, weight_offset=0.0, mult=1.0, gate=None,
              out_dtype=torch.bfloat16):
    """y = f(x) @ weight.T for 1..4 bf16 rows.  GEMV_NONE: f(x) = x.  GEMV_POSTNORM: the norm of a sublayer's output x, the residual
    add x' = residual + mult * rms(x) * (weight_offset + norm_weight) in fp32, f = x' in bf16; returns (y, x', bf16 x').
    GEMV_NORMGATE: f = rms(x) * norm_weight * sigmoid(gate)."""
    _gpu(x, weight, residual, norm_weight, gate)
    M, Kd = x.shape
    N = weight.shape[0]
    if x.dtype != torch.bfloat16 or weight.dtype != torch.bfloat16 or weight.shape[1] != Kd or x.stride(1) != 1 or weight.stride(1) != 1:
        raise TimeViperHipError(f"gemv_post: bf16 rows x {tuple(x.shape)} against weight {tuple(weight.shape)}")
    y = torch.empty((M, N), dtype=out_dtype, device=x.device)
    xs = hs = None
    if prologue == GEMV_POSTNORM:
        if residual is None or residual.dtype != torch.float32 or residual.shape != x.shape or not residual.is_contiguous():
            raise TimeViperHipError("gemv_post: a dense fp32 residual of x's shape")
        xs, hs = torch.empty_like(residual), torch.empty((M, Kd), dtype=x.dtype, device=x.device)
    if gate is not None and (gate.shape != x.shape or gate.dtype != x.dtype or gate.stride(1) != 1):
        raise TimeViperHipError("gemv_post: gate must have x's shape and dtype")
    if norm_weight is not None:
        _vec(norm_weight, Kd, "gemv_post norm weight")
    check(_capi.lib().tv_gemv_post_fwd(
        _p(x), _p(weight), _p(y), _DT[out_dtype], M, N, Kd, x.stride(0), weight.stride(0), N, int(prologue), _p(residual), _p(xs), _p(hs),
        _p(norm_weight), 0 if norm_weight is None else _dt(norm_weight), float(weight_offset), float(mult), float(eps), _p(gate),
        0 if gate is None else gate.stride(0), _stream()), "tv_gemv_post_fwd")
    return (y, xs, hs) if prologue == GEMV_POSTNORM else y


def gemv_rows_take(rows: int, width: int, dtype) -> bool:
    """Shapes of gemv_pair, gemv_add and gemv_glu: 1..4 bf16 rows that fit the LDS."""
    return dtype == torch.bfloat16 and 1 <= rows <= 4 and width % 8 == 0 and rows * width * 2 <= 128 * 1024


def _gemv_rows(what, weight, *rows):
    if weight.dtype != torch.bfloat16 or weight.dim() != 2 or weight.stride(1) != 1 or any(
            t.dtype != torch.bfloat16 or t.shape != rows[0].shape or t.shape[1] != weight.shape[1] or t.stride(1) != 1 for t in rows):
        raise TimeViperHipError(f"{what}: bf16 rows {tuple(rows[0].shape)} against weight {tuple(weight.shape)}")


def _bf16_bias(t, n, what):
    if t is not None:
        _vec(t, n, what)
        if t.dtype != torch.bfloat16:
            raise TimeViperHipError(f"{what}: bf16")


def gemv_pair(x, x2, weight, n1, bias=None, act_out=None):
    """Both input products of a parallel layer for 1..4 bf16 rows, one launch: y = x @ weight[:n1].T (returned) and, when weight has more
    rows (gate | up), act_out = gelu_tanh(x2 @ gate.T + b) * (x2 @ up.T + b), bias = their biases."""
    _gpu(x, x2, weight, bias, act_out)
    M, D = x.shape
    ff = (weight.shape[0] - n1) // 2
    _gemv_rows("gemv_pair", weight, x, *((x2,) if ff else ()))
    if weight.shape[0] != n1 + 2 * ff or n1 < 1 or (ff and (bias is None or act_out is None or act_out.shape != (M, ff) or act_out.dtype != x.dtype
                                                          or act_out.stride(1) != 1)):
        raise TimeViperHipError(f"gemv_pair: weight rows {n1} + 2 x {ff}, biases and an (M, {ff}) output for the second part")
    if ff:
        _bf16_bias(bias, 2 * ff, "gemv_pair bias")
    y = torch.empty((M, n1), dtype=x.dtype, device=x.device)
    check(_capi.lib().tv_gemv_pair_fwd(_p(x), _p(x2) if ff else None, _p(weight), _p(bias), _p(y), _p(act_out) if ff else None, M, int(n1), ff, D,
                                       x.stride(0), x2.stride(0) if ff else 0, weight.stride(0), n1, act_out.stride(0) if ff else 0, _stream()),
          "tv_gemv_pair_fwd")
    return y


def gemv_add(x, weight, residual, bias=None):
    """(residual + x @ weight.T + bias in fp32, its bf16 rounding) for 1..4 bf16 rows; residual (M, N) fp32"""
    _gpu(x, weight, bias, residual)
    _gemv_rows("gemv_add", weight, x)
    M, N = x.shape[0], weight.shape[0]
    _bf16_bias(bias, N, "gemv_add bias")
    if residual.dtype != torch.float32 or residual.shape != (M, N) or not residual.is_contiguous():
        raise TimeViperHipError("gemv_add: a dense fp32 residual (M, N)")
    xo, h = torch.empty_like(residual), torch.empty((M, N), dtype=x.dtype, device=x.device)
    check(_capi.lib().tv_gemv_add_fwd(_p(x), _p(weight), _p(bias), _p(residual), _p(xo), _p(h), M, N, x.shape[1], x.stride(0), weight.stride(0),
                                      _stream()), "tv_gemv_add_fwd")
    return xo, h


def gemv_glu(z, u, weight, ids=None):
    """(gelu_tanh(z) * u) @ weight.T for 1..4 bf16 rows; `ids` (int64): row m meets u[ids[m]]"""
    _gpu(z, u, weight, ids)
    _gemv_rows("gemv_glu", weight, z)
    M, N = z.shape[0], weight.shape[0]
    if (u.dtype != z.dtype or u.stride(1) != 1 or u.shape[1] != z.shape[1] or (ids is None and u.shape[0] != M)
            or (ids is not None and (ids.dtype != torch.int64 or ids.numel() != M or not ids.is_contiguous()))):
        raise TimeViperHipError("gemv_glu: u rows of z's width, one per row or by int64 ids")
    y = torch.empty((M, N), dtype=z.dtype, device=z.device)
    check(_capi.lib().tv_gemv_glu_fwd(_p(z), _p(u), _p(ids), u.shape[0], _p(weight), _p(y), M, N, z.shape[1], z.stride(0), u.stride(0), weight.stride(0),
                                      N, _stream()), "tv_gemv_glu_fwd")
    return y


# ------------------------------------------------- mixture of experts
MOE_NONE, MOE_RELU2 = 0, 1


def moe_router(x, weight, correction, top):
    """softmax router: (ids (T, top) int32, weights (T, top) fp32) of the `top` outputs with the largest softmax + correction; the
    weights are the softmax values."""
    _gpu(x, weight, correction)
    T, D = x.shape
    E = weight.shape[0]
    if weight.shape[1] != D or not weight.is_contiguous() or x.stride(1) != 1:
        raise TimeViperHipError("moe_router: x (T, D), weight (outputs, D)")
    if correction is not None:
        _vec(correction, E, "moe_router correction")
        if correction.dtype != weight.dtype:
            raise TimeViperHipError("moe_router: correction of the weight's dtype")
    ids = torch.empty((T, top), dtype=torch.int32, device=x.device)
    w = torch.empty((T, top), dtype=torch.float32, device=x.device)
    check(_capi.lib().tv_moe_router_fwd(_p(x), _p(weight), _p(correction), _p(ids), _p(w), T, D, E, top, x.stride(0), _dt(x), _dt(weight),
                                        _stream()), "tv_moe_router_fwd")
    return ids, w


def moe_plan(ids, experts):
    """The choices (T, top) sorted by expert: (offsets (experts + 1), row_token (T * top), pos (T, top)) int32; pos -1: id >= experts
    (an identity expert, no row)."""
    _gpu(ids)
    T, top = ids.shape
    _i32(ids, T * top, "moe_plan ids")
    dev = ids.device
    counts = torch.empty(experts, dtype=torch.int32, device=dev)
    offsets = torch.empty(experts + 1, dtype=torch.int32, device=dev)
    row_token = torch.empty(T * top, dtype=torch.int32, device=dev)
    pos = torch.empty((T, top), dtype=torch.int32, device=dev)
    check(_capi.lib().tv_moe_plan(_p(ids), _p(counts), _p(offsets), _p(row_token), _p(pos), T * top, experts, top, _stream()), "tv_moe_plan")
    return offsets, row_token, pos


def moe_gemm(a, w, offsets, max_rows, row_token=None, act=MOE_NONE):
    """C (max_rows, N): rows [offsets[e], offsets[e + 1]) = act(a[row_token] @ w[e].T); w (experts, N, K)."""
    _gpu(a, w, offsets, row_token)
    E, N, Kd = w.shape
    _i32(offsets, E + 1, "moe_gemm offsets")
    _i32(row_token, max_rows, "moe_gemm row_token")
    if a.shape[1] != Kd or a.dtype != w.dtype or a.stride(1) != 1 or not w.is_contiguous() or (row_token is None and a.shape[0] < max_rows):
        raise TimeViperHipError(f"moe_gemm: a {tuple(a.shape)} against w {tuple(w.shape)}")
    c = torch.empty((max_rows, N), dtype=a.dtype, device=a.device)
    check(_capi.lib().tv_moe_gemm_fwd(_p(a), _p(w), _p(c), _p(offsets), _p(row_token), a.shape[0], max_rows, E, N, Kd, a.stride(0), c.stride(0), int(act),
                                      _dt(a), _stream()), "tv_moe_gemm_fwd")
    return c


def moe_decode_takes(tokens: int, n_out: int, top: int, width: int, ff: int, dtype) -> bool:
    """Shapes of tv_moe_decode_fwd."""
    return (dtype == torch.bfloat16 and tokens <= 4 and n_out <= 256 and top <= 32 and width % 8 == 0 and width <= 8192 and ff % 8 == 0
            and top * ff * 2 <= 128 * 1024)


def moe_decode(logits, correction, h, x, up, down, top):
    """Mixture of experts for a few single tokens: router logits (T, outputs) fp32, h (T, D) bf16 and the fp32 rows x it was rounded from,
    up (E, ff, D), down (E, D, ff).  Returns (sum of the chosen experts' outputs (T, D) bf16, ids (T, top) int32)."""
    _gpu(logits, correction, h, x, up, down)
    T, D = h.shape
    E, ff, _ = up.shape
    n_out = logits.shape[1]
    if (logits.shape != (T, n_out) or logits.dtype != torch.float32 or not logits.is_contiguous() or up.shape != (E, ff, D)
            or down.shape != (E, D, ff) or x.shape != h.shape or x.dtype != torch.float32 or any(t.dtype != torch.bfloat16 for t in (h, up, down, correction))
            or not all(t.is_contiguous() for t in (h, x, up, down))):
        raise TimeViperHipError("moe_decode: dense fp32 logits and x, dense bf16 h, up and down of matching sizes")
    _vec(correction, n_out, "moe_decode correction")
    dev = h.device
    ids = torch.empty((T, top), dtype=torch.int32, device=dev)
    wts = torch.empty((T, top), dtype=torch.float32, device=dev)
    u = torch.empty((T * top, ff), dtype=h.dtype, device=dev)
    y = torch.empty((T, D), dtype=h.dtype, device=dev)
    check(_capi.lib().tv_moe_decode_fwd(_p(logits), _p(correction), _p(h), _p(x), _p(up), _p(down), _p(ids), _p(wts), _p(u), _p(y), T, E, n_out, top,
                                        D, ff, _stream()), "tv_moe_decode_fwd")
    return y, ids
