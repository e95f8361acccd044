"""State-space duality (Mamba-2): the recurrence over matrix states with one decay a head, and the gated norm by parts
behind it."""

from __future__ import annotations

from typing import Optional

import torch

from .base import KernelError, _gpu, _stream, check, core, dtype_code
from .sequence_ops import ScanSegments, _step_rows, state_region

#: the most channels of a state that the kernels take (a head's own channels: any number)
SSD_MAX_STATE = 256
#: tokens of a segment when a prompt's segments run side by side, the longest row of a step from which on they do, and
#: the most channels of a state and of a head for which they do
SSD_SEGMENT = 64
SSD_SEGMENTS_FROM = 32
SSD_SEGMENT_CHANNELS = 128


def ssd_segments_supported(dtype: torch.dtype, n_heads: int, v_head_dim: int, state_size: int, n_groups: int) -> bool:
    """Whether ``ssd`` takes segments for these sizes (bfloat16 models: in 32-bit every row is walked in one piece, so
    that no bit depends on how a prompt was cut into steps)."""
    return (dtype == torch.bfloat16 and state_size % 8 == 0 and v_head_dim % 4 == 0 and (n_heads * v_head_dim) % 8 == 0
            and max(state_size, v_head_dim) <= SSD_SEGMENT_CHANNELS)


def ssd(
    xbc: torch.Tensor,
    dt_pre: torch.Tensor,
    dt_bias: torch.Tensor,
    A: torch.Tensor,
    D: torch.Tensor,
    state: torch.Tensor,
    state_offset: int,
    qo_indptr: torch.Tensor,
    slot_ids: torch.Tensor,
    n_groups: int,
    v_head_dim: int,
    state_size: int,
    segments: Optional[ScanSegments] = None,
    single_rows: int = 0,
) -> torch.Tensor:
    """The recurrence over each request's tokens, in 32-bit.  ``xbc`` [n, H dv + 2 G N] (x | B | C, convolved and
    activated), ``dt_pre`` [n, H] (some columns of a wider matrix will do); ``dt_bias``, ``A`` (negative) and ``D`` float32
    [H].  Per head h, which reads B and C of group ``h // (H / G)``: ``dt = softplus(dt_pre + dt_bias); S <- exp(A dt) S +
    dt B x^T; y = S^T C + D x``.  ``S`` lives at ``state_offset`` of the request's state row, H * dv * N floats.  Returns
    float32 [n, H * dv].

    With ``segments`` (of at most ``SSD_SEGMENT`` tokens, bfloat16; see ``ssd_segments_supported``) the first
    ``single_rows`` rows of the step, one token each, are walked, and of the others the segments run side by side on the
    matrix cores: what a segment leaves by itself, the states that enter the segments, the results."""
    _gpu(xbc, dt_pre, dt_bias, A, D)
    H, G, dv, N = A.numel(), n_groups, v_head_dim, state_size
    n = xbc.shape[0]
    if xbc.dim() != 2 or xbc.stride(1) != 1 or G <= 0 or H % G or xbc.shape[1] != H * dv + 2 * G * N:
        raise KernelError(f"ssd: xbc must be [n, {H * dv + 2 * G * N}] with contiguous rows, the heads a multiple of the groups")
    if tuple(dt_pre.shape) != (n, H) or dt_pre.stride(1) != 1 or dt_pre.dtype != xbc.dtype:
        raise KernelError(f"ssd: dt_pre must be [n, {H}] of xbc's dtype with contiguous rows")
    for v in (dt_bias, A, D):
        if tuple(v.shape) != (H,) or v.dtype != torch.float32 or not v.is_contiguous():
            raise KernelError(f"ssd: dt_bias, A and D must be float32 vectors of {H} entries")
    n_seqs = _step_rows(None, qo_indptr, slot_ids, n, state)
    region, stride = state_region(state, state_offset, H * dv * N)
    y = torch.empty((n, H * dv), dtype=torch.float32, device=xbc.device)
    dt_stride = dt_pre.stride(0) if n > 1 else max(dt_pre.stride(0), H)
    shared = (xbc.data_ptr(), xbc.stride(0), dt_pre.data_ptr(), dt_stride, dt_bias.data_ptr(), A.data_ptr(), D.data_ptr(), region, stride)

    def walk(rows: int) -> None:
        check(core().tl_ssd(*shared, qo_indptr.data_ptr(), slot_ids.data_ptr(), y.data_ptr(), rows, H, G, dv, N, dtype_code(xbc.dtype), _stream()))

    if segments is None:
        walk(n_seqs)
        return y
    if not ssd_segments_supported(xbc.dtype, H, dv, N, G) or segments.length > SSD_SEGMENT:
        raise KernelError(f"ssd: segments are not for {xbc.dtype} with heads of {dv} and states of {N} channels, or too long")
    n_rows = n_seqs - single_rows
    if not 0 <= single_rows <= n_seqs or segments.row_seg.numel() != n_rows + 1:
        raise KernelError("ssd: the segments are not those of this step's rows")
    if single_rows:
        walk(single_rows)
    ws = torch.empty((segments.n, H * dv * N), dtype=torch.float32, device=xbc.device)
    keep = torch.empty((segments.n, H), dtype=torch.float32, device=xbc.device)
    slots = slot_ids[single_rows:]
    check(core().tl_ssd_chunks(*shared, slots.data_ptr(), y.data_ptr(), n_rows, H, G, dv, N, segments.segs.data_ptr(), segments.row_seg.data_ptr(),
                               segments.n, ws.data_ptr(), keep.data_ptr(), dtype_code(xbc.dtype), _stream()))
    return y


def gated_norm(y: torch.Tensor, z: torch.Tensor, weight: torch.Tensor, parts: int, eps: float) -> torch.Tensor:
    """``g = y * silu(z)``; each of the ``parts`` equal parts of a row of g over its own root mean square, times ``weight``:
    ``y`` float32 [n, width], ``z`` [n, width] (some columns of a wider matrix will do), ``weight`` float32 [width].
    Returns [n, width] of z's dtype, rounded once."""
    _gpu(y, z, weight)
    if y.dim() != 2 or y.dtype != torch.float32 or not y.is_contiguous():
        raise KernelError("gated_norm: y must be a contiguous float32 matrix")
    n, width = y.shape
    if tuple(z.shape) != (n, width) or z.stride(1) != 1:
        raise KernelError("gated_norm: z must have y's shape and contiguous rows")
    if tuple(weight.shape) != (width,) or weight.dtype != torch.float32 or not weight.is_contiguous():
        raise KernelError(f"gated_norm: weight must be a float32 vector of {width} entries")
    if parts <= 0 or width % parts:
        raise KernelError(f"gated_norm: {width} columns do not fall into {parts} parts")
    out = torch.empty((n, width), dtype=z.dtype, device=z.device)
    check(core().tl_gated_norm(y.data_ptr(), z.data_ptr(), z.stride(0) if n > 1 else max(z.stride(0), width), weight.data_ptr(), out.data_ptr(), n,
                               parts, width // parts, float(eps), dtype_code(z.dtype), _stream()))
    return out
