// State-space duality (Mamba-2): per request and head h a state S [N][dv] in 32-bit, kept transposed in
// state[slot][h][j][i] (column j of S is contiguous).  For every token, in order,
//   dt = softplus(dt_pre + dt_bias_h);  S <- exp(A_h dt) S + dt B x^T;  y = S^T C + D_h x
// with A_h < 0; x a head's dv columns, B and C the N columns of the head's group (head h reads group h / (H / G)).  y
// stays 32-bit; a second kernel multiplies it by silu(z), divides it part by part by its root mean square and rounds it.
// xbc [n_tokens, stride]: x (H * dv columns) | B (G * N) | C (G * N), already convolved and activated; dt_pre: a column a
// head.  Step sizes, decays, sums, state and norm are 32-bit.
#include "recurrence.h"

namespace {

template <typename T>
struct SsdArgs {
  const T* xbc;
  int stride;
  const T* dt_pre;
  int dt_stride;
  const float* dt_bias;  // [H]
  const float* A;        // [H]
  const float* D;        // [H]
  float* state;
  long long state_stride;
  const int32_t* qo_indptr;
  const int32_t* slot_ids;
  float* y;  // [n_tokens, H * dv]
  int H, G, dv, N;
};

__device__ __forceinline__ float softplus_ssd(float z) { return z > 20.f ? z : log1pf(expf(z)); }

template <typename T>
__device__ __forceinline__ float step_size(const SsdArgs<T>& a, size_t t, int h) {
  return softplus_ssd(to_f32(a.dt_pre[t * a.dt_stride + h]) + a.dt_bias[h]);
}

// ----------------------------------------------------------------------------- token after token
// A block takes up to 128 columns of one (request, head), two a lane, and eight neighbouring lanes share a column: lane p
// of them holds rows 4 (p + 8 u) .. + 3 for u = 0 .. R / 4 - 1, so that the eight lanes read 128 bytes on end.  Tokens
// come in tiles of kWalkTile whose B (times the step size), C, x and decay lie in LDS; a tile's tokens follow each other
// without a barrier.  Every sum has an order fixed by the element (four chains a lane, then the eight lanes), whatever
// the tile: a token has the same bits in a prompt and in a decode step.  VEC: rows and state can be read four elements at
// a time.
constexpr int kWalkTile = 16;
constexpr int kWalkCols = 128;

template <typename T, bool VEC, int R>
__global__ void __launch_bounds__(512) ssd_walk_kernel(const SsdArgs<T> a, int cols, int col_groups) {
#pragma clang fp contract(off)
  constexpr int kPitch = 8 * R;  // a token's B in LDS, zeros behind N
  extern __shared__ __attribute__((aligned(16))) float lds[];
  float* b_l = lds;                              // [kWalkTile][kPitch]
  float* c_l = b_l + kWalkTile * kPitch;         // [kWalkTile][kPitch]
  float* x_l = c_l + kWalkTile * kPitch;         // [kWalkTile][cols]
  float* y_l = x_l + kWalkTile * cols;           // [kWalkTile][cols]
  float* dt_l = y_l + kWalkTile * cols;          // [kWalkTile] step sizes
  float* keep_l = dt_l + kWalkTile;              // [kWalkTile] decays
  const int row = blockIdx.y;
  const int h = blockIdx.x / col_groups, cg = blockIdx.x % col_groups;
  const int start = a.qo_indptr[row], end = a.qo_indptr[row + 1];
  const int n_threads = blockDim.x, tid = threadIdx.x;
  const int part = tid % 8, j_loc = 2 * (tid / 8);
  const int N = a.N, dv = a.dv;
  const int b_at = a.H * dv + h / (a.H / a.G) * N, c_at = b_at + a.G * N;
  float* st = a.state + (long long)a.slot_ids[row] * a.state_stride + (size_t)h * dv * N;
  const float A = a.A[h], D = a.D[h];
  float S[2][R];
#pragma unroll
  for (int c = 0; c < 2; ++c) {
    const int j = cg * cols + j_loc + c;
#pragma unroll
    for (int u = 0; u < R / 4; ++u) {
      const int i = 4 * (part + 8 * u);
      if (VEC) {  // (asked for whether it is there or not, so that nothing waits between the loads)
        const bool there = j < dv && i < N;
        const float4 s4 = *reinterpret_cast<const float4*>(st + (there ? (size_t)j * N + i : 0));
        S[c][4 * u] = there ? s4.x : 0.f; S[c][4 * u + 1] = there ? s4.y : 0.f;
        S[c][4 * u + 2] = there ? s4.z : 0.f; S[c][4 * u + 3] = there ? s4.w : 0.f;
      } else {
#pragma unroll
        for (int e = 0; e < 4; ++e) S[c][4 * u + e] = j < dv && i + e < N ? st[(size_t)j * N + i + e] : 0.f;
      }
    }
  }
  for (int t0 = start; t0 < end; t0 += kWalkTile) {
    const int nt = min(kWalkTile, end - t0);
    __syncthreads();  // the tile before has been read to its end
    if (tid < nt) {
      const float dt = step_size(a, (size_t)(t0 + tid), h);
      dt_l[tid] = dt;
      keep_l[tid] = expf(A * dt);
    }
    if (VEC) {
      for (int e = tid; e < nt * (kPitch / 2); e += n_threads) {  // four channels of a B, then of a C
        const int tt = e / (kPitch / 2), f = e % (kPitch / 2);
        const bool is_b = f < kPitch / 4;
        const int i = 4 * (is_b ? f : f - kPitch / 4);
        float v[4] = {0.f, 0.f, 0.f, 0.f};
        if (i < N) {
          const Four<T> raw = *reinterpret_cast<const Four<T>*>(a.xbc + (size_t)(t0 + tt) * a.stride + (is_b ? b_at : c_at) + i);
#pragma unroll
          for (int c = 0; c < 4; ++c) v[c] = to_f32(raw.e[c]);
        }
        *reinterpret_cast<float4*>((is_b ? b_l : c_l) + tt * kPitch + i) = float4{v[0], v[1], v[2], v[3]};
      }
    } else {
      for (int e = tid; e < nt * kPitch; e += n_threads) {
        const int tt = e / kPitch, i = e % kPitch;
        const T* tok = a.xbc + (size_t)(t0 + tt) * a.stride;
        b_l[e] = i < N ? to_f32(tok[b_at + i]) : 0.f;
        c_l[e] = i < N ? to_f32(tok[c_at + i]) : 0.f;
      }
    }
    for (int e = tid; e < nt * cols; e += n_threads) {
      const int tt = e / cols, j = cg * cols + e % cols;
      x_l[e] = j < dv ? to_f32(a.xbc[(size_t)(t0 + tt) * a.stride + h * dv + j]) : 0.f;
    }
    __syncthreads();
    struct Operands {
      float b[R], c[R], x[2], dt, keep;
    };
    auto read = [&](Operands& o, int tt_raw) {
      const int tt = tt_raw < kWalkTile ? tt_raw : kWalkTile - 1;
#pragma unroll
      for (int u = 0; u < R / 4; ++u) {
        const float4 b4 = *reinterpret_cast<const float4*>(b_l + tt * kPitch + 4 * (part + 8 * u));
        const float4 c4 = *reinterpret_cast<const float4*>(c_l + tt * kPitch + 4 * (part + 8 * u));
        o.b[4 * u] = b4.x; o.b[4 * u + 1] = b4.y; o.b[4 * u + 2] = b4.z; o.b[4 * u + 3] = b4.w;
        o.c[4 * u] = c4.x; o.c[4 * u + 1] = c4.y; o.c[4 * u + 2] = c4.z; o.c[4 * u + 3] = c4.w;
      }
      o.x[0] = x_l[tt * cols + j_loc];
      o.x[1] = x_l[tt * cols + j_loc + 1];
      o.dt = dt_l[tt];
      o.keep = keep_l[tt];
    };
    auto token = [&](const Operands& o, int tt) {
#pragma unroll
      for (int c = 0; c < 2; ++c) {
        const float dx = o.dt * o.x[c];
        float sum[4] = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int r = 0; r < R; ++r) {
          S[c][r] = fmaf(o.b[r], dx, o.keep * S[c][r]);
          sum[r % 4] = fmaf(S[c][r], o.c[r], sum[r % 4]);
        }
        const float y = sum_of_eight_lanes((sum[0] + sum[1]) + (sum[2] + sum[3]));
        if (part == 0) y_l[tt * cols + j_loc + c] = fmaf(D, o.x[c], y);
      }
    };
    Operands xa, xb;
    read(xa, 0);
#pragma unroll 1
    for (int tt = 0; tt < nt; tt += 2) {
      read(xb, tt + 1);
      token(xa, tt);
      if (tt + 1 < nt) {
        read(xa, tt + 2);
        token(xb, tt + 1);
      }
    }
    __syncthreads();
    for (int e = tid; e < nt * cols; e += n_threads) {
      const int tt = e / cols, j = cg * cols + e % cols;
      if (j < dv) a.y[((size_t)(t0 + tt) * a.H + h) * dv + j] = y_l[e];
    }
  }
#pragma unroll
  for (int c = 0; c < 2; ++c) {
    const int j = cg * cols + j_loc + c;
#pragma unroll
    for (int u = 0; u < R / 4; ++u) {
      const int i = 4 * (part + 8 * u);
      if (VEC) {
        if (j < dv && i < N) *reinterpret_cast<float4*>(st + (size_t)j * N + i) = float4{S[c][4 * u], S[c][4 * u + 1], S[c][4 * u + 2], S[c][4 * u + 3]};
      } else {
#pragma unroll
        for (int e = 0; e < 4; ++e)
          if (j < dv && i + e < N) st[(size_t)j * N + i + e] = S[c][4 * u + e];
      }
    }
  }
}

// Whether B, C and the state can be read four elements at a time.
template <typename T>
bool in_fours(const SsdArgs<T>& a) {
  return a.N % 4 == 0 && a.stride % 4 == 0 && (a.H * a.dv) % 4 == 0 && (uintptr_t)a.xbc % (4 * sizeof(T)) == 0 && (uintptr_t)a.state % 16 == 0 &&
         a.state_stride % 4 == 0;
}

template <typename T>
int launch_walk(const SsdArgs<T>& a, int n_seqs, hipStream_t stream) {
  const int cols = a.dv >= kWalkCols ? kWalkCols : (a.dv + 15) / 16 * 16;
  const int col_groups = (a.dv + cols - 1) / cols;
  const int threads = cols / 2 * 8;
  const int r = a.N <= 32 ? 4 : a.N <= 64 ? 8 : a.N <= 128 ? 16 : 32;
  const size_t lds = (size_t)kWalkTile * (2 * 8 * r + 2 * cols + 2) * sizeof(float);
  const dim3 grid(a.H * col_groups, n_seqs);
  const bool vec = in_fours(a);
#define TL_WALK(R)                                                                                   \
  do {                                                                                               \
    if (vec) ssd_walk_kernel<T, true, R><<<grid, threads, lds, stream>>>(a, cols, col_groups);       \
    else ssd_walk_kernel<T, false, R><<<grid, threads, lds, stream>>>(a, cols, col_groups);          \
  } while (0)
  if (r == 4) TL_WALK(4);
  else if (r == 8) TL_WALK(8);
  else if (r == 16) TL_WALK(16);
  else TL_WALK(32);
#undef TL_WALK
  return tl_check_launch("ssd_walk");
}

// ----------------------------------------------------------------------------- segments of a prompt side by side
// A row's tokens in segments of up to kSeg (bfloat16 rows).  With l_t the sum of A dt over the segment's tokens up to and
// with t, three launches compute, per (segment, head):
//   1. what the segment alone leaves, L = sum_t exp(l_last - l_t) dt_t B_t x_t^T, and exp(l_last);
//   2. the states that enter: S_0 = the request's state, S_(s+1) = exp(l_last) S_s + L_s, which takes L's place; the last
//      one becomes the request's state;
//   3. y_t = exp(l_t) S_in^T C_t + sum_(s <= t) exp(l_t - l_s) dt_s (C_t . B_s) x_s + D x_t.
// B_s . C_t is a bfloat16 product with 32-bit sums (both are bfloat16 as they come), formed as (B C^T)[s][t]: its results
// are, step for step, the other operand of the 32-bit product (P x)[t][j], so they stay in their registers.  Products with
// a state are 32-bit ones (16x16x4).
constexpr int kSeg = 64;
constexpr int kChunkThreads = 256;
typedef __bf16 bf16x8_t __attribute__((ext_vector_type(8)));

// Logarithms of the decays up to and with every token of the segment (l_l) and the step sizes (dt_l, zero behind the
// segment), by the first wave of the block: lane t has token t.
// `raw`: what dt_pre holds for the lane's token (`fetch_step`: asked for at the top, ahead of everything else).
__device__ __forceinline__ bf16_t fetch_step(const SsdArgs<bf16_t>& a, int first, int len, int h) {
  return a.dt_pre[(size_t)(first + min((int)threadIdx.x % kSeg, len - 1)) * a.dt_stride + h];
}
__device__ __forceinline__ void fill_decays(const SsdArgs<bf16_t>& a, bf16_t raw, int len, int h, float* l_l, float* dt_l) {
  const int t = threadIdx.x;
  if (t >= kSeg) return;
  const float dt = t < len ? softplus_ssd(to_f32(raw) + a.dt_bias[h]) : 0.f;
  float l = a.A[h] * dt;
#pragma unroll
  for (int off = 1; off < kSeg; off <<= 1) {
    const float before = __shfl_up(l, off, kWave);
    if (t >= off) l += before;
  }
  l_l[t] = l;  // (tokens behind the segment repeat the last one's)
  dt_l[t] = dt;
}

// NP, DVP: channels of the state and of a head rounded up to 64 or 128 (what lies beyond is zero).
template <int NP, int DVP>
__global__ void __launch_bounds__(kChunkThreads)
ssd_local_kernel(const SsdArgs<bf16_t> a, const int32_t* __restrict__ segs, float* __restrict__ ws, float* __restrict__ seg_keep) {
  constexpr int PB = NP + 4, PV = DVP + 4;
  extern __shared__ __attribute__((aligned(16))) float lds[];
  float* b_l = lds;                // [kSeg][PB]: B times exp(l_last - l_t) dt_t
  float* v_l = b_l + kSeg * PB;    // [kSeg][PV]
  float* l_l = v_l + kSeg * PV;    // [kSeg]
  float* dt_l = l_l + kSeg;        // [kSeg]
  const int seg = blockIdx.x, h = blockIdx.y;
  const int first = segs[2 * seg], len = segs[2 * seg + 1] - first;
  const int N = a.N, dv = a.dv;
  const int b_at = a.H * dv + h / (a.H / a.G) * N;
  const bf16_t step = fetch_step(a, first, len, h);
  // rows of B and x are on their way while the decays are formed
  constexpr int BL = kSeg * (NP / 4) / kChunkThreads, VL = kSeg * (DVP / 4) / kChunkThreads;
  Four<bf16_t> braw[BL], vraw[VL];
#pragma unroll
  for (int u = 0; u < BL; ++u) {
    const int e = threadIdx.x + u * kChunkThreads, t = e / (NP / 4), i = 4 * (e % (NP / 4));
    const bool there = t < len && i < N;
    braw[u] = *reinterpret_cast<const Four<bf16_t>*>(a.xbc + (size_t)(first + (there ? t : 0)) * a.stride + b_at + (there ? i : 0));
    if (!there) braw[u] = Four<bf16_t>{};
  }
#pragma unroll
  for (int u = 0; u < VL; ++u) {
    const int e = threadIdx.x + u * kChunkThreads, t = e / (DVP / 4), j = 4 * (e % (DVP / 4));
    const bool there = t < len && j < dv;
    vraw[u] = *reinterpret_cast<const Four<bf16_t>*>(a.xbc + (size_t)(first + (there ? t : 0)) * a.stride + h * dv + (there ? j : 0));
    if (!there) vraw[u] = Four<bf16_t>{};
  }
  fill_decays(a, step, len, h, l_l, dt_l);
  __syncthreads();
  const float l_last = l_l[kSeg - 1];
  if (threadIdx.x == 0) seg_keep[(size_t)seg * a.H + h] = expf(l_last);
#pragma unroll
  for (int u = 0; u < BL; ++u) {
    const int e = threadIdx.x + u * kChunkThreads, t = e / (NP / 4), i = 4 * (e % (NP / 4));
    const float w = expf(l_last - l_l[t]) * dt_l[t];
    *reinterpret_cast<float4*>(b_l + t * PB + i) =
        float4{to_f32(braw[u].e[0]) * w, to_f32(braw[u].e[1]) * w, to_f32(braw[u].e[2]) * w, to_f32(braw[u].e[3]) * w};
  }
#pragma unroll
  for (int u = 0; u < VL; ++u) {
    const int e = threadIdx.x + u * kChunkThreads, t = e / (DVP / 4), j = 4 * (e % (DVP / 4));
    *reinterpret_cast<float4*>(v_l + t * PV + j) = float4{to_f32(vraw[u].e[0]), to_f32(vraw[u].e[1]), to_f32(vraw[u].e[2]), to_f32(vraw[u].e[3])};
  }
  __syncthreads();
  constexpr int MT = DVP / 16 / 4, NT = NP / 16;  // tiles of 16 columns j a wave takes, tiles of 16 rows i
  const int wave = threadIdx.x / kWave, lane = threadIdx.x % kWave, n16 = lane % 16, g4 = lane / 16;
  f32x4_t acc[MT][NT];
#pragma unroll
  for (int m = 0; m < MT; ++m)
#pragma unroll
    for (int n = 0; n < NT; ++n) acc[m][n] = f32x4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll 4
  for (int t = 0; t < kSeg; t += 4) {
    float va[MT], kb[NT];
#pragma unroll
    for (int m = 0; m < MT; ++m) va[m] = v_l[(t + g4) * PV + 16 * (wave * MT + m) + n16];
#pragma unroll
    for (int n = 0; n < NT; ++n) kb[n] = b_l[(t + g4) * PB + 16 * n + n16];
#pragma unroll
    for (int m = 0; m < MT; ++m)
#pragma unroll
      for (int n = 0; n < NT; ++n) acc[m][n] = mfma_f32(va[m], kb[n], acc[m][n]);
  }
  float* dst = ws + ((size_t)seg * a.H + h) * dv * N;
#pragma unroll
  for (int m = 0; m < MT; ++m)
#pragma unroll
    for (int n = 0; n < NT; ++n)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int j = 16 * (wave * MT + m) + 4 * g4 + r, i = 16 * n + n16;
        if (j < dv && i < N) dst[(size_t)j * N + i] = acc[m][n][r];
      }
}

// A thread takes four elements of a row's state through the row's segments; their L are asked for eight ahead.
constexpr int kCarryAhead = 8;
__global__ void __launch_bounds__(256) ssd_carry_kernel(const SsdArgs<bf16_t> a, const int32_t* __restrict__ row_seg, float* __restrict__ ws,
                                                        const float* __restrict__ seg_keep) {
  const size_t per_seg = (size_t)a.H * a.dv * a.N;
  const size_t e = 4 * ((size_t)blockIdx.x * 256 + threadIdx.x);
  if (e >= per_seg) return;
  const int row = blockIdx.y;
  const int h = (int)(e / ((size_t)a.dv * a.N));
  const int s0 = row_seg[row], s1 = row_seg[row + 1];
  float4* st = reinterpret_cast<float4*>(a.state + (long long)a.slot_ids[row] * a.state_stride + e);
  float4 S = *st;
  for (int s = s0; s < s1; s += kCarryAhead) {
    float4 L[kCarryAhead];
    float f[kCarryAhead];
#pragma unroll
    for (int u = 0; u < kCarryAhead; ++u) {
      const int at = s + u < s1 ? s + u : s1 - 1;
      L[u] = *reinterpret_cast<const float4*>(ws + at * per_seg + e);
      f[u] = seg_keep[(size_t)at * a.H + h];
    }
#pragma unroll
    for (int u = 0; u < kCarryAhead; ++u) {
      if (s + u >= s1) break;
      *reinterpret_cast<float4*>(ws + (size_t)(s + u) * per_seg + e) = S;
      S = float4{fmaf(f[u], S.x, L[u].x), fmaf(f[u], S.y, L[u].y), fmaf(f[u], S.z, L[u].z), fmaf(f[u], S.w, L[u].w)};
    }
  }
  *st = S;
}

// A wave takes 16 * MT of the head's columns for all tokens of the segment, so that the state that entered is read once and
// every wave has the same products to do; the weighted scores are formed once, sixteen tokens a wave, and go through LDS.
template <int NP, int DVP>
__global__ void __launch_bounds__(kChunkThreads)
ssd_read_kernel(const SsdArgs<bf16_t> a, const int32_t* __restrict__ segs, const float* __restrict__ ws) {
  constexpr int PV = DVP + 4, PS = kSeg + 4;
  constexpr int NK = NP / 32, MT = DVP / 64, NS = kSeg / 16;
  extern __shared__ __attribute__((aligned(16))) float lds[];
  float* x_l = lds;               // [kSeg][PV]
  float* p_l = x_l + kSeg * PV;   // [kSeg tokens t][PS]: what token s <= t counts, for the sixteens up to t's own
  float* l_l = p_l + kSeg * PS;   // [kSeg]
  float* dt_l = l_l + kSeg;       // [kSeg]
  const int seg = blockIdx.x, h = blockIdx.y;
  const int first = segs[2 * seg], len = segs[2 * seg + 1] - first;
  const int N = a.N, dv = a.dv;
  const int b_at = a.H * dv + h / (a.H / a.G) * N, c_at = b_at + a.G * N;
  const int wave = threadIdx.x / kWave, lane = threadIdx.x % kWave, n16 = lane % 16, g4 = lane / 16;
  const bf16_t step = fetch_step(a, first, len, h);
  bf16x8_t zero;
#pragma unroll
  for (int i = 0; i < 8; ++i) zero[i] = (__bf16)0.0f;
  // eight channels 32 u + 8 g4 .. + 7 of a token's B or C (zeros behind the segment and behind N)
  auto piece = [&](int at, int t, int u) {
    const int i = 32 * u + 8 * g4;
    const bool there = t < len && i < N;
    const bf16x8_t v = *reinterpret_cast<const bf16x8_t*>(a.xbc + (size_t)(first + (there ? t : 0)) * a.stride + at + (there ? i : 0));
    return there ? v : zero;
  };
  // this wave's sixteen tokens: lane (n16, g4) has the C of token 16 wave + n16
  const int tq = 16 * wave + n16;
  bf16x8_t q[NK];
#pragma unroll
  for (int u = 0; u < NK; ++u) q[u] = piece(c_at, tq, u);
  constexpr int VL = kSeg * (DVP / 4) / kChunkThreads;
#pragma unroll
  for (int u = 0; u < VL; ++u) {
    const int e = threadIdx.x + u * kChunkThreads, t = e / (DVP / 4), j = 4 * (e % (DVP / 4));
    const bool there = t < len && j < dv;
    const Four<bf16_t> v = *reinterpret_cast<const Four<bf16_t>*>(a.xbc + (size_t)(first + (there ? t : 0)) * a.stride + h * dv + (there ? j : 0));
    *reinterpret_cast<float4*>(x_l + t * PV + j) =
        there ? float4{to_f32(v.e[0]), to_f32(v.e[1]), to_f32(v.e[2]), to_f32(v.e[3])} : float4{0.f, 0.f, 0.f, 0.f};
  }
  fill_decays(a, step, len, h, l_l, dt_l);
  // the state that entered: lane (n16, g4) has channels 32 u + 8 g4 .. + 7 of columns 16 (wave MT + m) + n16
  const float* S_in = ws + ((size_t)seg * a.H + h) * dv * N;
  float4 st[MT][NK][2];
#pragma unroll
  for (int m = 0; m < MT; ++m) {
    const int j = 16 * (wave * MT + m) + n16;
#pragma unroll
    for (int u = 0; u < NK; ++u) {
      const int i = 32 * u + 8 * g4;
      const bool there = j < dv && i < N;
      const float4* src = reinterpret_cast<const float4*>(S_in + (there ? (size_t)j * N + i : 0));
      st[m][u][0] = src[0];
      st[m][u][1] = src[1];
      if (!there) st[m][u][0] = st[m][u][1] = float4{0.f, 0.f, 0.f, 0.f};
    }
  }
  __syncthreads();  // x and the decays are in LDS
  // (B C^T)[s][t] of the wave's sixteen tokens with every sixteen up to their own (results: rows s, column t), weighted
  {
    const float l_q = l_l[tq];
#pragma unroll
    for (int b = 0; b < NS; ++b) {
      if (b > wave) continue;  // (the same for the whole wave)
      f32x4_t p = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int u = 0; u < NK; ++u) p = __builtin_amdgcn_mfma_f32_16x16x32_bf16(piece(b_at, 16 * b + n16, u), q[u], p, 0, 0, 0);
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int s = 16 * b + 4 * g4 + r;
        p[r] = s <= tq ? p[r] * (expf(fminf(l_q - l_l[s], 0.f)) * dt_l[s]) : 0.f;
      }
      *reinterpret_cast<float4*>(p_l + tq * PS + 16 * b + 4 * g4) = float4{p[0], p[1], p[2], p[3]};
    }
  }
  // acc[tb][m] = rows t = 16 tb + 4 g4 + i, columns 16 (wave MT + m) + n16: first what the state that entered gives
  f32x4_t acc[NS][MT];
#pragma unroll
  for (int tb = 0; tb < NS; ++tb) {
    bf16x8_t c[NK];
#pragma unroll
    for (int u = 0; u < NK; ++u) c[u] = piece(c_at, 16 * tb + n16, u);
#pragma unroll
    for (int m = 0; m < MT; ++m) acc[tb][m] = f32x4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int u = 0; u < NK; ++u)
#pragma unroll
      for (int m = 0; m < MT; ++m) {
        const float sv[8] = {st[m][u][0].x, st[m][u][0].y, st[m][u][0].z, st[m][u][0].w, st[m][u][1].x, st[m][u][1].y, st[m][u][1].z, st[m][u][1].w};
#pragma unroll
        for (int e = 0; e < 8; ++e) acc[tb][m] = mfma_f32((float)c[u][e], sv[e], acc[tb][m]);
      }
  }
  const float D = a.D[h];
#pragma unroll
  for (int tb = 0; tb < NS; ++tb)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int t = 16 * tb + 4 * g4 + r;
      const float f = expf(l_l[t]);
#pragma unroll
      for (int m = 0; m < MT; ++m) acc[tb][m][r] = fmaf(D, x_l[t * PV + 16 * (wave * MT + m) + n16], acc[tb][m][r] * f);
    }
  __syncthreads();  // the scores are in LDS
#pragma unroll
  for (int b = 0; b < NS; ++b)
#pragma unroll
    for (int r = 0; r < 4; ++r)
#pragma unroll
      for (int m = 0; m < MT; ++m) {
        const float xv = x_l[(16 * b + 4 * g4 + r) * PV + 16 * (wave * MT + m) + n16];
#pragma unroll
        for (int tb = b; tb < NS; ++tb) acc[tb][m] = mfma_f32(p_l[(16 * tb + n16) * PS + 16 * b + 4 * g4 + r], xv, acc[tb][m]);
      }
#pragma unroll
  for (int tb = 0; tb < NS; ++tb)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int t = 16 * tb + 4 * g4 + r;
#pragma unroll
      for (int m = 0; m < MT; ++m) {
        const int j = 16 * (wave * MT + m) + n16;
        if (t < len && j < dv) a.y[((size_t)(first + t) * a.H + h) * dv + j] = acc[tb][m][r];
      }
    }
}

template <int NP, int DVP>
int launch_chunks(const SsdArgs<bf16_t>& a, int n_rows, int n_segs, const int32_t* segs, const int32_t* row_seg, float* ws, float* seg_keep,
                  hipStream_t stream) {
  constexpr int PB = NP + 4, PV = DVP + 4;
  const size_t lds_local = ((size_t)kSeg * (PB + PV) + 2 * kSeg) * sizeof(float);
  const size_t lds_read = ((size_t)kSeg * (PV + kSeg + 4) + 2 * kSeg) * sizeof(float);
  if (lds_local > 48 * 1024) {
    hipError_t e = hipFuncSetAttribute((const void*)ssd_local_kernel<NP, DVP>, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds_local);
    if (e != hipSuccess) return tl_fail(TL_ERR_HIP, "ssd: %s", hipGetErrorString(e));
  }
  if (lds_read > 48 * 1024) {
    hipError_t e = hipFuncSetAttribute((const void*)ssd_read_kernel<NP, DVP>, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds_read);
    if (e != hipSuccess) return tl_fail(TL_ERR_HIP, "ssd: %s", hipGetErrorString(e));
  }
  const dim3 grid(n_segs, a.H);
  ssd_local_kernel<NP, DVP><<<grid, kChunkThreads, lds_local, stream>>>(a, segs, ws, seg_keep);
  int rc = tl_check_launch("ssd_local");
  if (rc != TL_OK) return rc;
  const size_t fours = (size_t)a.H * a.dv * a.N / 4;
  ssd_carry_kernel<<<dim3((unsigned)((fours + 255) / 256), n_rows), 256, 0, stream>>>(a, row_seg, ws, seg_keep);
  rc = tl_check_launch("ssd_carry");
  if (rc != TL_OK) return rc;
  ssd_read_kernel<NP, DVP><<<grid, kChunkThreads, lds_read, stream>>>(a, segs, ws);
  return tl_check_launch("ssd_read");
}

// ----------------------------------------------------------------------------- the gate and the norm by parts
// out[t, part] = T(g / sqrt(mean(g^2) + eps) * w) with g = y[t, part] * silu(z[t, part]), a part being `width` neighbouring
// columns.  A block a (token, part); g stays in registers (CH pieces of V elements a thread) or, of wider parts, is formed
// twice.  A part's sum has an order that its width alone decides.
constexpr int kNormThreads = 256;
__device__ __forceinline__ float gated(float y, float z) { return y * (z / (1.0f + expf(-z))); }

template <typename T, int V, int CH>
__global__ void __launch_bounds__(kNormThreads)
gated_norm_kernel(const float* __restrict__ y, const T* __restrict__ z, int z_stride, const float* __restrict__ w, T* __restrict__ out,
                  int parts, int width, float eps) {
#pragma clang fp contract(off)
  __shared__ float scratch[kNormThreads / kWave];
  struct alignas(V * sizeof(T)) ZVec { T e[V]; };
  struct alignas(V * sizeof(float)) YVec { float e[V]; };
  const size_t t = blockIdx.x;
  const int part = blockIdx.y;
  const float* yr = y + (t * parts + part) * width;
  const T* zr = z + t * z_stride + (size_t)part * width;
  const float* wr = w + (size_t)part * width;
  T* o = out + (t * parts + part) * width;
  YVec yv[CH], wv[CH];
  ZVec zv[CH];
#pragma unroll
  for (int c = 0; c < CH; ++c) {
    const int i = V * ((int)threadIdx.x + c * kNormThreads), at = i < width ? i : 0;  // (past the end: the first once more, not used)
    yv[c] = *reinterpret_cast<const YVec*>(yr + at);
    zv[c] = *reinterpret_cast<const ZVec*>(zr + at);
    wv[c] = *reinterpret_cast<const YVec*>(wr + at);
  }
  float ss = 0.f;
#pragma unroll
  for (int c = 0; c < CH; ++c)
#pragma unroll
    for (int e = 0; e < V; ++e) {
      const bool in = V * ((int)threadIdx.x + c * kNormThreads) < width;
      yv[c].e[e] = in ? gated(yv[c].e[e], to_f32(zv[c].e[e])) : 0.f;
      ss += yv[c].e[e] * yv[c].e[e];
    }
  for (int i = V * ((int)threadIdx.x + CH * kNormThreads); i < width; i += V * kNormThreads)
    for (int e = 0; e < V; ++e) {
      const float g = gated(yr[i + e], to_f32(zr[i + e]));
      ss += g * g;
    }
  ss = block_sum<kNormThreads / kWave>(ss, scratch);
  const float inv = 1.0f / sqrtf(ss / (float)width + eps);
#pragma unroll
  for (int c = 0; c < CH; ++c) {
    const int i = V * ((int)threadIdx.x + c * kNormThreads);
    if (i >= width) continue;
    ZVec r;
#pragma unroll
    for (int e = 0; e < V; ++e) r.e[e] = from_f32<T>(yv[c].e[e] * inv * wv[c].e[e]);
    *reinterpret_cast<ZVec*>(o + i) = r;
  }
  for (int i = V * ((int)threadIdx.x + CH * kNormThreads); i < width; i += V * kNormThreads)
    for (int e = 0; e < V; ++e) o[i + e] = from_f32<T>(gated(yr[i + e], to_f32(zr[i + e])) * inv * wr[i + e]);
}

template <typename T>
int launch_gated_norm(const float* y, const T* z, int z_stride, const float* w, T* out, int n, int parts, int width, float eps, hipStream_t stream) {
  const bool fours = width % 4 == 0 && z_stride % 4 == 0 && (uintptr_t)y % 16 == 0 && (uintptr_t)w % 16 == 0 && (uintptr_t)z % (4 * sizeof(T)) == 0 &&
                     (uintptr_t)out % (4 * sizeof(T)) == 0;
  const dim3 grid(n, parts);
#define TL_NORM(V, CH) gated_norm_kernel<T, V, CH><<<grid, kNormThreads, 0, stream>>>(y, z, z_stride, w, out, parts, width, eps)
  if (!fours) TL_NORM(1, 8);
  else if (width <= 4 * kNormThreads) TL_NORM(4, 1);
  else if (width <= 16 * kNormThreads) TL_NORM(4, 4);
  else TL_NORM(4, 8);
#undef TL_NORM
  return tl_check_launch("gated_norm");
}

template <typename T>
SsdArgs<T> ssd_args(const void* xbc, int stride, const void* dt_pre, int dt_stride, const float* dt_bias, const float* A, const float* D,
                    float* state, long long state_stride, const int32_t* qo_indptr, const int32_t* slot_ids, float* y, int H, int G, int dv, int N) {
  return {(const T*)xbc, stride, (const T*)dt_pre, dt_stride, dt_bias, A, D, state, state_stride, qo_indptr, slot_ids, y, H, G, dv, N};
}

}  // namespace

// The most tokens of a segment of tl_ssd_chunks, and the most channels of a state and of a head that it takes.
TL_EXPORT int tl_ssd_segment() { return kSeg; }
TL_EXPORT int tl_ssd_chunk_channels() { return 128; }

// The recurrence over each request's tokens, token after token (see the head of this file).  Row r of the step holds
// tokens qo_indptr[r] .. qo_indptr[r + 1] - 1 of the request in slot slot_ids[r].
TL_EXPORT int tl_ssd(const void* xbc, int stride, const void* dt_pre, int dt_stride, const float* dt_bias, const float* A, const float* D,
                     float* state, long long state_stride, const int32_t* qo_indptr, const int32_t* slot_ids, float* y, int n_seqs, int H,
                     int G, int dv, int N, int dtype, hipStream_t stream) {
  TL_REQUIRE(n_seqs >= 0 && H > 0 && G > 0 && H % G == 0 && dv > 0 && N > 0, "ssd: bad sizes");
  TL_REQUIRE(stride >= H * dv + 2 * G * N && dt_stride >= H, "ssd: rows that do not hold x, B and C, or the step sizes");
  if (N > 256) return tl_fail(TL_ERR_UNSUPPORTED, "ssd: states of %d channels, at most 256", N);
  TL_REQUIRE(n_seqs <= 65535, "ssd: too many requests a step");
  if (n_seqs == 0) return TL_OK;
  if (dtype == TL_F32)
    return launch_walk(ssd_args<float>(xbc, stride, dt_pre, dt_stride, dt_bias, A, D, state, state_stride, qo_indptr, slot_ids, y, H, G, dv, N), n_seqs, stream);
  if (dtype == TL_BF16)
    return launch_walk(ssd_args<bf16_t>(xbc, stride, dt_pre, dt_stride, dt_bias, A, D, state, state_stride, qo_indptr, slot_ids, y, H, G, dv, N), n_seqs, stream);
  return tl_fail(TL_ERR_ARG, "ssd: unknown dtype %d", dtype);
}

// The recurrence of bfloat16 prompts by segments (see above).  segs: [n_segs][2] first token and one past the last of
// every segment (at most tl_ssd_segment() tokens), every row's in order; row_seg [n_rows + 1]: the first segment of every
// row; slot_ids [n_rows].  Tokens are rows of xbc, dt_pre and y.  ws: n_segs * H * dv * N floats, seg_keep: n_segs * H.
// N a multiple of 8 and dv one of 4, both up to tl_ssd_chunk_channels(); rows aligned so that eight elements can be read
// at a time.
TL_EXPORT int tl_ssd_chunks(const void* xbc, int stride, const void* dt_pre, int dt_stride, const float* dt_bias, const float* A, const float* D,
                            float* state, long long state_stride, const int32_t* slot_ids, float* y, int n_rows, int H, int G, int dv, int N,
                            const int32_t* segs, const int32_t* row_seg, int n_segs, float* ws, float* seg_keep, int dtype, hipStream_t stream) {
  TL_REQUIRE(n_rows >= 0 && n_segs >= 0 && H > 0 && G > 0 && H % G == 0 && dv > 0 && N > 0, "ssd: bad sizes");
  TL_REQUIRE(stride >= H * dv + 2 * G * N && dt_stride >= H, "ssd: rows that do not hold x, B and C, or the step sizes");
  if (dtype != TL_BF16) return tl_fail(TL_ERR_UNSUPPORTED, "ssd: segments are for bfloat16 models");
  if (N > 128 || dv > 128) return tl_fail(TL_ERR_UNSUPPORTED, "ssd: segments take states and heads of up to 128 channels, got %d and %d", N, dv);
  TL_REQUIRE(n_rows <= 65535 && H <= 65535, "ssd: too many requests or heads a step");
  if (n_rows == 0 || n_segs == 0) return TL_OK;
  TL_REQUIRE(segs && row_seg && ws && seg_keep && slot_ids, "ssd: no segments or no workspace");
  const SsdArgs<bf16_t> a = ssd_args<bf16_t>(xbc, stride, dt_pre, dt_stride, dt_bias, A, D, state, state_stride, nullptr, slot_ids, y, H, G, dv, N);
  TL_REQUIRE(in_fours(a) && N % 8 == 0 && dv % 4 == 0 && (H * dv) % 8 == 0 && stride % 8 == 0 && (uintptr_t)xbc % 16 == 0 && (uintptr_t)ws % 16 == 0 &&
                 (uintptr_t)y % 16 == 0,
             "ssd: rows that cannot be read eight elements at a time");
  if (N <= 64 && dv <= 64) return launch_chunks<64, 64>(a, n_rows, n_segs, segs, row_seg, ws, seg_keep, stream);
  if (N <= 64) return launch_chunks<64, 128>(a, n_rows, n_segs, segs, row_seg, ws, seg_keep, stream);
  if (dv <= 64) return launch_chunks<128, 64>(a, n_rows, n_segs, segs, row_seg, ws, seg_keep, stream);
  return launch_chunks<128, 128>(a, n_rows, n_segs, segs, row_seg, ws, seg_keep, stream);
}

// out [n, parts * width]: y (32-bit) times silu(z), each of the `parts` equal parts over its own root mean square, times w.
TL_EXPORT int tl_gated_norm(const float* y, const void* z, int z_stride, const float* w, void* out, int n, int parts, int width, float eps,
                            int dtype, hipStream_t stream) {
  TL_REQUIRE(n >= 0 && parts > 0 && parts <= 65535 && width > 0 && z_stride >= parts * width, "gated_norm: bad sizes");
  if (n == 0) return TL_OK;
  if (dtype == TL_F32) return launch_gated_norm<float>(y, (const float*)z, z_stride, w, (float*)out, n, parts, width, eps, stream);
  if (dtype == TL_BF16) return launch_gated_norm<bf16_t>(y, (const bf16_t*)z, z_stride, w, (bf16_t*)out, n, parts, width, eps, stream);
  return tl_fail(TL_ERR_ARG, "gated_norm: unknown dtype %d", dtype);
}
