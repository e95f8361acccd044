// Retention: linear attention whose state fades by a constant per head.  Per request and head h, state S [dk][dv] in
// 32-bit, kept transposed in state[slot][h][j][i] (column j of S is contiguous).  For every token, in order, with q and
// k rotated by the token's position and k times dk^-1/2:
//   S <- decay_h S + k v^T;  o = S^T q;  out[t, h, :] = T(o / sqrt(mean(o^2) + eps) * silu(gate[t, h, :]))
// proj: the layer's fused projection [n_tokens, stride], of which the columns of q, k (H * dk each), v and the gate
// (H * dv each) are read from their offsets.  cos_sin: the step's table [n_tokens][rot / 2][2] (channel i of a head is
// paired with channel i + rot / 2; channels from rot on pass).  Rotated keys and queries, decays, sums, state and norm
// are 32-bit.
#include "recurrence.h"

namespace {

template <typename T>
struct RetentionArgs {
  const T* proj;
  int stride, q_off, k_off, v_off, g_off;
  const float* cos_sin;
  int rot;
  const float* decay;  // [H]
  float* state;
  long long state_stride;
  const int32_t* qo_indptr;
  const int32_t* slot_ids;
  T* out;        // [n_tokens, H * dv]
  float* o_raw;  // [n_tokens, H, dv], where a head's columns are spread over several blocks
  int H, dk, dv;
  float eps, k_scale;
};

// Element i of a head after the rotation, from the head's row in the projection (x) and the token's table (cs).
template <typename T>
__device__ __forceinline__ float rotated(const T* x, const float* cs, int rot, int i) {
#pragma clang fp contract(off)
  const float v = to_f32(x[i]);
  if (i >= rot) return v;
  const int half = rot / 2;
  const bool low = i < half;
  const float other = to_f32(x[low ? i + half : i - half]);
  const float c = cs[2 * (low ? i : i - half)], s = cs[2 * (low ? i : i - half) + 1];
  return low ? v * c - other * s : v * c + other * s;
}

// Four consecutive elements i .. i + 3 of a head after the rotation (rot a multiple of 8, rows aligned to four
// elements: the four lie in one half, and so do their partners), the same bits as `rotated`.
template <typename T>
__device__ __forceinline__ void rotated_four(const T* x, const float* cs, int rot, int i, float (&out)[4]) {
#pragma clang fp contract(off)
  const Four<T> v = *reinterpret_cast<const Four<T>*>(x + i);
#pragma unroll
  for (int e = 0; e < 4; ++e) out[e] = to_f32(v.e[e]);
  if (i >= rot) return;
  const int half = rot / 2;
  const bool low = i < half;
  const int pair = low ? i : i - half;
  const Four<T> o = *reinterpret_cast<const Four<T>*>(x + (low ? i + half : pair));
  const float4 a = *reinterpret_cast<const float4*>(cs + 2 * pair), b = *reinterpret_cast<const float4*>(cs + 2 * pair + 4);
  const float c[4] = {a.x, a.z, b.x, b.z}, sn[4] = {a.y, a.w, b.y, b.w};
#pragma unroll
  for (int e = 0; e < 4; ++e) out[e] = low ? out[e] * c[e] - to_f32(o.e[e]) * sn[e] : out[e] * c[e] + to_f32(o.e[e]) * sn[e];
}

// One token's head by one wave: o (32-bit, dv elements, in LDS or memory) over its root mean square, times the gate.
// (The gate's first two elements of every lane may have been asked for earlier: g0, g1.)
template <typename T>
__device__ __forceinline__ void norm_and_gate(const float* o, const T* gate, T* out, int dv, float eps, int lane, T g0, T g1) {
#pragma clang fp contract(off)
  float ss = 0.f;
  for (int d = lane; d < dv; d += kWave) ss = fmaf(o[d], o[d], ss);
  ss = wave_sum(ss);
  const float inv = 1.0f / sqrtf(ss / (float)dv + eps);
  for (int d = lane; d < dv; d += kWave) {
    const float g = to_f32(d < kWave ? g0 : d < 2 * kWave ? g1 : gate[d]);
    out[d] = from_f32<T>(o[d] * inv * (g / (1.0f + expf(-g))));
  }
}

// ----------------------------------------------------------------------------- token after token
// A block takes up to 128 columns of one (request, head), two a lane, and eight neighbouring lanes share a column: lane
// p of them holds rows 4 (p + 8 u) .. + 3 for u = 0 .. R / 4 - 1, so that the eight lanes read 128 bytes on end, of the
// state as of a key.  Tokens come in tiles of kWalkTile whose rotated queries and keys lie in LDS; a tile's tokens
// follow each other without a barrier.  Every sum has an order fixed by the element (four chains a lane, then the
// eight lanes), whatever the tile: a token has the same bits in a prompt and in a decode step.  FUSED: the block has
// all columns of its head, and its waves norm and gate the tile's tokens at the tile's end.  VEC: rows, rotation and
// state can be read four elements at a time.
constexpr int kWalkTile = 16;
constexpr int kWalkCols = 128;

template <typename T, bool VEC, int R, bool FUSED>
__global__ void __launch_bounds__(512) retention_walk_kernel(const RetentionArgs<T> a, int cols, int col_groups) {
#pragma clang fp contract(off)
  constexpr int kPitch = 8 * R;  // a token's key in LDS, zeros behind dk
  extern __shared__ __attribute__((aligned(16))) float lds[];
  float* k_l = lds;                              // [kWalkTile][kPitch]
  float* q_l = k_l + kWalkTile * kPitch;         // [kWalkTile][kPitch]
  float* v_l = q_l + kWalkTile * kPitch;         // [kWalkTile][cols]
  float* o_l = v_l + kWalkTile * cols;           // [kWalkTile][cols]
  const int row = blockIdx.y;
  const int h = blockIdx.x / col_groups, cg = blockIdx.x % col_groups;
  const int start = a.qo_indptr[row], end = a.qo_indptr[row + 1];
  const int n_threads = blockDim.x, tid = threadIdx.x;
  const int part = tid % 8, j_loc = 2 * (tid / 8);
  const int dk = a.dk, dv = a.dv;
  float* st = a.state + (long long)a.slot_ids[row] * a.state_stride + (size_t)h * dv * dk;
  const float decay = a.decay[h];
  float S[2][R];
#pragma unroll
  for (int c = 0; c < 2; ++c) {
    const int j = cg * cols + j_loc + c;
#pragma unroll
    for (int u = 0; u < R / 4; ++u) {
      const int i = 4 * (part + 8 * u);
      if (VEC) {  // (asked for whether it is there or not, so that nothing waits between the loads)
        const bool there = j < dv && i < dk;
        const float4 s4 = *reinterpret_cast<const float4*>(st + (there ? (size_t)j * dk + i : 0));
        S[c][4 * u] = there ? s4.x : 0.f; S[c][4 * u + 1] = there ? s4.y : 0.f;
        S[c][4 * u + 2] = there ? s4.z : 0.f; S[c][4 * u + 3] = there ? s4.w : 0.f;
      } else {
#pragma unroll
        for (int e = 0; e < 4; ++e) S[c][4 * u + e] = j < dv && i + e < dk ? st[(size_t)j * dk + i + e] : 0.f;
      }
    }
  }
  const int wave = tid / kWave, lane = tid % kWave, n_waves = n_threads / kWave;
  for (int t0 = start; t0 < end; t0 += kWalkTile) {
    const int nt = min(kWalkTile, end - t0);
    __syncthreads();  // the tile before has been read to its end
    T g0 = from_f32<T>(0.f), g1 = from_f32<T>(0.f);  // the gate of the wave's first token of the tile
    auto fetch_gate = [&](int tt) {
      const T* gate = a.proj + (size_t)(t0 + tt) * a.stride + a.g_off + h * dv;
      g0 = gate[lane < dv ? lane : 0];
      g1 = gate[lane + kWave < dv ? lane + kWave : 0];
    };
    if (FUSED) fetch_gate(wave < nt ? wave : 0);
    if (VEC) {
      for (int e = tid; e < nt * (kPitch / 2); e += n_threads) {  // four channels of a key, then of a query
        const int tt = e / (kPitch / 2), f = e % (kPitch / 2);
        const bool is_k = f < kPitch / 4;
        const int i = 4 * (is_k ? f : f - kPitch / 4);
        float x4[4] = {0.f, 0.f, 0.f, 0.f};
        if (i < dk)
          rotated_four(a.proj + (size_t)(t0 + tt) * a.stride + (is_k ? a.k_off : a.q_off) + h * dk, a.cos_sin + (size_t)(t0 + tt) * a.rot,
                       a.rot, i, x4);
        const float f4 = is_k ? a.k_scale : 1.f;
        *reinterpret_cast<float4*>((is_k ? k_l : q_l) + tt * kPitch + i) = float4{x4[0] * f4, x4[1] * f4, x4[2] * f4, x4[3] * f4};
      }
    } else
    for (int e = tid; e < nt * kPitch; e += n_threads) {
      const int tt = e / kPitch, i = e % kPitch;
      const T* tok = a.proj + (size_t)(t0 + tt) * a.stride;
      const float* cs = a.cos_sin + (size_t)(t0 + tt) * a.rot;
      k_l[e] = i < dk ? rotated(tok + a.k_off + h * dk, cs, a.rot, i) * a.k_scale : 0.f;
      q_l[e] = i < dk ? rotated(tok + a.q_off + h * dk, cs, a.rot, i) : 0.f;
    }
    for (int e = tid; e < nt * cols; e += n_threads) {
      const int tt = e / cols, j = cg * cols + e % cols;
      v_l[e] = j < dv ? to_f32(a.proj[(size_t)(t0 + tt) * a.stride + a.v_off + h * dv + j]) : 0.f;
    }
    __syncthreads();
    struct Operands {
      float k[R], q[R], v[2];
    };
    auto read = [&](Operands& x, int tt_raw) {
      const int tt = tt_raw < kWalkTile ? tt_raw : kWalkTile - 1;
#pragma unroll
      for (int u = 0; u < R / 4; ++u) {
        const float4 k4 = *reinterpret_cast<const float4*>(k_l + tt * kPitch + 4 * (part + 8 * u));
        const float4 q4 = *reinterpret_cast<const float4*>(q_l + tt * kPitch + 4 * (part + 8 * u));
        x.k[4 * u] = k4.x; x.k[4 * u + 1] = k4.y; x.k[4 * u + 2] = k4.z; x.k[4 * u + 3] = k4.w;
        x.q[4 * u] = q4.x; x.q[4 * u + 1] = q4.y; x.q[4 * u + 2] = q4.z; x.q[4 * u + 3] = q4.w;
      }
      x.v[0] = v_l[tt * cols + j_loc];
      x.v[1] = v_l[tt * cols + j_loc + 1];
    };
    auto token = [&](const Operands& x, int tt) {
#pragma unroll
      for (int c = 0; c < 2; ++c) {
        float sq[4] = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int r = 0; r < R; ++r) {
          S[c][r] = fmaf(x.k[r], x.v[c], decay * S[c][r]);
          sq[r % 4] = fmaf(S[c][r], x.q[r], sq[r % 4]);
        }
        const float o = sum_of_eight_lanes((sq[0] + sq[1]) + (sq[2] + sq[3]));
        if (part == 0) o_l[tt * cols + j_loc + c] = o;
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
    if constexpr (FUSED) {
      for (int tt = wave; tt < nt; tt += n_waves) {
        if (tt != wave) fetch_gate(tt);
        norm_and_gate<T>(o_l + tt * cols, (const T*)nullptr, a.out + ((size_t)(t0 + tt) * a.H + h) * dv, dv, a.eps, lane, g0, g1);
      }
    } else {
      for (int e = tid; e < nt * cols; e += n_threads) {
        const int tt = e / cols, j = cg * cols + e % cols;
        if (j < dv) a.o_raw[((size_t)(t0 + tt) * a.H + h) * dv + j] = o_l[e];
      }
    }
  }
#pragma unroll
  for (int c = 0; c < 2; ++c) {
    const int j = cg * cols + j_loc + c;
#pragma unroll
    for (int u = 0; u < R / 4; ++u) {
      const int i = 4 * (part + 8 * u);
      if (VEC) {
        if (j < dv && i < dk) *reinterpret_cast<float4*>(st + (size_t)j * dk + i) = float4{S[c][4 * u], S[c][4 * u + 1], S[c][4 * u + 2], S[c][4 * u + 3]};
      } else {
#pragma unroll
        for (int e = 0; e < 4; ++e)
          if (j < dv && i + e < dk) st[(size_t)j * dk + i + e] = S[c][4 * u + e];
      }
    }
  }
}

// The norm and the gate where a head's columns are spread over several blocks: one wave a (token, head).
constexpr int kOutWaves = 4;
template <typename T>
__global__ void __launch_bounds__(kOutWaves* kWave) retention_output_kernel(const RetentionArgs<T> a, int t_first) {
  const size_t t = (size_t)t_first + blockIdx.x;
  const int h = blockIdx.y * kOutWaves + threadIdx.x / kWave;
  if (h >= a.H) return;
  const int lane = threadIdx.x % kWave;
  const T* gate = a.proj + t * a.stride + a.g_off + (size_t)h * a.dv;
  norm_and_gate<T>(a.o_raw + (t * a.H + h) * a.dv, gate, a.out + (t * a.H + h) * a.dv, a.dv, a.eps, lane, gate[lane < a.dv ? lane : 0],
                   gate[lane + kWave < a.dv ? lane + kWave : 0]);
}

// Whether keys, queries, their rotation and the state can be read four elements at a time.
template <typename T>
bool in_fours(const RetentionArgs<T>& a) {
  const bool rows = a.dk % 4 == 0 && a.stride % 4 == 0 && a.q_off % 4 == 0 && a.k_off % 4 == 0 && (uintptr_t)a.proj % (4 * sizeof(T)) == 0;
  return rows && a.rot % 8 == 0 && (uintptr_t)a.cos_sin % 16 == 0 && (uintptr_t)a.state % 16 == 0 && a.state_stride % 4 == 0;
}

template <typename T>
int launch_walk(const RetentionArgs<T>& a, int n_seqs, int n_tokens, hipStream_t stream) {
  const int cols = a.dv >= kWalkCols ? kWalkCols : (a.dv + 15) / 16 * 16;
  const int col_groups = (a.dv + cols - 1) / cols;
  const int threads = cols / 2 * 8;
  const int r = a.dk <= 32 ? 4 : a.dk <= 64 ? 8 : a.dk <= 128 ? 16 : 32;
  const size_t lds = (size_t)kWalkTile * (2 * 8 * r + 2 * cols) * sizeof(float);
  const dim3 grid(a.H * col_groups, n_seqs);
  const bool vec = in_fours(a);
#define TL_WALK_V(VEC, R)                                                                                        \
  do {                                                                                                           \
    if (col_groups == 1) retention_walk_kernel<T, VEC, R, true><<<grid, threads, lds, stream>>>(a, cols, 1);     \
    else retention_walk_kernel<T, VEC, R, false><<<grid, threads, lds, stream>>>(a, cols, col_groups);           \
  } while (0)
#define TL_WALK(R)                   \
  do {                               \
    if (vec) TL_WALK_V(true, R);     \
    else TL_WALK_V(false, R);        \
  } while (0)
  if (r == 4) TL_WALK(4);
  else if (r == 8) TL_WALK(8);
  else if (r == 16) TL_WALK(16);
  else TL_WALK(32);
#undef TL_WALK
#undef TL_WALK_V
  int rc = tl_check_launch("retention_walk");
  if (rc != TL_OK || col_groups == 1) return rc;
  for (int t0 = 0; t0 < n_tokens; t0 += 65535) {
    const int nt = n_tokens - t0 < 65535 ? n_tokens - t0 : 65535;
    retention_output_kernel<T><<<dim3(nt, (a.H + kOutWaves - 1) / kOutWaves), kOutWaves * kWave, 0, stream>>>(a, t0);
  }
  return tl_check_launch("retention_output");
}

// ----------------------------------------------------------------------------- segments of a prompt side by side
// A row's tokens in segments of up to kSeg.  With w_t = decay^(tokens behind t in its segment) three launches compute,
// per (segment, head) and in 32-bit on the matrix cores (16x16x4 f32):
//   1. what the segment alone leaves, L = sum_t w_t k_t v_t^T;
//   2. the states that enter: S_0 = the request's state, S_(s+1) = decay^len S_s + L_s, which takes L's place; the last
//      one becomes the request's state;
//   3. o_t = decay^(t + 1) S_in^T q_t + sum_(s <= t) decay^(t - s) (q_t . k_s) v_s, the norm and the gate.
// The MFMA's operands: lane (n16, g4) = (lane % 16, lane / 16) holds row or column n16 at depth g4; its results are rows
// 4 g4 + i, column n16.  Four steps over sixteen channels take channel 4 g4 + step, so that a lane's operands of four
// steps are four consecutive floats.  The scores are formed as (K Q^T)[s][t]: their results are, step for step, the
// other operand of (P V)[t][j], so they stay in their registers.
constexpr int kSeg = 64;
constexpr int kChunkThreads = 256;
// decay^n for n = 0 .. kSeg into LDS, by the first threads of the block.
__device__ __forceinline__ void fill_powers(float* pw, float decay) {
  if (threadIdx.x <= kSeg) pw[threadIdx.x] = powf(decay, (float)threadIdx.x);
}

// DKP, DVP: channels of keys and values rounded up to 64 or 128 (what lies beyond is zero).
template <typename T, int DKP, int DVP>
__global__ void __launch_bounds__(kChunkThreads) retention_local_kernel(const RetentionArgs<T> a, const int32_t* __restrict__ segs, float* __restrict__ ws) {
  constexpr int PK = DKP + 4, PV = DVP + 4;
  extern __shared__ __attribute__((aligned(16))) float lds[];
  float* k_l = lds;               // [kSeg][PK]: keys, rotated, scaled, times w_t
  float* v_l = k_l + kSeg * PK;   // [kSeg][PV]
  float* pw = v_l + kSeg * PV;    // decay^n, n = 0 .. kSeg
  const int seg = blockIdx.x, h = blockIdx.y;
  const int first = segs[2 * seg], len = segs[2 * seg + 1] - first;
  const int dk = a.dk, dv = a.dv;
  fill_powers(pw, a.decay[h]);
  __syncthreads();
  for (int e = threadIdx.x; e < kSeg * (DKP / 4); e += kChunkThreads) {
    const int t = e / (DKP / 4), i = 4 * (e % (DKP / 4));
    float x[4] = {0.f, 0.f, 0.f, 0.f};
    if (t < len && i < dk)
      rotated_four(a.proj + (size_t)(first + t) * a.stride + a.k_off + h * dk, a.cos_sin + (size_t)(first + t) * a.rot, a.rot, i, x);
    const float w = a.k_scale * pw[len - 1 - t < 0 ? 0 : len - 1 - t];
    *reinterpret_cast<float4*>(k_l + t * PK + i) = float4{x[0] * w, x[1] * w, x[2] * w, x[3] * w};
  }
  for (int e = threadIdx.x; e < kSeg * (DVP / 4); e += kChunkThreads) {
    const int t = e / (DVP / 4), j = 4 * (e % (DVP / 4));
    float x[4] = {0.f, 0.f, 0.f, 0.f};
    if (t < len && j < dv) {
      const Four<T> v = *reinterpret_cast<const Four<T>*>(a.proj + (size_t)(first + t) * a.stride + a.v_off + h * dv + j);
#pragma unroll
      for (int c = 0; c < 4; ++c) x[c] = to_f32(v.e[c]);
    }
    *reinterpret_cast<float4*>(v_l + t * PV + j) = float4{x[0], x[1], x[2], x[3]};
  }
  __syncthreads();
  constexpr int MT = DVP / 16 / 4, NT = DKP / 16;  // tiles of 16 columns j a wave takes, tiles of 16 rows i
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
    for (int n = 0; n < NT; ++n) kb[n] = k_l[(t + g4) * PK + 16 * n + n16];
#pragma unroll
    for (int m = 0; m < MT; ++m)
#pragma unroll
      for (int n = 0; n < NT; ++n) acc[m][n] = mfma_f32(va[m], kb[n], acc[m][n]);
  }
  float* dst = ws + ((size_t)seg * a.H + h) * dv * dk;
#pragma unroll
  for (int m = 0; m < MT; ++m)
#pragma unroll
    for (int n = 0; n < NT; ++n)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int j = 16 * (wave * MT + m) + 4 * g4 + r, i = 16 * n + n16;
        if (j < dv && i < dk) dst[(size_t)j * dk + i] = acc[m][n][r];
      }
}

// A thread takes four elements of a row's state through the row's segments; their L are asked for eight ahead.
constexpr int kCarryAhead = 8;
template <typename T>
__global__ void __launch_bounds__(256) retention_carry_kernel(const RetentionArgs<T> a, const int32_t* __restrict__ segs,
                                                              const int32_t* __restrict__ row_seg, float* __restrict__ ws) {
  const size_t per_seg = (size_t)a.H * a.dv * a.dk;
  const size_t e = 4 * ((size_t)blockIdx.x * 256 + threadIdx.x);
  if (e >= per_seg) return;
  const int row = blockIdx.y;
  const float decay = a.decay[e / ((size_t)a.dv * a.dk)];
  const int s0 = row_seg[row], s1 = row_seg[row + 1];
  float4* st = reinterpret_cast<float4*>(a.state + (long long)a.slot_ids[row] * a.state_stride + e);
  const float whole = powf(decay, (float)kSeg);
  float4 S = *st;
  for (int s = s0; s < s1; s += kCarryAhead) {
    float4 L[kCarryAhead];
    int len[kCarryAhead];
#pragma unroll
    for (int u = 0; u < kCarryAhead; ++u) {
      const int at = s + u < s1 ? s + u : s1 - 1;
      L[u] = *reinterpret_cast<const float4*>(ws + at * per_seg + e);
      len[u] = segs[2 * at + 1] - segs[2 * at];
    }
#pragma unroll
    for (int u = 0; u < kCarryAhead; ++u) {
      if (s + u >= s1) break;
      *reinterpret_cast<float4*>(ws + (size_t)(s + u) * per_seg + e) = S;
      const float f = len[u] == kSeg ? whole : powf(decay, (float)len[u]);
      S = float4{fmaf(f, S.x, L[u].x), fmaf(f, S.y, L[u].y), fmaf(f, S.z, L[u].z), fmaf(f, S.w, L[u].w)};
    }
  }
  *st = S;
}

template <typename T, int DKP, int DVP>
__global__ void __launch_bounds__(kChunkThreads) retention_read_kernel(const RetentionArgs<T> a, const int32_t* __restrict__ segs, const float* __restrict__ ws) {
  constexpr int PK = DKP + 4, PV = DVP + 4;
  constexpr int NK = DKP / 16, NV = DVP / 16, NS = kSeg / 16;
  extern __shared__ __attribute__((aligned(16))) float lds[];
  float* x_l = lds;                                  // keys, then values, then the results: [kSeg][PK or PV]
  float* pw = lds + kSeg * (PK > PV ? PK : PV);      // decay^n, n = 0 .. kSeg
  const int seg = blockIdx.x, h = blockIdx.y;
  const int first = segs[2 * seg], len = segs[2 * seg + 1] - first;
  const int dk = a.dk, dv = a.dv;
  const int wave = threadIdx.x / kWave, lane = threadIdx.x % kWave, n16 = lane % 16, g4 = lane / 16;
  fill_powers(pw, a.decay[h]);
  // this wave's sixteen queries, rotated: lane (n16, g4) has query 16 wave + n16, channels 16 u + 4 g4 .. + 3
  const int tq = 16 * wave + n16;
  float q[NK][4];
#pragma unroll
  for (int u = 0; u < NK; ++u) {
    const int i = 16 * u + 4 * g4;
#pragma unroll
    for (int c = 0; c < 4; ++c) q[u][c] = 0.f;
    if (tq < len && i < dk)
      rotated_four(a.proj + (size_t)(first + tq) * a.stride + a.q_off + h * dk, a.cos_sin + (size_t)(first + tq) * a.rot, a.rot, i, q[u]);
  }
  for (int e = threadIdx.x; e < kSeg * (DKP / 4); e += kChunkThreads) {
    const int t = e / (DKP / 4), i = 4 * (e % (DKP / 4));
    float x[4] = {0.f, 0.f, 0.f, 0.f};
    if (t < len && i < dk)
      rotated_four(a.proj + (size_t)(first + t) * a.stride + a.k_off + h * dk, a.cos_sin + (size_t)(first + t) * a.rot, a.rot, i, x);
    *reinterpret_cast<float4*>(x_l + t * PK + i) = float4{x[0] * a.k_scale, x[1] * a.k_scale, x[2] * a.k_scale, x[3] * a.k_scale};
  }
  // the segment's values, on their way while the scores are formed
  constexpr int VL = kSeg * (DVP / 4) / kChunkThreads;
  Four<T> vraw[VL];
#pragma unroll
  for (int u = 0; u < VL; ++u) {
    const int e = threadIdx.x + u * kChunkThreads;
    const int t = e / (DVP / 4), j = 4 * (e % (DVP / 4));
    const bool there = t < len && j < dv;
    vraw[u] = *reinterpret_cast<const Four<T>*>(a.proj + (size_t)(first + (there ? t : 0)) * a.stride + a.v_off + h * dv + (there ? j : 0));
    if (!there) vraw[u] = Four<T>{};
  }
  // what the state that entered gives: acc[n] = rows t = 4 g4 + i, columns j = 16 n + n16
  f32x4_t acc[NV];
  const float* S_in = ws + ((size_t)seg * a.H + h) * dv * dk;
#pragma unroll
  for (int n = 0; n < NV; ++n) {
    acc[n] = f32x4_t{0.f, 0.f, 0.f, 0.f};
    const int j = 16 * n + n16;
    float4 s4[NK];
#pragma unroll
    for (int u = 0; u < NK; ++u) {
      const int i = 16 * u + 4 * g4;
      const bool there = j < dv && i < dk;
      s4[u] = *reinterpret_cast<const float4*>(S_in + (there ? (size_t)j * dk + i : 0));
      if (!there) s4[u] = float4{0.f, 0.f, 0.f, 0.f};
    }
#pragma unroll
    for (int u = 0; u < NK; ++u) {
      acc[n] = mfma_f32(q[u][0], s4[u].x, acc[n]);
      acc[n] = mfma_f32(q[u][1], s4[u].y, acc[n]);
      acc[n] = mfma_f32(q[u][2], s4[u].z, acc[n]);
      acc[n] = mfma_f32(q[u][3], s4[u].w, acc[n]);
    }
  }
  __syncthreads();  // keys and powers are in LDS
  {
    float f[4];
#pragma unroll
    for (int r = 0; r < 4; ++r) f[r] = pw[16 * wave + 4 * g4 + r + 1];
#pragma unroll
    for (int n = 0; n < NV; ++n)
#pragma unroll
      for (int r = 0; r < 4; ++r) acc[n][r] *= f[r];
  }
  // scores P[s][t] of the wave's queries with the keys of every sixteen up to its own (results: rows s, column t)
  f32x4_t p[NS];
#pragma unroll
  for (int b = 0; b < NS; ++b) {
    p[b] = f32x4_t{0.f, 0.f, 0.f, 0.f};
    if (b <= wave) {  // (the same for the whole wave)
#pragma unroll
      for (int u = 0; u < NK; ++u) {
        const float4 k4 = *reinterpret_cast<const float4*>(x_l + (16 * b + n16) * PK + 16 * u + 4 * g4);
        p[b] = mfma_f32(k4.x, q[u][0], p[b]);
        p[b] = mfma_f32(k4.y, q[u][1], p[b]);
        p[b] = mfma_f32(k4.z, q[u][2], p[b]);
        p[b] = mfma_f32(k4.w, q[u][3], p[b]);
      }
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int dist = tq - (16 * b + 4 * g4 + r);
        const float f = pw[dist < 0 ? 0 : dist];
        p[b][r] = dist < 0 ? 0.f : p[b][r] * f;
      }
    }
  }
  __syncthreads();  // everybody has read the keys
#pragma unroll
  for (int u = 0; u < VL; ++u) {
    const int e = threadIdx.x + u * kChunkThreads;
    const int t = e / (DVP / 4), j = 4 * (e % (DVP / 4));
    *reinterpret_cast<float4*>(x_l + t * PV + j) = float4{to_f32(vraw[u].e[0]), to_f32(vraw[u].e[1]), to_f32(vraw[u].e[2]), to_f32(vraw[u].e[3])};
  }
  __syncthreads();
#pragma unroll
  for (int b = 0; b < NS; ++b) {
    if (b > wave) continue;
#pragma unroll
    for (int r = 0; r < 4; ++r)
#pragma unroll
      for (int n = 0; n < NV; ++n) acc[n] = mfma_f32(p[b][r], x_l[(16 * b + 4 * g4 + r) * PV + 16 * n + n16], acc[n]);
  }
  // every token's head over its root mean square: a token's columns lie in the sixteen lanes of its row group
  float inv[4];
#pragma unroll
  for (int r = 0; r < 4; ++r) {
    float ss = 0.f;
#pragma unroll
    for (int n = 0; n < NV; ++n) ss = fmaf(acc[n][r], acc[n][r], ss);
    ss = sum_of_eight_lanes(ss);
    ss += __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(ss), 0x140, 0xf, 0xf, false));
    inv[r] = 1.0f / sqrtf(ss / (float)dv + a.eps);
  }
  __syncthreads();  // everybody has read the values
#pragma unroll
  for (int n = 0; n < NV; ++n)
#pragma unroll
    for (int r = 0; r < 4; ++r) x_l[(16 * wave + 4 * g4 + r) * PV + 16 * n + n16] = acc[n][r] * inv[r];
  __syncthreads();
  for (int e = threadIdx.x; e < len * (DVP / 4); e += kChunkThreads) {
    const int t = e / (DVP / 4), j = 4 * (e % (DVP / 4));
    if (j >= dv) continue;
    const float4 o = *reinterpret_cast<const float4*>(x_l + t * PV + j);
    const Four<T> g = *reinterpret_cast<const Four<T>*>(a.proj + (size_t)(first + t) * a.stride + a.g_off + h * dv + j);
    const float ov[4] = {o.x, o.y, o.z, o.w};
    Four<T> out;
#pragma unroll
    for (int c = 0; c < 4; ++c) {
      const float gv = to_f32(g.e[c]);
      out.e[c] = from_f32<T>(ov[c] * (gv / (1.0f + expf(-gv))));
    }
    *reinterpret_cast<Four<T>*>(a.out + ((size_t)(first + t) * a.H + h) * dv + j) = out;
  }
}

template <typename T, int DKP, int DVP>
int launch_chunks(const RetentionArgs<T>& a, int n_rows, int n_segs, const int32_t* segs, const int32_t* row_seg, float* ws, hipStream_t stream) {
  constexpr int PK = DKP + 4, PV = DVP + 4;
  const size_t lds_local = ((size_t)kSeg * (PK + PV) + kSeg + 1) * sizeof(float);
  const size_t lds_read = ((size_t)kSeg * (PK > PV ? PK : PV) + kSeg + 1) * sizeof(float);
  if (lds_local > 48 * 1024) {
    hipError_t e = hipFuncSetAttribute((const void*)retention_local_kernel<T, DKP, DVP>, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds_local);
    if (e != hipSuccess) return tl_fail(TL_ERR_HIP, "retention: %s", hipGetErrorString(e));
  }
  const dim3 grid(n_segs, a.H);
  retention_local_kernel<T, DKP, DVP><<<grid, kChunkThreads, lds_local, stream>>>(a, segs, ws);
  int rc = tl_check_launch("retention_local");
  if (rc != TL_OK) return rc;
  const size_t fours = (size_t)a.H * a.dv * a.dk / 4;
  retention_carry_kernel<T><<<dim3((unsigned)((fours + 255) / 256), n_rows), 256, 0, stream>>>(a, segs, row_seg, ws);
  rc = tl_check_launch("retention_carry");
  if (rc != TL_OK) return rc;
  retention_read_kernel<T, DKP, DVP><<<grid, kChunkThreads, lds_read, stream>>>(a, segs, ws);
  return tl_check_launch("retention_read");
}

}  // namespace

// The most tokens of a segment of tl_retention_chunks, and the most channels of keys and of values that it takes.
TL_EXPORT int tl_retention_segment() { return kSeg; }
TL_EXPORT int tl_retention_chunk_channels() { return 128; }

// The recurrence of bfloat16 prompts by segments (see above).  segs: [n_segs][2] first token and one past the last of
// every segment (at most tl_retention_segment() tokens), every row's in order; row_seg [n_rows + 1]: the first segment
// of every row; slot_ids [n_rows].  Tokens are rows of proj, cos_sin and out.  ws: n_segs * H * dv * dk floats.
// dk and dv: multiples of 4 up to tl_retention_chunk_channels(); rot a multiple of 8; rows, table and state aligned
// so that four elements can be read at a time.
TL_EXPORT int tl_retention_chunks(const void* proj, int stride, int q_off, int k_off, int v_off, int g_off, const float* cos_sin,
                                  int rot, const float* decay, float* state, long long state_stride, const int32_t* slot_ids,
                                  void* out, int n_rows, int H, int dk, int dv, float eps, const int32_t* segs, const int32_t* row_seg,
                                  int n_segs, float* ws, int dtype, hipStream_t stream) {
  TL_REQUIRE(n_rows >= 0 && n_segs >= 0 && H > 0 && dk > 0 && dv > 0 && rot >= 0 && rot <= dk, "retention: bad sizes");
  TL_REQUIRE(rot == 0 || cos_sin != nullptr, "retention: a rotation without its table");
  if (dtype != TL_BF16) return tl_fail(TL_ERR_UNSUPPORTED, "retention: segments are for bfloat16 models");
  if (dk > 128 || dv > 128) return tl_fail(TL_ERR_UNSUPPORTED, "retention: segments take keys and values of up to 128 channels, got %d and %d", dk, dv);
  TL_REQUIRE(n_rows <= 65535 && H <= 65535, "retention: too many requests or heads a step");
  if (n_rows == 0 || n_segs == 0) return TL_OK;
  TL_REQUIRE(segs && row_seg && ws && slot_ids, "retention: no segments or no workspace");
  const RetentionArgs<bf16_t> a = {(const bf16_t*)proj, stride, q_off, k_off, v_off, g_off, cos_sin, rot, decay, state, state_stride, nullptr,
                                   slot_ids, (bf16_t*)out, nullptr, H, dk, dv, eps, 1.0f / sqrtf((float)dk)};
  TL_REQUIRE(in_fours(a) && dv % 4 == 0 && v_off % 4 == 0 && g_off % 4 == 0 && (uintptr_t)out % 8 == 0 && (uintptr_t)ws % 16 == 0,
             "retention: rows that cannot be read four elements at a time");
  if (dk <= 64 && dv <= 64) return launch_chunks<bf16_t, 64, 64>(a, n_rows, n_segs, segs, row_seg, ws, stream);
  if (dk <= 64) return launch_chunks<bf16_t, 64, 128>(a, n_rows, n_segs, segs, row_seg, ws, stream);
  if (dv <= 64) return launch_chunks<bf16_t, 128, 64>(a, n_rows, n_segs, segs, row_seg, ws, stream);
  return launch_chunks<bf16_t, 128, 128>(a, n_rows, n_segs, segs, row_seg, ws, stream);
}

// Columns of one head that a block of tl_retention takes; a head with more values needs o_raw.
TL_EXPORT int tl_retention_block_columns() { return kWalkCols; }

// The recurrence over each request's tokens, token after token (see the head of this file).  Row r of the step holds
// tokens qo_indptr[r] .. qo_indptr[r + 1] - 1 of the request in slot slot_ids[r]; the n_seqs rows hold n_tokens tokens
// from token 0 on.  o_raw: a workspace of n_tokens * H * dv floats, needed when dv > tl_retention_block_columns().
TL_EXPORT int tl_retention(const void* proj, int stride, int q_off, int k_off, int v_off, int g_off, const float* cos_sin, int rot,
                           const float* decay, float* state, long long state_stride, const int32_t* qo_indptr,
                           const int32_t* slot_ids, void* out, float* o_raw, int n_tokens, int n_seqs, int H, int dk, int dv, float eps,
                           int dtype, hipStream_t stream) {
  TL_REQUIRE(n_seqs >= 0 && n_tokens >= 0 && H > 0 && dk > 0 && dv > 0 && rot >= 0 && rot % 2 == 0 && rot <= dk, "retention: bad sizes");
  if (dk > 256) return tl_fail(TL_ERR_UNSUPPORTED, "retention: keys of %d channels, at most 256", dk);
  TL_REQUIRE(n_seqs <= 65535, "retention: too many requests a step");
  TL_REQUIRE(rot == 0 || cos_sin != nullptr, "retention: a rotation without its table");
  TL_REQUIRE(dv <= kWalkCols || o_raw != nullptr, "retention: no workspace for values of %d channels", dv);
  if (n_seqs == 0 || n_tokens == 0) return TL_OK;
  const float k_scale = 1.0f / sqrtf((float)dk);
  if (dtype == TL_F32)
    return launch_walk<float>({(const float*)proj, stride, q_off, k_off, v_off, g_off, cos_sin, rot, decay, state, state_stride, qo_indptr,
                               slot_ids, (float*)out, o_raw, H, dk, dv, eps, k_scale}, n_seqs, n_tokens, stream);
  if (dtype == TL_BF16)
    return launch_walk<bf16_t>({(const bf16_t*)proj, stride, q_off, k_off, v_off, g_off, cos_sin, rot, decay, state, state_stride, qo_indptr,
                                slot_ids, (bf16_t*)out, o_raw, H, dk, dv, eps, k_scale}, n_seqs, n_tokens, stream);
  return tl_fail(TL_ERR_ARG, "retention: unknown dtype %d", dtype);
}
