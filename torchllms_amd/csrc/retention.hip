// Retention: linear attention whose state fades by a constant per head.  Per request and head h, state S [dk][dv] in
// 32-bit, kept transposed in state[slot][h][j][i] (column j of S is contiguous).  For every token, in order, with q and
// k rotated by the token's position and k times dk^-1/2:
//   S <- decay_h S + k v^T;  o = S^T q;  out[t, h, :] = T(o / sqrt(mean(o^2) + eps) * silu(gate[t, h, :]))
// proj: the layer's fused projection [n_tokens, stride], of which the columns of q, k (H * dk each), v and the gate
// (H * dv each) are read from their offsets.  cos_sin: the step's table [n_tokens][rot / 2][2] (channel i of a head is
// paired with channel i + rot / 2; channels from rot on pass).  Rotated keys and queries, decays, sums, state and norm
// are 32-bit.
#include "common.h"

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

__device__ __forceinline__ float lane_xor1(float v) {
  return __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(v), 0xB1, 0xf, 0xf, false));
}
__device__ __forceinline__ float lane_xor2(float v) {
  return __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(v), 0x4E, 0xf, 0xf, false));
}
__device__ __forceinline__ float lane_half_mirror(float v) {
  return __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(v), 0x141, 0xf, 0xf, false));
}
// The sum over eight neighbouring lanes; each of them gets the same bits.
__device__ __forceinline__ float sum_of_eight_lanes(float v) {
  v += lane_xor1(v);
  v += lane_xor2(v);
  v += lane_half_mirror(v);
  return v;
}

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

// One token's head by one wave: o (32-bit, dv elements, in LDS or memory) over its root mean square, times the gate.
template <typename T>
__device__ __forceinline__ void norm_and_gate(const float* o, const T* gate, T* out, int dv, float eps, int lane) {
#pragma clang fp contract(off)
  float ss = 0.f;
  for (int d = lane; d < dv; d += kWave) ss = fmaf(o[d], o[d], ss);
  ss = wave_sum(ss);
  const float inv = 1.0f / sqrtf(ss / (float)dv + eps);
  for (int d = lane; d < dv; d += kWave) {
    const float g = to_f32(gate[d]);
    out[d] = from_f32<T>(o[d] * inv * (g / (1.0f + expf(-g))));
  }
}

// ----------------------------------------------------------------------------- token after token
// A block takes up to 128 columns of one (request, head), two a lane, and eight neighbouring lanes share a column: lane
// p of them holds rows 4 (p + 8 u) .. + 3 for u = 0 .. R / 4 - 1, so that the eight lanes read 128 bytes on end, of the
// state as of a key.  Tokens come in tiles of kWalkTile whose rotated queries and keys lie in LDS; a tile's tokens
// follow each other without a barrier.  Every sum has an order fixed by the element (four chains a lane, then the
// eight lanes), whatever the tile: a token has the same bits in a prompt and in a decode step.  FUSED: the block has
// all columns of its head, and its waves norm and gate the tile's tokens at the tile's end.
constexpr int kWalkTile = 16;
constexpr int kWalkCols = 128;

template <typename T, int R, bool FUSED>
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
    for (int r = 0; r < R; ++r) {
      const int i = 4 * (part + 8 * (r / 4)) + r % 4;
      S[c][r] = j < dv && i < dk ? st[(size_t)j * dk + i] : 0.f;
    }
  }
  for (int t0 = start; t0 < end; t0 += kWalkTile) {
    const int nt = min(kWalkTile, end - t0);
    __syncthreads();  // the tile before has been read to its end
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
      for (int tt = tid / kWave; tt < nt; tt += n_threads / kWave)
        norm_and_gate<T>(o_l + tt * cols, a.proj + (size_t)(t0 + tt) * a.stride + a.g_off + h * dv,
                         a.out + ((size_t)(t0 + tt) * a.H + h) * dv, dv, a.eps, tid % kWave);
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
    for (int r = 0; r < R; ++r) {
      const int i = 4 * (part + 8 * (r / 4)) + r % 4;
      if (j < dv && i < dk) st[(size_t)j * dk + i] = S[c][r];
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
  norm_and_gate<T>(a.o_raw + (t * a.H + h) * a.dv, a.proj + t * a.stride + a.g_off + (size_t)h * a.dv, a.out + (t * a.H + h) * a.dv, a.dv,
                   a.eps, threadIdx.x % kWave);
}

template <typename T>
int launch_walk(const RetentionArgs<T>& a, int n_seqs, int n_tokens, hipStream_t stream) {
  const int cols = a.dv >= kWalkCols ? kWalkCols : (a.dv + 15) / 16 * 16;
  const int col_groups = (a.dv + cols - 1) / cols;
  const int threads = cols / 2 * 8;
  const int r = a.dk <= 32 ? 4 : a.dk <= 64 ? 8 : a.dk <= 128 ? 16 : 32;
  const size_t lds = (size_t)kWalkTile * (2 * 8 * r + 2 * cols) * sizeof(float);
  const dim3 grid(a.H * col_groups, n_seqs);
#define TL_WALK(R)                                                                                          \
  do {                                                                                                      \
    if (col_groups == 1) retention_walk_kernel<T, R, true><<<grid, threads, lds, stream>>>(a, cols, 1);     \
    else retention_walk_kernel<T, R, false><<<grid, threads, lds, stream>>>(a, cols, col_groups);           \
  } while (0)
  if (r == 4) TL_WALK(4);
  else if (r == 8) TL_WALK(8);
  else if (r == 16) TL_WALK(16);
  else TL_WALK(32);
#undef TL_WALK
  int rc = tl_check_launch("retention_walk");
  if (rc != TL_OK || col_groups == 1) return rc;
  for (int t0 = 0; t0 < n_tokens; t0 += 65535) {
    const int nt = n_tokens - t0 < 65535 ? n_tokens - t0 : 65535;
    retention_output_kernel<T><<<dim3(nt, (a.H + kOutWaves - 1) / kOutWaves), kOutWaves * kWave, 0, stream>>>(a, t0);
  }
  return tl_check_launch("retention_output");
}

}  // namespace

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
