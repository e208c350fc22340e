// The matrix state with a fixed decay per head, S <- lambda S + k v^T, o = S^T q, over portions of prompts:
// chunks of 64 tokens side by side instead of token by token.  For the tokens i of a chunk, S the state
// before it and n its length:
//
//   o_i     = lambda^(i+1) S^T q_i + sum_{j <= i} lambda^(i-j) (k_j . q_i) v_j
//   S_after = lambda^n S + sum_j lambda^(n-1-j) k_j v_j^T
//
// Three kernels: every chunk's own sum (its state had it started from zero) into a workspace; a walk over a
// request's chunks, element by element, which leaves the state before each chunk in the workspace and the
// last state in the request's slot; every chunk's results.  All products are float32 matrix instructions
// (16 x 16 x 4) with float32 operands, in either dtype of the model, so nothing is rounded that the
// token-by-token scan (linear_attention.hip) does not round.  Decay powers are taken of whole distances
// (never a quotient of powers), so no decay is too fast for a chunk.  Chunks are counted from a request's
// first token in the step.
//
// The instruction adds over the index lk of a lane (lane = 16 lk + li); both operands of a product are dealt
// in the same way, so four instructions whose lanes hold the elements 4 lk + i (i = 0..3) of a run of sixteen
// sum over the whole run, and a lane fetches its four with one 16-byte load.  A state in memory has its rows
// in fours (see linear_attention.hip), which is the order of an accumulator's four values.

#include <hip/hip_runtime.h>

#include "device_utils.h"
#include "kvcore_hip.h"

using namespace kvc;

namespace {

#define S(stream) reinterpret_cast<hipStream_t>(stream)

typedef float f32x4_t __attribute__((ext_vector_type(4)));

constexpr int kChunk = 64;
constexpr int kCols = 64;       // value channels a block
constexpr int kColPad = 4;      // floats between rows of 64 in LDS
constexpr int kVRow = kCols + kColPad;

struct ChunkArgs {
  float* out;         // [T, nh * dv]
  const float* q;     // rows of nqk heads of d
  int64_t q_stride;
  const float* k;
  int64_t k_stride;
  const float* v;     // rows of nh heads of dv
  int64_t v_stride;
  const float* decay;  // [nh]
  float* work;        // [chunks][nh][dpad][dv], rows in fours
  float* state;       // [slots][nh][dpad][dv], rows in fours
  const int32_t* positions;
  const int32_t* token_req;
  const int32_t* q_start;
  const int32_t* slots;
  int R, nh, nqk, d, dv, dpad;
  float q_scale;
  int silu_in;
};

// Which request and which of its chunks a block works on: first token and token count of the chunk (0: none).
struct ChunkPlace {
  int req, t0, n;
};
__device__ __forceinline__ ChunkPlace find_chunk(const ChunkArgs& a, int index) {
  for (int r = 0; r < a.R; ++r) {
    const int b = a.q_start[r], e = a.q_start[r + 1];
    const int chunks = (e - b + kChunk - 1) / kChunk;
    if (index < chunks) {
      const int t0 = b + index * kChunk;
      return {r, t0, e - t0 < kChunk ? e - t0 : kChunk};
    }
    index -= chunks;
  }
  return {-1, 0, 0};
}

// Rows of the chunk's tokens, columns [c0, c0 + width) of a head of `size` values, into LDS rows of `row`
// floats, zeros where there is no token or no column (up to `padded` columns); silu on the way where asked.
template <int VEC>
__device__ __forceinline__ void stage(float* dst, int row, const float* src, int64_t stride, const ChunkPlace& at,
                                      int size, int padded, int silu_in) {
  const int groups = padded / 4;
  for (int idx = threadIdx.x; idx < kChunk * groups; idx += blockDim.x) {
    const int i = idx / groups, c = 4 * (idx - i * groups);
    f32x4_t x = {0.f, 0.f, 0.f, 0.f};
    if (i < at.n) {
      const float* p = src + (at.t0 + i) * stride + c;
      if (VEC) {
        if (c < size) x = *reinterpret_cast<const f32x4_t*>(p);
      } else {
#pragma unroll
        for (int e = 0; e < 4; ++e)
          if (c + e < size) x[e] = p[e];
      }
      if (silu_in) {
#pragma unroll
        for (int e = 0; e < 4; ++e) x[e] = silu_of(x[e]);  // zero stays zero
      }
    }
    *reinterpret_cast<f32x4_t*>(dst + i * row + c) = x;
  }
}

// ---- every chunk's own sum.  Wave w takes the key channels 16 (w + 4 m) .., all of the block's columns.
template <int NM, int VEC>
__global__ __launch_bounds__(256) void chunk_sums_kernel(const ChunkArgs a) {
  extern __shared__ __attribute__((aligned(16))) float lds[];
  const ChunkPlace at = find_chunk(a, blockIdx.x);
  if (at.n == 0 || a.token_req[at.t0] < 0) return;  // nothing here, or padding: the same for the whole block
  const int h = blockIdx.y, c0 = blockIdx.z * kCols;
  const int hk = h / (a.nh / a.nqk);
  const int tid = threadIdx.x, lane = tid & 63, li = lane & 15, lk = lane >> 4;
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int dp = (a.d + 15) & ~15, krow = dp + kColPad;
  float* k_s = lds;                          // [64][krow]
  float* v_s = k_s + kChunk * krow;          // [64][kVRow]
  float* pw = v_s + kChunk * kVRow;          // [64] weight of token j
  if (tid < kChunk) pw[tid] = tid < at.n ? powf(a.decay[h], static_cast<float>(at.n - 1 - tid)) : 0.f;
  stage<VEC>(k_s, krow, a.k + static_cast<int64_t>(hk) * a.d, a.k_stride, at, a.d, dp, a.silu_in);
  const int cols = a.dv - c0 < kCols ? a.dv - c0 : kCols;
  stage<VEC>(v_s, kVRow, a.v + static_cast<int64_t>(h) * a.dv + c0, a.v_stride, at, cols, kCols, a.silu_in);
  __syncthreads();
  f32x4_t acc[NM][4];
#pragma unroll
  for (int m = 0; m < NM; ++m)
#pragma unroll
    for (int c = 0; c < 4; ++c) acc[m][c] = f32x4_t{0.f, 0.f, 0.f, 0.f};
  const int steps = (at.n + 15) / 16;
  for (int s = 0; s < steps; ++s) {
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int j = 16 * s + 4 * lk + i;
      const float w = pw[j];
      float ka[NM], vb[4];
#pragma unroll
      for (int m = 0; m < NM; ++m) {
        const int n0 = 16 * (wave + 4 * m);
        ka[m] = k_s[j * krow + (n0 < dp ? n0 : 0) + li] * w;
      }
#pragma unroll
      for (int c = 0; c < 4; ++c) vb[c] = v_s[j * kVRow + 16 * c + li];
#pragma unroll
      for (int m = 0; m < NM; ++m)
#pragma unroll
        for (int c = 0; c < 4; ++c) acc[m][c] = __builtin_amdgcn_mfma_f32_16x16x4f32(ka[m], vb[c], acc[m][c], 0, 0, 0);
    }
  }
  // lane holds column li and key channels 4 lk .. of its tiles: four rows of one column, one 16-byte store
  float* dst = a.work + (static_cast<int64_t>(blockIdx.x) * a.nh + h) * a.dpad * a.dv;
#pragma unroll
  for (int m = 0; m < NM; ++m) {
    const int n = 16 * (wave + 4 * m) + 4 * lk;
    if (n >= a.dpad) continue;
#pragma unroll
    for (int c = 0; c < 4; ++c) {
      const int col = c0 + 16 * c + li;
      if (col < a.dv) *reinterpret_cast<f32x4_t*>(dst + (static_cast<int64_t>(n >> 2) * a.dv + col) * 4) = acc[m][c];
    }
  }
}

// ---- the walk over a request's chunks: a thread four rows of one column
__global__ __launch_bounds__(256) void chunk_walk_kernel(const ChunkArgs a) {
  const int r = blockIdx.x, h = blockIdx.y;
  const int b = a.q_start[r], e = a.q_start[r + 1];
  if (e <= b || a.token_req[b] < 0) return;
  const int fours = a.dpad / 4 * a.dv;
  const int idx = blockIdx.z * blockDim.x + threadIdx.x;
  if (idx >= fours) return;
  int first = 0;  // the request's first chunk in the workspace
  for (int p = 0; p < r; ++p) first += (a.q_start[p + 1] - a.q_start[p] + kChunk - 1) / kChunk;
  const int chunks = (e - b + kChunk - 1) / kChunk;
  float* st = a.state + ((static_cast<int64_t>(a.slots[r]) * a.nh + h) * a.dpad * a.dv) + static_cast<int64_t>(idx) * 4;
  f32x4_t s = {0.f, 0.f, 0.f, 0.f};
  if (a.positions[b] != 0) {  // the same for the whole block
    s = *reinterpret_cast<const f32x4_t*>(st);
    const int n = idx / a.dv * 4;
#pragma unroll
    for (int i = 0; i < 4; ++i)
      if (n + i >= a.d) s[i] = 0.f;  // rows that pad the state are never written by anyone else
  }
  const float lambda = a.decay[h];
  const float whole = powf(lambda, static_cast<float>(kChunk));
  const int64_t step = static_cast<int64_t>(a.nh) * a.dpad * a.dv;
  float* w = a.work + (static_cast<int64_t>(first) * a.nh + h) * a.dpad * a.dv + static_cast<int64_t>(idx) * 4;
  constexpr int kAhead = 8;
  for (int c0 = 0; c0 < chunks; c0 += kAhead) {
    f32x4_t own[kAhead];
#pragma unroll
    for (int i = 0; i < kAhead; ++i) {
      const int c = c0 + i < chunks ? c0 + i : chunks - 1;
      own[i] = *reinterpret_cast<const f32x4_t*>(w + c * step);
    }
#pragma unroll
    for (int i = 0; i < kAhead; ++i) {
      const int c = c0 + i;
      if (c < chunks) {
        *reinterpret_cast<f32x4_t*>(w + c * step) = s;
        const int n = e - b - c * kChunk;
        s = s * (n >= kChunk ? whole : powf(lambda, static_cast<float>(n))) + own[i];
      }
    }
  }
  *reinterpret_cast<f32x4_t*>(st) = s;
}

// ---- every chunk's results.  Wave w takes the queries 16 w .. 16 w + 15 (an operand's columns); a query's
// values stay in registers: NS runs of sixteen channels, of which a lane holds four.
template <int NS, int VEC>
__global__ __launch_bounds__(256) void chunk_results_kernel(const ChunkArgs a) {
  extern __shared__ __attribute__((aligned(16))) float lds[];
  const ChunkPlace at = find_chunk(a, blockIdx.x);
  if (at.n == 0) return;
  const int h = blockIdx.y, c0 = blockIdx.z * kCols;
  const int tid = threadIdx.x, lane = tid & 63, li = lane & 15, lk = lane >> 4;
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int cols = a.dv - c0 < kCols ? a.dv - c0 : kCols;
  const int width = a.nh * a.dv;
  if (a.token_req[at.t0] < 0) {  // padding rows: zeros
    for (int idx = tid; idx < at.n * cols; idx += blockDim.x) {
      const int i = idx / cols, c = idx - i * cols;
      a.out[static_cast<int64_t>(at.t0 + i) * width + h * a.dv + c0 + c] = 0.f;
    }
    return;
  }
  const int hk = h / (a.nh / a.nqk);
  const int dp = (a.d + 15) & ~15, krow = dp + kColPad;
  float* k_s = lds;
  float* v_s = k_s + kChunk * krow;
  float* pw = v_s + kChunk * kVRow;  // [65] powers of the decay
  if (tid <= kChunk) pw[tid] = powf(a.decay[h], static_cast<float>(tid));
  const int query = 16 * wave + li;
  const bool live = query < at.n;
  // q, asked for first
  f32x4_t qv[NS];
  {
    const float* p = a.q + (at.t0 + (live ? query : 0)) * a.q_stride + static_cast<int64_t>(hk) * a.d + 4 * lk;
#pragma unroll
    for (int s = 0; s < NS; ++s) {
      qv[s] = f32x4_t{0.f, 0.f, 0.f, 0.f};
      const int n = 16 * s + 4 * lk;
      if (VEC) {
        if (n < a.d) qv[s] = *reinterpret_cast<const f32x4_t*>(p + 16 * s);
      } else {
#pragma unroll
        for (int e = 0; e < 4; ++e)
          if (n + e < a.d) qv[s][e] = p[16 * s + e];
      }
    }
  }
  stage<VEC>(k_s, krow, a.k + static_cast<int64_t>(hk) * a.d, a.k_stride, at, a.d, dp, a.silu_in);
  stage<VEC>(v_s, kVRow, a.v + static_cast<int64_t>(h) * a.dv + c0, a.v_stride, at, cols, kCols, a.silu_in);
#pragma unroll
  for (int s = 0; s < NS; ++s)
#pragma unroll
    for (int e = 0; e < 4; ++e) qv[s][e] = live ? (a.silu_in ? silu_of(qv[s][e]) : qv[s][e]) * a.q_scale : 0.f;
  __syncthreads();
  if (16 * wave >= at.n) return;  // scalar; no barrier follows

  // the state before the chunk: S^T q
  const float* st = a.work + (static_cast<int64_t>(blockIdx.x) * a.nh + h) * a.dpad * a.dv;
  f32x4_t far[4];
#pragma unroll
  for (int c = 0; c < 4; ++c) far[c] = f32x4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll
  for (int s = 0; s < NS; ++s) {
    if (16 * s < a.d) {  // scalar
      const int n = 16 * s + 4 * lk;
      const int row = n < a.dpad ? n >> 2 : 0;  // rows beyond read the first: their q is zero
      f32x4_t sv[4];
#pragma unroll
      for (int c = 0; c < 4; ++c) {
        const int col = c0 + 16 * c + li;
        sv[c] = *reinterpret_cast<const f32x4_t*>(st + (static_cast<int64_t>(row) * a.dv + (col < a.dv ? col : c0)) * 4);
      }
#pragma unroll
      for (int i = 0; i < 4; ++i)
#pragma unroll
        for (int c = 0; c < 4; ++c) far[c] = __builtin_amdgcn_mfma_f32_16x16x4f32(sv[c][i], qv[s][i], far[c], 0, 0, 0);
    }
  }
  // the chunk's own keys up to the query: tiles of sixteen keys
  f32x4_t own[4];
#pragma unroll
  for (int c = 0; c < 4; ++c) own[c] = f32x4_t{0.f, 0.f, 0.f, 0.f};
  for (int kt = 0; kt <= wave; ++kt) {  // scalar
    f32x4_t score = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int s = 0; s < NS; ++s) {
      if (16 * s < a.d) {  // scalar
        const f32x4_t kv = *reinterpret_cast<const f32x4_t*>(k_s + (16 * kt + li) * krow + 16 * s + 4 * lk);
#pragma unroll
        for (int i = 0; i < 4; ++i) score = __builtin_amdgcn_mfma_f32_16x16x4f32(kv[i], qv[s][i], score, 0, 0, 0);
      }
    }
    // lane holds query li, keys 4 lk + i of the tile: the operand order of the next product
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int back = query - (16 * kt + 4 * lk + i);
      score[i] = back >= 0 ? score[i] * pw[back] : 0.f;
    }
#pragma unroll
    for (int i = 0; i < 4; ++i)
#pragma unroll
      for (int c = 0; c < 4; ++c)
        own[c] = __builtin_amdgcn_mfma_f32_16x16x4f32(v_s[(16 * kt + 4 * lk + i) * kVRow + 16 * c + li], score[i], own[c], 0, 0, 0);
  }
  if (!live) return;
  const float reach = pw[query + 1];
  float* o = a.out + static_cast<int64_t>(at.t0 + query) * width + static_cast<int64_t>(h) * a.dv + c0;
#pragma unroll
  for (int c = 0; c < 4; ++c) {
    const f32x4_t y = far[c] * reach + own[c];
    const int col = 16 * c + 4 * lk;
    if (VEC) {
      if (col < cols) *reinterpret_cast<f32x4_t*>(o + col) = y;
    } else {
#pragma unroll
      for (int e = 0; e < 4; ++e)
        if (col + e < cols) o[col + e] = y[e];
    }
  }
}

size_t chunk_lds(int d) {
  return sizeof(float) * (kChunk * (((d + 15) & ~15) + kColPad) + kChunk * kVRow + kChunk + 16);
}

template <typename K>
int launch_chunks(K kernel, const ChunkArgs& a, const dim3& grid, hipStream_t stream) {
  const size_t lds = chunk_lds(a.d);
  if (lds > 64 * 1024 &&
      hipFuncSetAttribute(reinterpret_cast<const void*>(kernel), hipFuncAttributeMaxDynamicSharedMemorySize,
                          static_cast<int>(lds)) != hipSuccess)
    return kvc_fail("kvc_fixed_decay_chunks: the kernel's LDS size was refused");
  hipLaunchKernelGGL(kernel, grid, dim3(256), lds, stream, a);
  return 0;
}

}  // namespace

extern "C" int kvc_fixed_decay_chunk_tokens(void) { return kChunk; }

extern "C" int kvc_fixed_decay_chunks(float* out, const float* q, int64_t q_stride, const float* k, int64_t k_stride,
                                      const float* v, int64_t v_stride, const float* decay, float* state, float* work,
                                      int64_t work_chunks, const int32_t* positions, const int32_t* token_req,
                                      const int32_t* q_start, const int32_t* slots, int T, int R, int nh, int nqk, int d,
                                      int dv, float q_scale, int silu_in, kvc_stream stream) {
  if (T < 0 || R < 0 || nh <= 0 || nqk <= 0 || nh % nqk || d <= 0 || dv <= 0 || nh > 65535)
    return kvc_fail("kvc_fixed_decay_chunks: bad sizes");
  if (d > 256) return kvc_fail("kvc_fixed_decay_chunks: at most 256 key channels a head");
  if (q_stride < static_cast<int64_t>(nqk) * d || k_stride < static_cast<int64_t>(nqk) * d ||
      v_stride < static_cast<int64_t>(nh) * dv)
    return kvc_fail("kvc_fixed_decay_chunks: rows too short for the heads");
  if (T == 0 || R == 0) return 0;
  // every request may end in a ragged chunk
  const int64_t most = static_cast<int64_t>(T) / kChunk + R;
  const int64_t chunks = most < T ? most : T;
  if (work == nullptr || work_chunks < chunks) return kvc_fail("kvc_fixed_decay_chunks: the workspace is too small");
  if (((reinterpret_cast<uintptr_t>(state) | reinterpret_cast<uintptr_t>(work)) & 15) != 0)
    return kvc_fail("kvc_fixed_decay_chunks: state and workspace must be 16-byte aligned");
  const ChunkArgs a{out, q, q_stride, k, k_stride, v, v_stride, decay, work, state, positions, token_req, q_start,
                    slots, R, nh, nqk, d, dv, (d + 3) & ~3, q_scale, silu_in};
  const bool vec = d % 4 == 0 && dv % 4 == 0 && q_stride % 4 == 0 && k_stride % 4 == 0 && v_stride % 4 == 0 &&
                   ((reinterpret_cast<uintptr_t>(q) | reinterpret_cast<uintptr_t>(k) | reinterpret_cast<uintptr_t>(v) |
                     reinterpret_cast<uintptr_t>(out)) & 15) == 0;
  const dim3 grid(static_cast<unsigned>(chunks), nh, (dv + kCols - 1) / kCols);
  const int nm = (d + 63) / 64;  // 1 to 4
  int code = 0;
#define KVC_SUMS(NM_)                                                                          \
  code = vec ? launch_chunks(chunk_sums_kernel<NM_, 1>, a, grid, S(stream))                    \
             : launch_chunks(chunk_sums_kernel<NM_, 0>, a, grid, S(stream))
  if (nm == 1) KVC_SUMS(1);
  else if (nm == 2) KVC_SUMS(2);
  else KVC_SUMS(4);
#undef KVC_SUMS
  if (code) return code;
  const int fours = (d + 3) / 4 * dv;
  hipLaunchKernelGGL(chunk_walk_kernel, dim3(R, nh, (fours + 255) / 256), dim3(256), 0, S(stream), a);
#define KVC_RESULTS(NS_)                                                                       \
  code = vec ? launch_chunks(chunk_results_kernel<NS_, 1>, a, grid, S(stream))                 \
             : launch_chunks(chunk_results_kernel<NS_, 0>, a, grid, S(stream))
  if (d <= 16) KVC_RESULTS(1);
  else if (d <= 32) KVC_RESULTS(2);
  else if (d <= 64) KVC_RESULTS(4);
  else if (d <= 128) KVC_RESULTS(8);
  else KVC_RESULTS(16);
#undef KVC_RESULTS
  if (code) return code;
  return kvc_check_launch("kvc_fixed_decay_chunks");
}
