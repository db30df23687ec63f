// A recurrence with one constant decay a head,
//   S_t = d S_(t-1) + k_t v_t^T,  y_t = S_t^T q_t   (per head; k, q of N, v of P entries),
// over long segments that are cut into chunks of up to 64 tokens, as products on the matrix
// cores' float32 instruction (v_mfma_f32_32x32x2_f32: multiply and add in float32, none of the
// reduced-precision modes).  With i, j the places in a chunk of n tokens and S0 the state before it:
//   what the chunk leaves   A = sum_j d^(n-1-j) k_j v_j^T          (one kernel, all chunks at once)
//   the carry               S0 of the next chunk = d^n S0 + A      (a thread a number of the state)
//   its outputs             y_i = d^(i+1) S0^T q_i + sum_(j<=i) d^(i-j) (q_i . k_j) v_j   (one kernel)
// Queries and keys may be turned by the tokens' positions as they are read (the pairs of their
// first entries), keys multiplied by a number, all three passed through SiLU; and a head's
// outputs may be divided by their root mean square, weighted and gated before they are written.
// Everything is float32; only the order of the additions differs from the walk token by token.
//
// A workgroup takes one head of one chunk, the heads of a chunk are neighbours in the grid (a token's
// row is read whole at about one time; rows are thousands of entries apart).
// A wave computes 32 x 32 outputs.  Which k of a product an instruction takes is free as long as
// both operands agree: half h of a wave takes the four from 8 b + 4 h of every block of eight,
// so that an operand in LDS is read four entries (16 bytes) at a time.
#include "hal_common.h"
#include "hal_api.h"

#define DC_TOKENS 64  // of a chunk, at most
typedef __attribute__((ext_vector_type(16))) float dc_f32x16;

struct DecayRows {
  const float *v, *k, *q, *gate;  // [T] rows of heads, ld floats from one token to the next
  int ld;
  bool in_silu;
  const int* positions;
  const float *cos_t, *sin_t;  // [table_len, rot / 2]
  int rot, table_len;
  bool interleaved;
  float k_scale;
  const float* powers;  // [heads][DC_TOKENS + 1]: d^0 .. d^DC_TOKENS
  const int* chunks;    // [n][4]: first token, tokens, segment, unused
  int H, N, P;
};

// (SILU: the build for rows that may go through SiLU as they are read)
template <bool SILU>
__device__ __forceinline__ float dc_in(const DecayRows& a, float x) {
  if constexpr (SILU) return a.in_silu ? x / (1.0f + expf(-x)) : x;
  return x;
}

// A lane's 32 (or 4 NB) numbers of its column of `rows` rows, `stride` apart: those of the rows 8 b + 4 half + i
// (the last row again beyond the rows: the other operand is zero there).
template <int BLOCKS>
__device__ __forceinline__ void dc_column(const float* __restrict__ base, unsigned col, unsigned stride, int rows, int half,
                                          float (&out)[BLOCKS * 4]) {
  const unsigned first = 4 * half * stride + col, last = (rows - 1) * stride + col;
#pragma unroll
  for (int b = 0; b < BLOCKS; ++b)
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const unsigned at = first + (8 * b + i) * stride;
      out[b * 4 + i] = base[at < last ? at : last];
    }
}

// The chunk's rows of one head of k (and of q, with QUERIES) in LDS [DC_TOKENS][stride], turned, k's row j
// times scale(j); zeros beyond the tokens and between N and `width`.  A thread brings one pair (or one
// entry behind the turned ones) of every eighth row, several rows' loads on their way at a time.
template <bool QUERIES, bool SILU, typename F>
__device__ __forceinline__ void dc_stage(const DecayRows& a, int t0, int n, int h, float* ks, float* qs, int stride, int width,
                                         F scale) {
  constexpr int PASS = 8, AT_ONCE = 4;  // rows side by side (256 threads, 32 to a row), passes whose loads are in flight
  const int pairs = a.rot / 2, per = width - pairs, j0 = threadIdx.x / 32;
  const int pos0 = a.rot > 0 ? a.positions[t0] : 0;  // (a segment's positions follow one another)
  const size_t head = (size_t)t0 * a.ld + (size_t)h * a.N;
  for (int i = threadIdx.x % 32; i < per; i += 32) {
    const bool pair = i < pairs;
    const int ia = pair ? (a.interleaved ? 2 * i : i) : i + pairs;
    const int ib = pair ? (a.interleaved ? 2 * i + 1 : i + pairs) : ia;
    const bool there = ia < a.N;
#pragma unroll
    for (int p = 0; p < DC_TOKENS / PASS; p += AT_ONCE) {
      float ka[AT_ONCE], kb[AT_ONCE], qa[AT_ONCE], qb[AT_ONCE], c[AT_ONCE], s[AT_ONCE];
#pragma unroll
      for (int u = 0; u < AT_ONCE; ++u) {
        const int j = j0 + (p + u) * PASS;
        const bool have = there && j < n;
        const float* kr = a.k + head + (size_t)j * a.ld;
        ka[u] = have ? kr[ia] : 0.f;
        kb[u] = have && pair ? kr[ib] : 0.f;
        if (QUERIES) {
          const float* qr = a.q + head + (size_t)j * a.ld;
          qa[u] = have ? qr[ia] : 0.f;
          qb[u] = have && pair ? qr[ib] : 0.f;
        }
        c[u] = 1.f, s[u] = 0.f;
        if (have && pair) {
          const int pos = pos0 + j;
          const bool known = pos >= 0 && pos < a.table_len;  // checked on the host; else the row shows it
          c[u] = known ? a.cos_t[(size_t)pos * pairs + i] : NAN, s[u] = known ? a.sin_t[(size_t)pos * pairs + i] : NAN;
        }
      }
#pragma unroll
      for (int u = 0; u < AT_ONCE; ++u) {
        const int j = j0 + (p + u) * PASS;
        const float m = j < n ? scale(j) : 0.f, x = dc_in<SILU>(a, ka[u]), y = dc_in<SILU>(a, kb[u]);
        ks[j * stride + ia] = (x * c[u] - y * s[u]) * m;
        if (pair) ks[j * stride + ib] = (y * c[u] + x * s[u]) * m;
        if (QUERIES) {
          const float z = dc_in<SILU>(a, qa[u]), w = dc_in<SILU>(a, qb[u]);
          qs[j * stride + ia] = z * c[u] - w * s[u];
          if (pair) qs[j * stride + ib] = w * c[u] + z * s[u];
        }
      }
    }
  }
}

template <typename T>
__device__ __forceinline__ T dc_out(float y);
template <>
__device__ __forceinline__ float dc_out<float>(float y) { return y; }
template <>
__device__ __forceinline__ bf16_t dc_out<bf16_t>(float y) { return bf16_t{(uint16_t)pack_bf16x2(y, 0.f)}; }

__device__ __forceinline__ int dc_row(int v, int half) { return 8 * (v / 4) + 4 * half + v % 4; }  // of register v

// ---- what every chunk leaves from a zero state: sums [chunk][head][N][P], and d^n ------------------
template <bool SILU>
__global__ void __launch_bounds__(256, 3)
decay_sums_kernel(DecayRows a, float* __restrict__ sums, float* __restrict__ decays, int stride) {
  extern __shared__ float dc_lds[];
  __shared__ float pw[DC_TOKENS + 1];
  float* ks = dc_lds;  // [DC_TOKENS][stride]
  const int h = blockIdx.x, c = blockIdx.y, tid = threadIdx.x, lane = tid % HAL_WAVE, wave = tid / HAL_WAVE;
  const int half = lane / 32, l32 = lane % 32;
  const int t0 = a.chunks[c * 4], n = a.chunks[c * 4 + 1];
  if (n <= 0) return;
  if (tid <= DC_TOKENS) pw[tid] = a.powers[(size_t)h * (DC_TOKENS + 1) + tid];
  const int row_tiles = (a.N + 31) / 32, col_tiles = (a.P + 31) / 32;
  // a wave takes a tile of 32 columns and the tiles of 32 rows in turn (few columns: the waves share one)
  const int across = col_tiles >= 4 ? 4 : (col_tiles >= 2 ? 2 : 1), down = 4 / across;
  const int ct0 = wave % across + across * blockIdx.z;
  float vr[DC_TOKENS / 2];
  const float* vbase = a.v + (size_t)t0 * a.ld + (size_t)h * a.P;
  auto values = [&](int ct) {
    const int col = ct * 32 + l32;
    dc_column<DC_TOKENS / 8>(vbase, col < a.P ? col : a.P - 1, a.ld, n, half, vr);
  };
  values(ct0);
  __syncthreads();
  dc_stage<false, SILU>(a, t0, n, h, ks, nullptr, stride, row_tiles * 32, [&](int j) { return a.k_scale * pw[n - 1 - j]; });
  if (blockIdx.z == 0 && tid == 0) decays[(size_t)c * a.H + h] = pw[n];
  __syncthreads();
  float* out = sums + ((size_t)c * a.H + h) * a.N * a.P;
  for (int ct = ct0; ct < col_tiles; ct += across * gridDim.z) {
    const int col = ct * 32 + l32;
    if (ct != ct0) values(ct);
#pragma unroll
    for (int i = 0; i < DC_TOKENS / 2; ++i) vr[i] = dc_in<SILU>(a, vr[i]);
    for (int rt = wave / across; rt < row_tiles; rt += down) {
      dc_f32x16 acc = {};
#pragma unroll
      for (int b = 0; b < DC_TOKENS / 8; ++b)
#pragma unroll
        for (int i = 0; i < 4; ++i)
          acc = __builtin_amdgcn_mfma_f32_32x32x2f32(ks[(8 * b + 4 * half + i) * stride + rt * 32 + l32], vr[b * 4 + i], acc, 0, 0, 0);
#pragma unroll
      for (int v = 0; v < 16; ++v) {
        const int row = rt * 32 + dc_row(v, half);
        if (row < a.N && col < a.P) out[(size_t)row * a.P + col] = acc[v];
      }
    }
  }
}

// ---- the outputs of every chunk from the state it starts from (`starts`, as the carry left it) -------
// NB: blocks of eight entries of a key, at most; CT: column tiles a wave.  GATED: normed, weighted and
// gated rows of T; else float32 rows as they are (and the rows read may go through SiLU).
template <int NB, int CT, bool GATED, typename T>
__global__ void __launch_bounds__(256, CT == 1 && NB < 16 ? 3 : 2)
decay_outputs_kernel(DecayRows a, const float* __restrict__ starts, const void* __restrict__ w, int w_dtype, bool silu,
                     float eps, T* __restrict__ out) {
  extern __shared__ float dc_lds[];
  __shared__ float pw[DC_TOKENS + 1];
  __shared__ float part[2][DC_TOKENS], rstd[DC_TOKENS];
  constexpr int LD = NB * 8 + 4, LP = DC_TOKENS + 4;
  constexpr bool SILU = !GATED;
  float* qs = dc_lds;                   // [DC_TOKENS][LD]
  float* ks = dc_lds + DC_TOKENS * LD;  // [DC_TOKENS][LD], then the scores [DC_TOKENS][LP]
  const int h = blockIdx.x, c = blockIdx.y, tid = threadIdx.x, lane = tid % HAL_WAVE, wave = tid / HAL_WAVE;
  const int half = lane / 32, l32 = lane % 32;
  const int t0 = a.chunks[c * 4], n = a.chunks[c * 4 + 1];
  if (n <= 0) return;
  if (tid <= DC_TOKENS) pw[tid] = a.powers[(size_t)h * (DC_TOKENS + 1) + tid];
  const int rt = wave % 2, side = wave / 2;  // a wave's tile of 32 rows, and which half of the columns
  // the state's and the values' entries of a wave's column, asked for long before they are needed
  const float* S0 = starts + ((size_t)c * a.H + h) * a.N * a.P;
  float s0[NB * 4], vr[DC_TOKENS / 2];
  auto column = [&](int u) {
    const int col = (side + 2 * u) * 32 + l32;
    return col < a.P ? col : a.P - 1;
  };
  auto ask_state = [&](int u) { dc_column<NB>(S0, column(u), a.P, a.N, half, s0); };
  const float* vbase = a.v + (size_t)t0 * a.ld + (size_t)h * a.P;
  auto ask_values = [&](int u) { dc_column<DC_TOKENS / 8>(vbase, column(u), a.ld, n, half, vr); };
  ask_state(0);
  dc_stage<true, SILU>(a, t0, n, h, ks, qs, LD, NB * 8, [&](int) { return a.k_scale; });
  __syncthreads();
  ask_values(0);
  dc_f32x16 acc[CT];
#pragma unroll
  for (int u = 0; u < CT; ++u) {  // what the queries read of the state before the chunk
    acc[u] = dc_f32x16{};
    if ((side + 2 * u) * 32 >= a.P) continue;
    if (u > 0) ask_state(u);
    const float* qr = qs + (rt * 32 + l32) * LD + 4 * half;
#pragma unroll
    for (int b = 0; b < NB; ++b) {
      const float4 x = *(const float4*)(qr + 8 * b);
      acc[u] = __builtin_amdgcn_mfma_f32_32x32x2f32(x.x, s0[b * 4], acc[u], 0, 0, 0);
      acc[u] = __builtin_amdgcn_mfma_f32_32x32x2f32(x.y, s0[b * 4 + 1], acc[u], 0, 0, 0);
      acc[u] = __builtin_amdgcn_mfma_f32_32x32x2f32(x.z, s0[b * 4 + 2], acc[u], 0, 0, 0);
      acc[u] = __builtin_amdgcn_mfma_f32_32x32x2f32(x.w, s0[b * 4 + 3], acc[u], 0, 0, 0);
    }
#pragma unroll
    for (int v = 0; v < 16; ++v) acc[u][v] *= pw[rt * 32 + dc_row(v, half) + 1];
  }
  // scores: wave 0 the tile (0, 0), wave 1 (1, 0), wave 3 (1, 1); (0, 1) lies behind every query
  dc_f32x16 sc = {};
  const bool scores = wave != 2;
  if (scores) {
    const float* qr = qs + (rt * 32 + l32) * LD + 4 * half;
    const float* kr = ks + (side * 32 + l32) * LD + 4 * half;
#pragma unroll
    for (int b = 0; b < NB; ++b) {
      const float4 x = *(const float4*)(qr + 8 * b), y = *(const float4*)(kr + 8 * b);
      sc = __builtin_amdgcn_mfma_f32_32x32x2f32(x.x, y.x, sc, 0, 0, 0);
      sc = __builtin_amdgcn_mfma_f32_32x32x2f32(x.y, y.y, sc, 0, 0, 0);
      sc = __builtin_amdgcn_mfma_f32_32x32x2f32(x.z, y.z, sc, 0, 0, 0);
      sc = __builtin_amdgcn_mfma_f32_32x32x2f32(x.w, y.w, sc, 0, 0, 0);
    }
  }
  __syncthreads();  // the keys are read
  float* ps = ks;
  if (scores) {
#pragma unroll
    for (int v = 0; v < 16; ++v) {
      const int i = rt * 32 + dc_row(v, half), j = side * 32 + l32;
      ps[i * LP + j] = i >= j ? sc[v] * pw[i - j] : 0.f;
    }
  }
  __syncthreads();
#pragma unroll
  for (int u = 0; u < CT; ++u) {  // the chunk's own values by the scores
    if ((side + 2 * u) * 32 >= a.P) continue;
    if (u > 0) ask_values(u);
    const float* pr = ps + (rt * 32 + l32) * LP + 4 * half;
    auto weigh = [&](int b) {
      const float4 x = *(const float4*)(pr + 8 * b);
      acc[u] = __builtin_amdgcn_mfma_f32_32x32x2f32(x.x, dc_in<SILU>(a, vr[b * 4]), acc[u], 0, 0, 0);
      acc[u] = __builtin_amdgcn_mfma_f32_32x32x2f32(x.y, dc_in<SILU>(a, vr[b * 4 + 1]), acc[u], 0, 0, 0);
      acc[u] = __builtin_amdgcn_mfma_f32_32x32x2f32(x.z, dc_in<SILU>(a, vr[b * 4 + 2]), acc[u], 0, 0, 0);
      acc[u] = __builtin_amdgcn_mfma_f32_32x32x2f32(x.w, dc_in<SILU>(a, vr[b * 4 + 3]), acc[u], 0, 0, 0);
    };
#pragma unroll
    for (int b = 0; b < 4; ++b) weigh(b);
    if (rt == 1) {
#pragma unroll
      for (int b = 4; b < 8; ++b) weigh(b);
    }
  }
  if constexpr (GATED) {
    // every row's sum of squares over the head's columns: the 32 lanes of a half hold a row's columns in
    // register v; halving the registers at every exchange leaves a lane one row
    float r[16];
#pragma unroll
    for (int v = 0; v < 16; ++v) {
      r[v] = 0.f;
#pragma unroll
      for (int u = 0; u < CT; ++u)
        if ((side + 2 * u) * 32 + l32 < a.P) r[v] = fmaf(acc[u][v], acc[u][v], r[v]);
    }
#pragma unroll
    for (int k = 8; k >= 1; k >>= 1) {
      const int m = 2 * k;
      const bool up = (lane & m) != 0;
#pragma unroll
      for (int i = 0; i < 8; ++i) {
        if (i >= k) break;
        const float keep = up ? r[i + k] : r[i], give = up ? r[i] : r[i + k];
        r[i] = keep + __shfl_xor(give, m, HAL_WAVE);
      }
    }
    r[0] += __shfl_xor(r[0], 1, HAL_WAVE);
    if (lane % 2 == 0) part[side][rt * 32 + dc_row(l32 / 2, half)] = r[0];
    __syncthreads();
    if (tid < DC_TOKENS) rstd[tid] = 1.0f / sqrtf((part[0][tid] + part[1][tid]) / (float)a.P + eps);
    __syncthreads();
  }
  const size_t head = (size_t)t0 * a.H * a.P + (size_t)h * a.P;
  const float* gbase = GATED ? a.gate + (size_t)t0 * a.ld + (size_t)h * a.P : nullptr;
#pragma unroll
  for (int u = 0; u < CT; ++u) {
    const int col = (side + 2 * u) * 32 + l32;
    if (col >= a.P) continue;
    if constexpr (GATED) {
      const float wt = w ? load_as_f32(w, w_dtype, (size_t)h * a.P + col) : 1.0f;
      float z[16];
      const unsigned first = (rt * 32 + 4 * half) * a.ld + col, last = (n - 1) * a.ld + col;
#pragma unroll
      for (int v = 0; v < 16; ++v) {
        const unsigned at = first + (8 * (v / 4) + v % 4) * a.ld;
        z[v] = gbase[at < last ? at : last];
      }
#pragma unroll
      for (int v = 0; v < 16; ++v) {
        // (one rounding of the reciprocal more or less: it is 1 + something)
        const float s = __builtin_amdgcn_rcpf(1.0f + expf(-z[v]));
        acc[u][v] *= rstd[rt * 32 + dc_row(v, half)] * wt * (silu ? z[v] * s : s);
      }
    }
    T* o = out + head + col;
#pragma unroll
    for (int v = 0; v < 16; ++v) {
      const int i = rt * 32 + dc_row(v, half);
      if (i < n) o[(unsigned)i * (unsigned)(a.H * a.P)] = dc_out<T>(acc[u][v]);
    }
  }
}

template <int NB, int CT, bool GATED, typename T>
static int dc_outputs(const DecayRows& a, int n_chunks, const float* starts, const void* w, int w_dtype, bool silu, float eps,
                      void* out, hipStream_t stream) {
  constexpr int LD = NB * 8 + 4, LP = DC_TOKENS + 4;
  const size_t smem = sizeof(float) * DC_TOKENS * (LD + (LD > LP ? LD : LP));
  if (smem > 48 * 1024)
    HAL_CHECK_HIP(hipFuncSetAttribute((const void*)decay_outputs_kernel<NB, CT, GATED, T>,
                                      hipFuncAttributeMaxDynamicSharedMemorySize, (int)smem));
  hipLaunchKernelGGL((decay_outputs_kernel<NB, CT, GATED, T>), dim3(a.H, n_chunks), dim3(256), smem, stream, a, starts, w,
                     w_dtype, silu, eps, (T*)out);
  HAL_LAUNCH_CHECK();
  return 0;
}

template <bool GATED, typename T>
static int dc_outputs_by_size(const DecayRows& a, int n_chunks, const float* starts, const void* w, int w_dtype, bool silu,
                              float eps, void* out, hipStream_t stream) {
#define DC_COLS(NB_)                                                                                               \
  do {                                                                                                             \
    if (a.P <= 64) return dc_outputs<NB_, 1, GATED, T>(a, n_chunks, starts, w, w_dtype, silu, eps, out, stream);    \
    if (a.P <= 128) return dc_outputs<NB_, 2, GATED, T>(a, n_chunks, starts, w, w_dtype, silu, eps, out, stream);   \
    return dc_outputs<NB_, 4, GATED, T>(a, n_chunks, starts, w, w_dtype, silu, eps, out, stream);                   \
  } while (0)
  if (a.N <= 32) DC_COLS(4);
  if (a.N <= 64) DC_COLS(8);
  DC_COLS(16);
#undef DC_COLS
}

extern "C" int hal_decay_chunks(const float* v, const float* k, const float* q, const float* gate, int ld, int in_silu,
                                const int* positions, const float* cos_t, const float* sin_t, int rot, int table_len,
                                int interleaved, float k_scale, const float* powers, float* state, const int* seg_q_start,
                                const int* seg_q_len, const int* token_slot, const int* chunks, const int* seg_chunks,
                                int n_chunks, float* sums, float* decays, const void* w, int w_dtype, int silu, float eps,
                                void* out, int dtype, int n_segs, int H, int N, int P, hipStream_t stream) {
  HAL_REQUIRE(n_segs >= 0 && n_chunks >= 0 && H > 0 && H <= 65535 && N > 0 && N <= 128 && P > 0 && P <= 256,
              "hal_decay_chunks: bad sizes segments=%d chunks=%d heads=%d state %d x %d", n_segs, n_chunks, H, N, P);
  HAL_REQUIRE(ld >= H * P && ld >= H * N && v && k && q && powers && state && chunks && seg_chunks && sums && decays,
              "hal_decay_chunks: arguments");
  HAL_REQUIRE(rot >= 0 && rot % 2 == 0 && rot <= N && (rot == 0 || (cos_t && sin_t && positions && table_len > 0)),
              "hal_decay_chunks: %d turned entries of %d", rot, N);
  HAL_REQUIRE((dtype == HAL_F32 || dtype == HAL_BF16) && (gate ? !in_silu : dtype == HAL_F32) &&
                  (w == nullptr || w_dtype == HAL_F32 || w_dtype == HAL_BF16),
              "hal_decay_chunks: dtypes %d, %d", dtype, w_dtype);
  HAL_REQUIRE(n_chunks <= 65535, "hal_decay_chunks: %d chunks exceed the grid limit", n_chunks);
  if (n_segs == 0 || n_chunks == 0) return 0;
  const DecayRows a = {v, k, q, gate, ld, in_silu != 0, positions, cos_t, sin_t, rot, table_len, interleaved != 0,
                       k_scale, powers, chunks, H, N, P};
  const int stride = (N + 31) / 32 * 32 + 8, col_tiles = (P + 31) / 32;
  int z = 1;  // few chunks and heads: the columns of a state are shared by several workgroups
  while (z < 4 && (long long)n_chunks * H * z < 512 && z * 4 < col_tiles) z *= 2;
  if (in_silu)
    hipLaunchKernelGGL(decay_sums_kernel<true>, dim3(H, n_chunks, z), dim3(256), sizeof(float) * DC_TOKENS * stride, stream, a,
                       sums, decays, stride);
  else
    hipLaunchKernelGGL(decay_sums_kernel<false>, dim3(H, n_chunks, z), dim3(256), sizeof(float) * DC_TOKENS * stride, stream, a,
                       sums, decays, stride);
  HAL_LAUNCH_CHECK();
  if (int rc = hal_ssd_carry(state, sums, decays, seg_chunks, seg_q_start, seg_q_len, token_slot, n_segs, H, N * P, stream))
    return rc;
  if (!gate) return dc_outputs_by_size<false, float>(a, n_chunks, sums, w, w_dtype, silu != 0, eps, out, stream);
  if (dtype == HAL_F32) return dc_outputs_by_size<true, float>(a, n_chunks, sums, w, w_dtype, silu != 0, eps, out, stream);
  return dc_outputs_by_size<true, bf16_t>(a, n_chunks, sums, w, w_dtype, silu != 0, eps, out, stream);
}
