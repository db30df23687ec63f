// Time mixing: a recurrence with a matrix state per head, a decay per key channel that is made
// from the token, and a bonus for the current token alone,
//
//   o_t = (S_(t-1) + diag(u) k_t v_t^T)^T r_t,   S_t = diag(w_t) S_(t-1) + k_t v_t^T,
//   w = exp(-exp(w0 + W2 tanh(x1))),
//
// whose projections read the token's row mixed with the row before it (the token shift).  The
// states (float32) and the last row of every request live in rows, one per request slot; a step's
// tokens come as a flat batch of segments, as for the other recurrences.  Everything here is
// float32 whatever the activations' type is.
#include "hal_common.h"
#include "hal_api.h"

#define WKV_MAX_RANK 1024

// ---- the token shift: a workgroup a token; N rows at a time from two ------------------------
// mu [n_mixes][W]; `last` [slots][W]: the row before the step's first token of every request
template <typename T, int V>
__global__ void token_shift_kernel(const T* __restrict__ x, const void* __restrict__ mu, int mu_dtype, int n_mixes,
                                   float* __restrict__ last, const int* __restrict__ token_seg,
                                   const int* __restrict__ seg_q_start, const int* __restrict__ token_slot, bool single,
                                   T* __restrict__ out, long long mix_stride, int row_stride, T* __restrict__ out_last,
                                   int W) {
  const size_t t = blockIdx.x;
  const bool first = single || (int)t == seg_q_start[token_seg[t]];
  float* before = last + (size_t)token_slot[t] * W;
  for (int c = (blockIdx.y * blockDim.x + threadIdx.x) * V; c < W; c += gridDim.y * blockDim.x * V) {
    float h[V], d[V];
    if constexpr (V == 4) {
      float p[4];
      load4(x + t * W + c, h);
      if (first) load4(before + c, p);
      else load4(x + (t - 1) * W + c, p);
      if (single) store4(before + c, h);
#pragma unroll
      for (int i = 0; i < 4; ++i) d[i] = p[i] - h[i];
    } else {
      h[0] = to_f32(x[t * W + c]);
      d[0] = (first ? before[c] : to_f32(x[(t - 1) * W + c])) - h[0];
      if (single) before[c] = h[0];
    }
    for (int s = 0; s < n_mixes; ++s) {
      T* o = s == n_mixes - 1 ? out_last + t * W + c : out + s * mix_stride + t * row_stride + c;
      if constexpr (V == 4) {
        float m[4], y[4];
        load4_any(mu, mu_dtype, (size_t)s * W + c, m);
#pragma unroll
        for (int i = 0; i < 4; ++i) y[i] = fmaf(d[i], m[i], h[i]);
        store4(o, y);
      } else {
        *o = from_f32<T>(fmaf(d[0], load_as_f32(mu, mu_dtype, (size_t)s * W + c), h[0]));
      }
    }
  }
}

extern "C" int hal_token_shift(const void* x, int dtype, const void* mu, int mu_dtype, int n_mixes, float* last,
                               const int* token_seg, const int* seg_q_start, const int* token_slot, int single, void* out,
                               long long mix_stride, int row_stride, void* out_last, int n_tokens, int W,
                               hipStream_t stream) {
  HAL_REQUIRE(n_tokens >= 0 && W > 0 && n_mixes > 0 && row_stride >= W && mix_stride >= W,
              "hal_token_shift: bad sizes T=%d W=%d mixes=%d", n_tokens, W, n_mixes);
  HAL_REQUIRE((dtype == HAL_F32 || dtype == HAL_BF16) && (mu_dtype == HAL_F32 || mu_dtype == HAL_BF16),
              "hal_token_shift: dtypes %d, %d", dtype, mu_dtype);
  if (n_tokens == 0) return 0;
  const bool vec = W % 4 == 0 && row_stride % 4 == 0 && mix_stride % 4 == 0 && ((uintptr_t)x % 16) == 0 &&
                   ((uintptr_t)out % 16) == 0 && ((uintptr_t)out_last % 16) == 0 && ((uintptr_t)mu % 16) == 0 &&
                   ((uintptr_t)last % 16) == 0;
  const int per = vec ? 1024 : 256;
  const dim3 grid(n_tokens, n_tokens <= 64 ? (W + per - 1) / per : 1);
#define SHIFT_LAUNCH(T_, V_)                                                                                           \
  hipLaunchKernelGGL((token_shift_kernel<T_, V_>), grid, dim3(256), 0, stream, (const T_*)x, mu, mu_dtype, n_mixes, last, \
                     token_seg, seg_q_start, token_slot, single != 0, (T_*)out, mix_stride, row_stride, (T_*)out_last, W)
  if (dtype == HAL_F32) {
    if (vec) SHIFT_LAUNCH(float, 4);
    else SHIFT_LAUNCH(float, 1);
  } else {
    if (vec) SHIFT_LAUNCH(bf16_t, 4);
    else SHIFT_LAUNCH(bf16_t, 1);
  }
#undef SHIFT_LAUNCH
  HAL_LAUNCH_CHECK();
  return 0;
}

template <typename T>
__global__ void carry_rows_kernel(const T* __restrict__ x, float* __restrict__ last, const int* __restrict__ seg_q_start,
                                  const int* __restrict__ seg_q_len, const int* __restrict__ token_slot, int W) {
  const int s = blockIdx.x, n = seg_q_len[s];
  if (n <= 0) return;
  const size_t t = (size_t)seg_q_start[s] + n - 1;
  float* to = last + (size_t)token_slot[t] * W;
  for (int c = blockIdx.y * blockDim.x + threadIdx.x; c < W; c += gridDim.y * blockDim.x) to[c] = to_f32(x[t * W + c]);
}

extern "C" int hal_carry_rows(const void* x, int dtype, float* last, const int* seg_q_start, const int* seg_q_len,
                              const int* token_slot, int n_segs, int W, hipStream_t stream) {
  HAL_REQUIRE(n_segs >= 0 && W > 0, "hal_carry_rows: bad sizes segments=%d W=%d", n_segs, W);
  HAL_REQUIRE(dtype == HAL_F32 || dtype == HAL_BF16, "hal_carry_rows: dtype %d", dtype);
  if (n_segs == 0) return 0;
  const dim3 grid(n_segs, (W + 255) / 256 < 16 ? (W + 255) / 256 : 16);
  if (dtype == HAL_F32)
    hipLaunchKernelGGL(carry_rows_kernel<float>, grid, dim3(256), 0, stream, (const float*)x, last, seg_q_start, seg_q_len, token_slot, W);
  else
    hipLaunchKernelGGL(carry_rows_kernel<bf16_t>, grid, dim3(256), 0, stream, (const bf16_t*)x, last, seg_q_start, seg_q_len, token_slot, W);
  HAL_LAUNCH_CHECK();
  return 0;
}

// ---- the decays of many tokens: a thread a channel, whose row of W2 it holds in registers
// (WKV_RANK entries at a time) for the workgroup's TT tokens -------------------------------------
#define WKV_RANK 32
template <int TT, typename W>
__global__ void __launch_bounds__(256)
wkv_decay_kernel(const float* __restrict__ x1, int ldx1, const W* __restrict__ w2, const W* __restrict__ w0, int rank,
                 float* __restrict__ decay, int ldd, int n_tokens, int n) {
  __shared__ __align__(16) float tl[TT][WKV_RANK];
  const int t0 = blockIdx.x * TT;
  const int nt = n_tokens - t0 < TT ? n_tokens - t0 : TT;
  const int c = blockIdx.y * blockDim.x + threadIdx.x;
  const size_t ch = c < n ? c : n - 1;
  float z[TT];
  const float z0 = to_f32(w0[ch]);
#pragma unroll
  for (int i = 0; i < TT; ++i) z[i] = z0;
  const bool vec = rank % 4 == 0;
  for (int j0 = 0; j0 < rank; j0 += WKV_RANK) {
    const int nj = rank - j0 < WKV_RANK ? rank - j0 : WKV_RANK;
    __syncthreads();
    for (int i = threadIdx.x; i < TT * WKV_RANK; i += blockDim.x) {
      const int tok = i / WKV_RANK, j = i % WKV_RANK;
      tl[tok][j] = (tok < nt && j < nj) ? tanhf(x1[(size_t)(t0 + tok) * ldx1 + j0 + j]) : 0.f;
    }
    float w[WKV_RANK];
    const W* row = w2 + ch * rank + j0;
    if (vec && nj == WKV_RANK) {
#pragma unroll
      for (int j = 0; j < WKV_RANK; j += 4) {
        float q[4];
        load4(row + j, q);
        w[j] = q[0], w[j + 1] = q[1], w[j + 2] = q[2], w[j + 3] = q[3];
      }
    } else {
#pragma unroll
      for (int j = 0; j < WKV_RANK; ++j) w[j] = j < nj ? to_f32(row[j]) : 0.f;
    }
    __syncthreads();
#pragma unroll
    for (int i = 0; i < TT; ++i)
#pragma unroll
      for (int j = 0; j < WKV_RANK; j += 4) {
        const float4 x4 = *(const float4*)&tl[i][j];
        z[i] = fmaf(w[j], x4.x, z[i]);
        z[i] = fmaf(w[j + 1], x4.y, z[i]);
        z[i] = fmaf(w[j + 2], x4.z, z[i]);
        z[i] = fmaf(w[j + 3], x4.w, z[i]);
      }
  }
  if (c >= n) return;
#pragma unroll
  for (int i = 0; i < TT; ++i)
    if (i < nt) decay[(size_t)(t0 + i) * ldd + c] = expf(-expf(z[i]));
}

extern "C" int hal_wkv_decay(const float* x1, int ldx1, const void* w2, const void* w0, int w_dtype, int rank, float* decay,
                             int ldd, int n_tokens, int n, hipStream_t stream) {
  HAL_REQUIRE(n_tokens >= 0 && n > 0 && rank > 0 && ldx1 >= rank && ldd >= n,
              "hal_wkv_decay: bad sizes T=%d channels=%d rank=%d", n_tokens, n, rank);
  HAL_REQUIRE(w_dtype == HAL_F32 || w_dtype == HAL_BF16, "hal_wkv_decay: dtype %d", w_dtype);
  HAL_REQUIRE((n + 255) / 256 <= 65535, "hal_wkv_decay: %d channels exceed the grid limit", n);
  if (n_tokens == 0) return 0;
#define DECAY_LAUNCH(TT_, W_)                                                                                       \
  hipLaunchKernelGGL((wkv_decay_kernel<TT_, W_>), dim3((n_tokens + TT_ - 1) / TT_, (n + 255) / 256), dim3(256), 0, stream, \
                     x1, ldx1, (const W_*)w2, (const W_*)w0, rank, decay, ldd, n_tokens, n)
  if (n_tokens < 256) {
    if (w_dtype == HAL_F32) DECAY_LAUNCH(1, float);
    else DECAY_LAUNCH(1, bf16_t);
  } else {
    if (w_dtype == HAL_F32) DECAY_LAUNCH(16, float);
    else DECAY_LAUNCH(16, bf16_t);
  }
#undef DECAY_LAUNCH
  HAL_LAUNCH_CHECK();
  return 0;
}

// The sum of a value over the wave's four quarters of 16 lanes, in every lane (two swaps of lane
// halves inside the vector unit).
__device__ __forceinline__ float wkv_quarters_sum(float x) {
  const unsigned b = __float_as_uint(x);
  const auto p = __builtin_amdgcn_permlane16_swap(b, b, false, false);
  const unsigned s = __float_as_uint(__uint_as_float(p[0]) + __uint_as_float(p[1]));
  const auto q = __builtin_amdgcn_permlane32_swap(s, s, false, false);
  return __uint_as_float(q[0]) + __uint_as_float(q[1]);
}

// ---- the walk: a wave takes 16 * C value channels of one head of one run of tokens.  Its four
// quarters of 16 lanes share the head's key channels (KR each), so a lane holds KR x C numbers of
// the state in registers, an LDS read of four key channels serves C columns, and the read of
// the state crosses the quarters inside the vector unit.  The tokens' decays, keys and reads go
// through LDS in blocks of TB tokens, the next block's on their way from memory meanwhile.
// MODE 0: a run is a segment, from the request's state to its next one.
// MODE 1: a run is a chunk of a segment, from nothing; what it leaves and the product of its decays
// are written.  Then a pass over every segment's chunks carries the request's state through them
// (`wkv_carry_kernel`), and MODE 2 walks the chunks again from the states they begin with. ------
template <int KR, int C, int MODE>
__global__ void __launch_bounds__(HAL_WAVE)
wkv_scan_kernel(const float* __restrict__ r, const float* __restrict__ k, const float* __restrict__ v,
                const float* __restrict__ decay, int ld, const void* __restrict__ bonus, int b_dtype,
                float* __restrict__ state, const int* __restrict__ seg_q_start, const int* __restrict__ seg_q_len,
                const int* __restrict__ token_slot, float* __restrict__ o, const int* __restrict__ chunks,
                float* __restrict__ sums, float* __restrict__ decays, int H, int D, bool vec4) {
  constexpr int DP = 4 * KR;
  constexpr int TB = DP <= 64 ? 8 : DP == 128 ? 4 : 2;
  constexpr int NV = MODE == 1 ? 2 : 3;  // decay, key, read
  constexpr int PER = TB * DP / HAL_WAVE;
  static_assert(TB * DP % HAL_WAVE == 0 && KR % 4 == 0, "a block of tokens is whole loads of the wave");
  __shared__ __align__(16) float vec[2][NV][TB * DP];
  const int s = blockIdx.x, h = blockIdx.y, lane = threadIdx.x;
  const int col = blockIdx.z * 16 * C + (lane % 16) * C, row0 = (lane / 16) * KR;
  const int t0 = MODE == 0 ? seg_q_start[s] : chunks[s * 4], n = MODE == 0 ? seg_q_len[s] : chunks[s * 4 + 1];
  if (n <= 0) return;
  const size_t hd = (size_t)h * D;
  float* st = (MODE == 0 ? state + ((size_t)token_slot[t0] * H + h) * D * D : sums + ((size_t)s * H + h) * D * D) + col;
  float S[KR][C];
  float u[KR], prod[KR];
#pragma unroll
  for (int j = 0; j < KR; ++j) {
#pragma unroll
    for (int i = 0; i < C; ++i) S[j][i] = (MODE != 1 && row0 + j < D && col + i < D) ? st[(size_t)(row0 + j) * D + i] : 0.f;
    u[j] = (MODE != 1 && row0 + j < D) ? load_as_f32(bonus, b_dtype, hd + row0 + j) : 0.f;
    prod[j] = 1.f;
  }
  // where this lane's loads of a block lie from the block's first token on (channels beyond D: zero)
  int at[PER], tok[PER];
  bool in[PER];
#pragma unroll
  for (int x = 0; x < PER; ++x) {
    const int i = lane + x * HAL_WAVE, c = i % DP;
    tok[x] = i / DP;
    in[x] = c < D;
    at[x] = tok[x] * ld + (in[x] ? c : 0);
  }
  float next[NV][PER], v_next[TB][C];
  const bool whole = vec4 && C == 4 && col + C <= D;
  auto ask = [&](int t, int cnt) {  // tokens t .. t + cnt - 1
    const size_t from = (size_t)t * ld + hd;
#pragma unroll
    for (int x = 0; x < PER; ++x) {
      const bool have = in[x] && tok[x] < cnt;
      next[0][x] = have ? decay[from + at[x]] : 0.f;
      next[1][x] = have ? k[from + at[x]] : 0.f;
      if (MODE != 1) next[NV - 1][x] = have ? r[from + at[x]] : 0.f;
    }
#pragma unroll
    for (int j = 0; j < TB; ++j) {
      const float* vp = v + from + (size_t)j * ld + col;
      if constexpr (C == 4) {
        float q[4] = {0.f, 0.f, 0.f, 0.f};
        if (j < cnt) {
          if (whole) load4(vp, q);
          else {
#pragma unroll
            for (int i = 0; i < C; ++i)
              if (col + i < D) q[i] = vp[i];
          }
        }
#pragma unroll
        for (int i = 0; i < C; ++i) v_next[j][i] = q[i];
      } else {
#pragma unroll
        for (int i = 0; i < C; ++i) v_next[j][i] = (j < cnt && col + i < D) ? vp[i] : 0.f;
      }
    }
  };
  float* op = o + (size_t)t0 * H * D + hd + col;
  auto token = [&](int b, int jt, const float (&val)[C]) {
    float acc[C];
#pragma unroll
    for (int i = 0; i < C; ++i) acc[i] = 0.f;
    float own = 0.f;  // r . (u * k), this quarter's part
#pragma unroll
    for (int j4 = 0; j4 < KR; j4 += 4) {
      const float4 w4 = *(const float4*)&vec[b][0][jt * DP + row0 + j4];
      const float4 k4 = *(const float4*)&vec[b][1][jt * DP + row0 + j4];
      const float wj[4] = {w4.x, w4.y, w4.z, w4.w}, kj[4] = {k4.x, k4.y, k4.z, k4.w};
      float rj[4] = {0.f, 0.f, 0.f, 0.f};
      if (MODE != 1) {
        const float4 r4 = *(const float4*)&vec[b][NV - 1][jt * DP + row0 + j4];
        rj[0] = r4.x, rj[1] = r4.y, rj[2] = r4.z, rj[3] = r4.w;
      }
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        const int j = j4 + e;
        if (MODE != 1) own = fmaf(rj[e] * u[j], kj[e], own);
        else prod[j] *= wj[e];
#pragma unroll
        for (int i = 0; i < C; ++i) {
          if (MODE != 1) acc[i] = fmaf(rj[e], S[j][i], acc[i]);
          S[j][i] = fmaf(wj[e], S[j][i], kj[e] * val[i]);
        }
      }
    }
    if (MODE != 1) {
#pragma unroll
      for (int i = 0; i < C; ++i) acc[i] = wkv_quarters_sum(fmaf(own, val[i], acc[i]));
      if (lane < 16) {
        if (C == 4 && whole) {
          *(float4*)op = make_float4(acc[0], acc[1 % C], acc[2 % C], acc[3 % C]);
        } else {
#pragma unroll
          for (int i = 0; i < C; ++i)
            if (col + i < D) op[i] = acc[i];
        }
      }
      op += (size_t)H * D;
    }
  };
  ask(t0, n < TB ? n : TB);
  for (int b = 0; b * TB < n; ++b) {
    const int left = n - b * TB, buf = b & 1;
#pragma unroll
    for (int w = 0; w < NV; ++w)
#pragma unroll
      for (int x = 0; x < PER; ++x) vec[buf][w][lane + x * HAL_WAVE] = next[w][x];
    float vv[TB][C];
#pragma unroll
    for (int j = 0; j < TB; ++j)
#pragma unroll
      for (int i = 0; i < C; ++i) vv[j][i] = v_next[j][i];
    if (left > TB) ask(t0 + (b + 1) * TB, left - TB < TB ? left - TB : TB);
    __builtin_amdgcn_fence(__ATOMIC_RELEASE, "wavefront");
    __builtin_amdgcn_wave_barrier();
    __builtin_amdgcn_fence(__ATOMIC_ACQUIRE, "wavefront");
    if (left >= TB) {
#pragma unroll
      for (int jt = 0; jt < TB; ++jt) token(buf, jt, vv[jt]);
    } else {
#pragma unroll
      for (int jt = 0; jt < TB; ++jt)
        if (jt < left) token(buf, jt, vv[jt]);
    }
  }
  if (MODE != 2) {
#pragma unroll
    for (int j = 0; j < KR; ++j)
#pragma unroll
      for (int i = 0; i < C; ++i)
        if (row0 + j < D && col + i < D) st[(size_t)(row0 + j) * D + i] = S[j][i];
  }
  if (MODE == 1 && blockIdx.z == 0 && lane % 16 == 0) {
#pragma unroll
    for (int j = 0; j < KR; ++j)
      if (row0 + j < D) decays[(size_t)s * H * D + hd + row0 + j] = prod[j];
  }
}

// A thread takes one number of the state of one head of one segment through the segment's chunks:
// every chunk's sums become the state it begins with; four chunks are asked for at a time.
__global__ void __launch_bounds__(256)
wkv_carry_kernel(float* __restrict__ state, float* __restrict__ sums, const float* __restrict__ decays,
                 const int* __restrict__ seg_chunks, const int* __restrict__ seg_q_start,
                 const int* __restrict__ seg_q_len, const int* __restrict__ token_slot, int H, int D) {
  const int s = blockIdx.x, h = blockIdx.y, e = blockIdx.z * blockDim.x + threadIdx.x;
  if (seg_q_len[s] <= 0 || e >= D * D) return;
  const int c0 = seg_chunks[s * 2], nc = seg_chunks[s * 2 + 1];
  float* st = state + ((size_t)token_slot[seg_q_start[s]] * H + h) * D * D + e;
  float S = *st;
  constexpr int AHEAD = 4;
  for (int c = c0; c < c0 + nc; c += AHEAD) {
    float left[AHEAD], decay[AHEAD];
#pragma unroll
    for (int x = 0; x < AHEAD; ++x) {
      const size_t cx = c + x < c0 + nc ? c + x : c0 + nc - 1;
      left[x] = sums[(cx * H + h) * D * D + e];
      decay[x] = decays[(cx * H + h) * D + e / D];
    }
#pragma unroll
    for (int x = 0; x < AHEAD; ++x) {
      if (c + x < c0 + nc) {
        sums[((size_t)(c + x) * H + h) * D * D + e] = S;
        S = fmaf(decay[x], S, left[x]);
      }
    }
  }
  *st = S;
}

extern "C" int hal_wkv_scan(const float* r, const float* k, const float* v, const float* decay, int ld, const void* bonus,
                            int b_dtype, float* state, const int* seg_q_start, const int* seg_q_len,
                            const int* token_slot, float* o, int n_segs, int H, int D, const int* chunks,
                            const int* seg_chunks, int n_chunks, float* sums, float* decays, hipStream_t stream) {
  HAL_REQUIRE(n_segs >= 0 && H > 0 && D > 0 && ld >= H * D, "hal_wkv_scan: bad sizes segments=%d heads=%d dim=%d rows of %d",
              n_segs, H, D, ld);
  HAL_REQUIRE(D <= 256, "hal_wkv_scan: a head of %d channels exceeds 256", D);
  HAL_REQUIRE(H <= 65535, "hal_wkv_scan: %d heads exceed the grid limit", H);
  HAL_REQUIRE(b_dtype == HAL_F32 || b_dtype == HAL_BF16, "hal_wkv_scan: dtype %d", b_dtype);
  const bool cut = chunks != nullptr;
  HAL_REQUIRE(!cut || (seg_chunks && sums && decays && n_chunks >= 0), "hal_wkv_scan: chunks without their buffers");
  if (n_segs == 0) return 0;
  const bool vec4 = D % 4 == 0 && ld % 4 == 0 && ((uintptr_t)v % 16) == 0 && ((uintptr_t)o % 16) == 0;
#define WKV_LAUNCH(KR_, C_, MODE_, RUNS_)                                                                             \
  hipLaunchKernelGGL((wkv_scan_kernel<KR_, C_, MODE_>), dim3(RUNS_, H, (D + 16 * C_ - 1) / (16 * C_)), dim3(HAL_WAVE), 0, \
                     stream, r, k, v, decay, ld, bonus, b_dtype, state, seg_q_start, seg_q_len, token_slot, o, chunks,   \
                     sums, decays, H, D, vec4)
#define WKV_STEPS(KR_, C_)                                                                                          \
  do {                                                                                                              \
    if (!cut) {                                                                                                     \
      WKV_LAUNCH(KR_, C_, 0, n_segs);                                                                               \
    } else if (n_chunks > 0) {                                                                                      \
      WKV_LAUNCH(KR_, C_, 1, n_chunks);                                                                             \
      hipLaunchKernelGGL(wkv_carry_kernel, dim3(n_segs, H, (D * D + 255) / 256), dim3(256), 0, stream, state, sums,  \
                         decays, seg_chunks, seg_q_start, seg_q_len, token_slot, H, D);                             \
      WKV_LAUNCH(KR_, C_, 2, n_chunks);                                                                             \
    }                                                                                                               \
  } while (0)
  if (D <= 16) WKV_STEPS(4, 1);
  else if (D <= 32) WKV_STEPS(8, 2);
  else if (D <= 64) WKV_STEPS(16, 4);
  else if (D <= 128) WKV_STEPS(32, 4);
  else WKV_STEPS(64, 2);
#undef WKV_STEPS
#undef WKV_LAUNCH
  HAL_LAUNCH_CHECK();
  return 0;
}

// ---- a step in which every request brings one token: a workgroup takes one head of one request.
// It starts the loads of the state (whole rows, 16 bytes a thread), makes the token's decay and
// bonus meanwhile, crosses the waves through LDS for the sum over the key channels, writes the
// state back, and finishes the head: its root mean square, weight and gate. ---------------------
template <int D, typename W, typename T>
__global__ void __launch_bounds__(D >= 32 ? 256 : 64)
wkv_step_kernel(const float* __restrict__ r, const float* __restrict__ k, const float* __restrict__ v,
                const float* __restrict__ gate, int ld, const float* __restrict__ x1, int ldx1, const W* __restrict__ w2,
                const W* __restrict__ w0, const W* __restrict__ bonus, const W* __restrict__ norm_w, int rank, float eps,
                float* __restrict__ state, const int* __restrict__ token_slot, T* __restrict__ out, int H) {
  constexpr int THREADS = D >= 32 ? 256 : 64;
  constexpr int CG = D / 4, RG = THREADS / CG, R = D / RG, WAVES = THREADS / HAL_WAVE, PARTS = THREADS / D;
  static_assert(CG <= HAL_WAVE && THREADS % CG == 0 && D % RG == 0 && R >= 1, "a head of 16, 32, 64 or 128 channels");
  __shared__ float decay_s[D], k_s[D], r_s[D];
  __shared__ float tl[WKV_MAX_RANK];
  __shared__ float zpart[PARTS][D];
  __shared__ float own_s[WAVES];
  __shared__ float4 red[WAVES][CG];
  const size_t t = blockIdx.x;
  const int h = blockIdx.y, tid = threadIdx.x;
  const int cg = tid % CG, rg = tid / CG, col = cg * 4, wave = tid / HAL_WAVE;
  float* st = state + ((size_t)token_slot[t] * H + h) * D * D + col;
  float4 S[R];
#pragma unroll
  for (int j = 0; j < R; ++j) S[j] = *(const float4*)(st + (size_t)(rg + j * RG) * D);
  const float* vr = v + t * ld + (size_t)h * D + col;
  const float4 vv = make_float4(vr[0], vr[1], vr[2], vr[3]);
  const bool channel = tid < D;
  const size_t ch = (size_t)h * D + (channel ? tid : 0);
  const float kc = channel ? k[t * ld + ch] : 0.f, rc = channel ? r[t * ld + ch] : 0.f;
  const float part = wave_sum(channel ? rc * to_f32(bonus[ch]) * kc : 0.f);
  if (tid % HAL_WAVE == 0) own_s[wave] = part;
  for (int j = tid; j < rank; j += THREADS) tl[j] = tanhf(x1[t * ldx1 + j]);
  __syncthreads();
  {  // the decay's sum over the rank, a part of it a thread: thread = (part, channel)
    const int c = tid % D, p = tid / D;
    const int per = ((rank + PARTS - 1) / PARTS + 3) & ~3, j0 = p * per;
    const int n = rank - j0 < per ? rank - j0 : per;
    const W* row = w2 + ((size_t)h * D + c) * rank + j0;
    float z0 = 0.f, z1 = 0.f;
    int j = 0;
    if (rank % 4 == 0) {
      for (; j + 4 <= n; j += 4) {
        float w[4];
        load4(row + j, w);
        z0 = fmaf(w[0], tl[j0 + j], z0);
        z1 = fmaf(w[1], tl[j0 + j + 1], z1);
        z0 = fmaf(w[2], tl[j0 + j + 2], z0);
        z1 = fmaf(w[3], tl[j0 + j + 3], z1);
      }
    }
    for (; j < n; ++j) z0 = fmaf(to_f32(row[j]), tl[j0 + j], z0);
    zpart[p][c] = z0 + z1;
  }
  __syncthreads();
  if (channel) {
    float z = to_f32(w0[ch]);
#pragma unroll
    for (int p = 0; p < PARTS; ++p) z += zpart[p][tid];
    decay_s[tid] = expf(-expf(z));
    k_s[tid] = kc;
    r_s[tid] = rc;
  }
  __syncthreads();
  float own = 0.f;
#pragma unroll
  for (int w = 0; w < WAVES; ++w) own += own_s[w];
  float4 acc = make_float4(0.f, 0.f, 0.f, 0.f);
#pragma unroll
  for (int j = 0; j < R; ++j) {
    const int row = rg + j * RG;
    const float w = decay_s[row], kr = k_s[row], rr = r_s[row];
    acc.x = fmaf(S[j].x, rr, acc.x), acc.y = fmaf(S[j].y, rr, acc.y), acc.z = fmaf(S[j].z, rr, acc.z), acc.w = fmaf(S[j].w, rr, acc.w);
    S[j].x = fmaf(w, S[j].x, kr * vv.x);
    S[j].y = fmaf(w, S[j].y, kr * vv.y);
    S[j].z = fmaf(w, S[j].z, kr * vv.z);
    S[j].w = fmaf(w, S[j].w, kr * vv.w);
    *(float4*)(st + (size_t)row * D) = S[j];
  }
#pragma unroll
  for (int m = CG; m < HAL_WAVE; m <<= 1) {
    acc.x += __shfl_xor(acc.x, m, HAL_WAVE);
    acc.y += __shfl_xor(acc.y, m, HAL_WAVE);
    acc.z += __shfl_xor(acc.z, m, HAL_WAVE);
    acc.w += __shfl_xor(acc.w, m, HAL_WAVE);
  }
  if (tid % HAL_WAVE < CG) red[wave][cg] = acc;
  __syncthreads();
  if (tid >= HAL_WAVE) return;
  // the first wave: lane group 0 holds the head's result, four channels a lane
  float4 y = make_float4(own * vv.x, own * vv.y, own * vv.z, own * vv.w);
#pragma unroll
  for (int w = 0; w < WAVES; ++w) {
    const float4 p = red[w][cg];
    y.x += p.x, y.y += p.y, y.z += p.z, y.w += p.w;
  }
  float ss = (y.x * y.x + y.y * y.y) + (y.z * y.z + y.w * y.w);
#pragma unroll
  for (int m = 1; m < CG; m <<= 1) ss += __shfl_xor(ss, m, HAL_WAVE);
  if (tid >= CG) return;
  const float rstd = 1.0f / sqrtf(ss / (float)D + eps);
  const float yv[4] = {y.x, y.y, y.z, y.w};
  const size_t c0 = (size_t)h * D + col;
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const float g = gate[t * ld + c0 + i];
    out[t * H * D + c0 + i] = from_f32<T>(yv[i] * rstd * to_f32(norm_w[c0 + i]) * (g / (1.0f + expf(-g))));
  }
}

extern "C" int hal_wkv_step(const float* r, const float* k, const float* v, const float* gate, int ld, const float* x1,
                            int ldx1, const void* w2, const void* w0, const void* bonus, const void* norm_w, int w_dtype,
                            int rank, float eps, float* state, const int* token_slot, void* out, int dtype,
                            int n_tokens, int H, int D, hipStream_t stream) {
  HAL_REQUIRE(n_tokens >= 0 && H > 0 && H <= 65535 && ld >= H * D && rank > 0 && rank <= WKV_MAX_RANK && ldx1 >= rank,
              "hal_wkv_step: bad sizes T=%d heads=%d dim=%d rank=%d", n_tokens, H, D, rank);
  HAL_REQUIRE(D == 16 || D == 32 || D == 64 || D == 128, "hal_wkv_step: a head of %d channels", D);
  HAL_REQUIRE((w_dtype == HAL_F32 || w_dtype == HAL_BF16) && (dtype == HAL_F32 || dtype == HAL_BF16),
              "hal_wkv_step: dtypes %d, %d", w_dtype, dtype);
  if (n_tokens == 0) return 0;
  const dim3 grid(n_tokens, H);
#define WKV_STEP(D_, W_, T_)                                                                                          \
  hipLaunchKernelGGL((wkv_step_kernel<D_, W_, T_>), grid, dim3(D_ >= 32 ? 256 : 64), 0, stream, r, k, v, gate, ld, x1, \
                     ldx1, (const W_*)w2, (const W_*)w0, (const W_*)bonus, (const W_*)norm_w, rank, eps, state,        \
                     token_slot, (T_*)out, H)
#define WKV_STEP_OF(W_, T_)               \
  do {                                    \
    if (D == 16) WKV_STEP(16, W_, T_);    \
    else if (D == 32) WKV_STEP(32, W_, T_); \
    else if (D == 64) WKV_STEP(64, W_, T_); \
    else WKV_STEP(128, W_, T_);           \
  } while (0)
  if (w_dtype == HAL_F32) {
    if (dtype == HAL_F32) WKV_STEP_OF(float, float);
    else WKV_STEP_OF(float, bf16_t);
  } else {
    if (dtype == HAL_F32) WKV_STEP_OF(bf16_t, float);
    else WKV_STEP_OF(bf16_t, bf16_t);
  }
#undef WKV_STEP_OF
#undef WKV_STEP
  HAL_LAUNCH_CHECK();
  return 0;
}
