// Small kernels around a latent attention and a mixture of experts.  All arithmetic is
// float32; T is the element type of activations (float or bf16).
//
//   * RMSNorm of the float32 stream with one or two weights at once (the two norms of a
//     block whose mixer and feed-forward read the same rows), x * rstd * w in float32 and
//     one rounding at the end;
//   * the step between the down projections of a latent attention and its cache: norms of
//     the query latent and of the key/value latent, and the key and value rows that the
//     paged attention kernels take;
//   * column ranges copied head by head;
//   * the router of a mixture of experts: scores, the chosen `top` (also by corrected scores and
//     among the best groups of neighbours), their weights;
//   * a counting sort of the (token, choice) pairs by expert, on the device;
//   * the weighted sum of the chosen experts' results, added into the stream.
#include "hal_common.h"
#include "hal_api.h"

// ---------------------------------------------------------------------------------
// out1[r] = T(x * rstd * w1), out2[r] = T(x * rstd * w2) with x = h[rows ? rows[r] : r]
// ---------------------------------------------------------------------------------
template <typename T>
__global__ void norm_pair_kernel(const float* __restrict__ h, const int* __restrict__ rows,
                                 const void* __restrict__ w1, const void* __restrict__ w2, int w_dtype,
                                 float eps, T* __restrict__ out1, T* __restrict__ out2, int d) {
  __shared__ float scratch[16];
  const int r = blockIdx.x;
  const float* hr = h + (size_t)(rows ? rows[r] : r) * d;
  float ss = 0.f;
  for (int i = threadIdx.x; i < d; i += blockDim.x) {
    const float x = hr[i];
    ss += x * x;
  }
  const float total = block_sum(ss, scratch);
  const float rstd = 1.0f / sqrtf(total / (float)d + eps);
  for (int i = threadIdx.x; i < d; i += blockDim.x) {
    const float x = hr[i] * rstd;
    out1[(size_t)r * d + i] = from_f32<T>(x * load_as_f32(w1, w_dtype, i));
    if (w2) out2[(size_t)r * d + i] = from_f32<T>(x * load_as_f32(w2, w_dtype, i));
  }
}

extern "C" int hal_norm_pair(const float* h, const int* rows, const void* w1, const void* w2,
                             int w_dtype, float eps, void* out1, void* out2, int dtype, int n_rows,
                             int d, hipStream_t stream) {
  HAL_REQUIRE(n_rows >= 0 && d > 0, "hal_norm_pair: bad sizes rows=%d d=%d", n_rows, d);
  HAL_REQUIRE(dtype == HAL_F32 || dtype == HAL_BF16, "hal_norm_pair: dtype %d", dtype);
  HAL_REQUIRE((w2 == nullptr) == (out2 == nullptr), "hal_norm_pair: a second weight and a second result come together");
  if (n_rows == 0) return 0;
  int threads = ((d + 3) / 4 + 63) / 64 * 64;
  if (threads > 1024) threads = 1024;
  if (dtype == HAL_F32)
    hipLaunchKernelGGL(norm_pair_kernel<float>, dim3(n_rows), dim3(threads), 0, stream, h, rows, w1, w2,
                       w_dtype, eps, (float*)out1, (float*)out2, d);
  else
    hipLaunchKernelGGL(norm_pair_kernel<bf16_t>, dim3(n_rows), dim3(threads), 0, stream, h, rows, w1,
                       w2, w_dtype, eps, (bf16_t*)out1, (bf16_t*)out2, d);
  HAL_LAUNCH_CHECK();
  return 0;
}

// ---------------------------------------------------------------------------------
// a [T, lda] float32 holds, per token, the query latent (q_rank, from column q_col0; none
// if q_rank == 0), then at kv_col0 the key/value latent (kv_rank) and the shared rotated key
// part (rot, not normed).
//   cq[t]         = T(rmsnorm(query latent) * wq)
//   k row of t    = [rotated part (not yet rotated) | T(rmsnorm(latent) * wkv) | 0 ...]   (D)
//   v row of t    = [0 ...                          | the same                 | 0 ...]   (D)
// in the packed rows `qkv` at columns k_col0 and k_col0 + D.
// ---------------------------------------------------------------------------------
template <typename T>
__global__ void latent_prep_kernel(const float* __restrict__ a, int lda, int q_col0, int q_rank,
                                   int kv_col0, int kv_rank, int rot, int D, const void* wq,
                                   const void* wkv, int w_dtype, float eps, T* __restrict__ cq,
                                   T* __restrict__ qkv, int row_stride, int k_col0) {
  __shared__ float scratch[16];
  const int t = blockIdx.x;
  const float* ar = a + (size_t)t * lda;
  if (q_rank > 0) {
    float ss = 0.f;
    for (int i = threadIdx.x; i < q_rank; i += blockDim.x) ss += ar[q_col0 + i] * ar[q_col0 + i];
    const float rstd = 1.0f / sqrtf(block_sum(ss, scratch) / (float)q_rank + eps);
    for (int i = threadIdx.x; i < q_rank; i += blockDim.x)
      cq[(size_t)t * q_rank + i] = from_f32<T>(ar[q_col0 + i] * rstd * load_as_f32(wq, w_dtype, i));
  }
  float ss = 0.f;
  for (int i = threadIdx.x; i < kv_rank; i += blockDim.x) ss += ar[kv_col0 + i] * ar[kv_col0 + i];
  const float rstd = 1.0f / sqrtf(block_sum(ss, scratch) / (float)kv_rank + eps);
  T* k = qkv + (size_t)t * row_stride + k_col0;
  T* v = k + D;
  for (int i = threadIdx.x; i < D; i += blockDim.x) {
    float kx = 0.f, vx = 0.f;
    if (i < rot) {
      kx = ar[kv_col0 + kv_rank + i];
    } else if (i < rot + kv_rank) {
      const int c = i - rot;
      // rounded once, so that keys and values hold the same number
      kx = vx = to_f32(from_f32<T>(ar[kv_col0 + c] * rstd * load_as_f32(wkv, w_dtype, c)));
    }
    k[i] = from_f32<T>(kx);
    v[i] = from_f32<T>(vx);
  }
}

extern "C" int hal_latent_prep(const float* a, int lda, int q_col0, int q_rank, int kv_col0,
                               int kv_rank, int rot, int D, const void* wq, const void* wkv,
                               int w_dtype, float eps, void* cq, void* qkv, int row_stride,
                               int k_col0, int dtype, int n_tokens, hipStream_t stream) {
  HAL_REQUIRE(n_tokens >= 0 && kv_rank > 0 && rot >= 0 && q_rank >= 0 && D >= rot + kv_rank,
              "hal_latent_prep: bad sizes T=%d q_rank=%d kv_rank=%d rot=%d D=%d", n_tokens, q_rank, kv_rank,
              rot, D);
  HAL_REQUIRE(q_col0 >= 0 && kv_col0 >= 0 && q_col0 + q_rank <= lda && kv_col0 + kv_rank + rot <= lda &&
                  k_col0 >= 0 && k_col0 + 2 * D <= row_stride,
              "hal_latent_prep: columns outside the rows");
  HAL_REQUIRE(dtype == HAL_F32 || dtype == HAL_BF16, "hal_latent_prep: dtype %d", dtype);
  if (n_tokens == 0) return 0;
  if (dtype == HAL_F32)
    hipLaunchKernelGGL(latent_prep_kernel<float>, dim3(n_tokens), dim3(256), 0, stream, a, lda, q_col0,
                       q_rank, kv_col0, kv_rank, rot, D, wq, wkv, w_dtype, eps, (float*)cq, (float*)qkv,
                       row_stride, k_col0);
  else
    hipLaunchKernelGGL(latent_prep_kernel<bf16_t>, dim3(n_tokens), dim3(256), 0, stream, a, lda, q_col0,
                       q_rank, kv_col0, kv_rank, rot, D, wq, wkv, w_dtype, eps, (bf16_t*)cq,
                       (bf16_t*)qkv, row_stride, k_col0);
  HAL_LAUNCH_CHECK();
  return 0;
}

// ---------------------------------------------------------------------------------
// y[t, h * ys + y0 + j] = x[t, h * xs + x0 + j] for j < n, and zero for the `n_zero` columns
// from h * ys + z0 on
// ---------------------------------------------------------------------------------
template <typename T>
__global__ void head_cols_kernel(const T* __restrict__ x, int ldx, int xs, int x0, T* __restrict__ y,
                                 int ldy, int ys, int y0, int n, int z0, int n_zero, int H) {
  const int t = blockIdx.x;
  const int per = n + n_zero;
  for (int e = threadIdx.x; e < H * per; e += blockDim.x) {
    const int h = e / per, j = e % per;
    if (j < n) y[(size_t)t * ldy + h * ys + y0 + j] = x[(size_t)t * ldx + h * xs + x0 + j];
    else y[(size_t)t * ldy + h * ys + z0 + (j - n)] = from_f32<T>(0.f);
  }
}

extern "C" int hal_head_cols(const void* x, int ldx, int xs, int x0, void* y, int ldy, int ys, int y0,
                             int n, int z0, int n_zero, int H, int dtype, int n_tokens,
                             hipStream_t stream) {
  HAL_REQUIRE(n_tokens >= 0 && H > 0 && n >= 0 && n_zero >= 0, "hal_head_cols: bad sizes");
  HAL_REQUIRE(x0 >= 0 && x0 + n <= xs && H * xs <= ldx && y0 >= 0 && y0 + n <= ys && z0 >= 0 &&
                  z0 + n_zero <= ys && H * ys <= ldy,
              "hal_head_cols: columns outside the rows");
  HAL_REQUIRE(dtype == HAL_F32 || dtype == HAL_BF16, "hal_head_cols: dtype %d", dtype);
  if (n_tokens == 0 || n + n_zero == 0) return 0;
  if (dtype == HAL_F32)
    hipLaunchKernelGGL(head_cols_kernel<float>, dim3(n_tokens), dim3(256), 0, stream, (const float*)x, ldx,
                       xs, x0, (float*)y, ldy, ys, y0, n, z0, n_zero, H);
  else
    hipLaunchKernelGGL(head_cols_kernel<bf16_t>, dim3(n_tokens), dim3(256), 0, stream, (const bf16_t*)x,
                       ldx, xs, x0, (bf16_t*)y, ldy, ys, y0, n, z0, n_zero, H);
  HAL_LAUNCH_CHECK();
  return 0;
}

// ---------------------------------------------------------------------------------
// x[i] *= s
// ---------------------------------------------------------------------------------
__global__ void scale_f32_kernel(float* __restrict__ x, size_t n, float s) {
  const size_t i = (size_t)blockIdx.x * blockDim.x + threadIdx.x;
  if (i < n) x[i] *= s;
}

extern "C" int hal_scale_f32(float* x, long long n, float s, hipStream_t stream) {
  HAL_REQUIRE(n >= 0, "hal_scale_f32: n=%lld", n);
  if (n == 0) return 0;
  hipLaunchKernelGGL(scale_f32_kernel, dim3((unsigned)((n + 255) / 256)), dim3(256), 0, stream, x, (size_t)n, s);
  HAL_LAUNCH_CHECK();
  return 0;
}

// ---------------------------------------------------------------------------------
#define MOE_MAX_EXPERTS 1024
// Router: z [T, E] float32 logits.  score = sigmoid(z) (or, softmax == 1, the softmax over
// the experts); the `top` largest scores (the lower index wins a tie); weights = the chosen
// scores, divided by their sum + norm_eps if `normalize`, times `scale`.  `correction` (or null)
// [E]: added to the scores for the choice alone.  `groups` > 0: the experts form so many equal
// groups of neighbours, and only experts of the `keep` groups with the largest sums of their two
// largest (corrected) scores are chosen from (the lower group wins a tie).
//
// One wave a token: lane l holds the scores of the experts l, l + 64, ... in W words (W is the
// build for so many experts: the code of a step that runs once is mostly fetched, so it is kept
// short).  A score is shown to all lanes by reading it from its lane at a uniform index.
// ---------------------------------------------------------------------------------
struct MoeChoice {
  int softmax, normalize;
  float norm_eps, scale;
  const void* correction;
  int c_dtype, groups, keep;
};
__device__ __forceinline__ float lane_value(float v, int lane) {
  return __uint_as_float(__builtin_amdgcn_readlane(__float_as_uint(v), lane));
}
// how many of the first n numbers (lane l of word w holds number w * 64 + l) come before lane's own
// ones: larger, or equal and of a lower index
template <int W>
__device__ __forceinline__ void places_before(const float (&v)[W], int n, int lane, int (&before)[W]) {
#pragma unroll
  for (int u = 0; u < W; ++u) before[u] = 0;
#pragma unroll
  for (int w = 0; w < W; ++w) {
    const int m = n - w * HAL_WAVE < HAL_WAVE ? n - w * HAL_WAVE : HAL_WAVE;
    for (int l = 0; l < m; ++l) {
      const float x = lane_value(v[w], l);
#pragma unroll
      for (int u = 0; u < W; ++u)
        before[u] += (x > v[u] || (x == v[u] && w * HAL_WAVE + l < u * HAL_WAVE + lane)) ? 1 : 0;
    }
  }
}

// The scores of experts outside the best groups become -infinity.  Lane g (word g / 64) holds what
// belongs to group g.
template <int W>
__device__ __forceinline__ void moe_close_groups(float (&s)[W], int E, int groups, int keep, int lane) {
  const int per = E / groups;
  float first[W], second[W];  // a group's two largest
#pragma unroll
  for (int u = 0; u < W; ++u) first[u] = second[u] = -INFINITY;
  int g = 0, in_group = 0;
#pragma unroll
  for (int w = 0; w < W; ++w) {
    const int m = E - w * HAL_WAVE < HAL_WAVE ? E - w * HAL_WAVE : HAL_WAVE;
    for (int l = 0; l < m; ++l) {
      const float x = lane_value(s[w], l);
#pragma unroll
      for (int u = 0; u < W; ++u)
        if (lane + u * HAL_WAVE == g) second[u] = fmaxf(second[u], fminf(first[u], x)), first[u] = fmaxf(first[u], x);
      if (++in_group == per) in_group = 0, ++g;
    }
  }
  if (per > 1) {
#pragma unroll
    for (int u = 0; u < W; ++u) first[u] += second[u];
  }
  int before[W];
  places_before<W>(first, groups, lane, before);
#pragma unroll
  for (int u = 0; u < W; ++u) {
    const int e = lane + u * HAL_WAVE, mine = e < E ? e / per : 0;
    int place = 0;
#pragma unroll
    for (int w = 0; w < W; ++w) {
      const int got = __shfl(before[w], mine % HAL_WAVE, HAL_WAVE);
      if (w == mine / HAL_WAVE) place = got;
    }
    if (place >= keep) s[u] = -INFINITY;
  }
}

template <int W>
__device__ __forceinline__ void moe_route_token(const float* __restrict__ z, int ldz, int E, int top, const MoeChoice& how,
                                                int* __restrict__ idx, float* __restrict__ wgt, int t, int lane) {
  const float* zr = z + (size_t)t * ldz;
  float s[W], w[W];  // what the choice is made by, and the scores as weights
  float zmax = -INFINITY;
#pragma unroll
  for (int u = 0; u < W; ++u) {
    const int e = lane + u * HAL_WAVE;
    s[u] = e < E ? zr[e] : -INFINITY;
    zmax = fmaxf(zmax, s[u]);
  }
  if (how.softmax) {
    zmax = wave_max(zmax);
    float part = 0.f;
#pragma unroll
    for (int u = 0; u < W; ++u) {
      w[u] = expf(s[u] - zmax);  // (0 beyond the experts)
      part += w[u];
    }
    const float denom = wave_sum(part);
#pragma unroll
    for (int u = 0; u < W; ++u) w[u] = w[u] / denom;
  } else {
#pragma unroll
    for (int u = 0; u < W; ++u) w[u] = 1.0f / (1.0f + expf(-s[u]));
  }
#pragma unroll
  for (int u = 0; u < W; ++u) {
    const int e = lane + u * HAL_WAVE;
    s[u] = w[u];
    if (how.correction && e < E) s[u] += load_as_f32(how.correction, how.c_dtype, e);
    if (e >= E || s[u] != s[u]) s[u] = -INFINITY;  // (a choice among numbers that are none is some choice)
  }
  if (how.groups > 0) moe_close_groups<W>(s, E, how.groups, how.keep, lane);
  if constexpr (W <= 2) {  // few experts: every expert's place among all
    int place[W];
    places_before<W>(s, E, lane, place);
    float part = 0.f;
#pragma unroll
    for (int u = 0; u < W; ++u) part += (lane + u * HAL_WAVE < E && place[u] < top) ? w[u] : 0.f;
    const float sum = wave_sum(part) + how.norm_eps;
#pragma unroll
    for (int u = 0; u < W; ++u) {
      if (lane + u * HAL_WAVE >= E || place[u] >= top) continue;
      idx[(size_t)t * top + place[u]] = lane + u * HAL_WAVE;
      wgt[(size_t)t * top + place[u]] = (how.normalize ? w[u] / sum : w[u]) * how.scale;
    }
  } else {  // each of the `top` rounds finds the largest that is left across the wave
    float sum = 0.f, mine[W];
    int place[W];
#pragma unroll
    for (int u = 0; u < W; ++u) place[u] = -1;
    for (int j = 0; j < top; ++j) {
      float best = -INFINITY;
      int best_e = MOE_MAX_EXPERTS;
#pragma unroll
      for (int u = 0; u < W; ++u)  // rising index: the lower one stays on a tie
        if (lane + u * HAL_WAVE < E && place[u] < 0 && (s[u] > best || best_e == MOE_MAX_EXPERTS)) best = s[u], best_e = lane + u * HAL_WAVE;
#pragma unroll
      for (int off = HAL_WAVE / 2; off > 0; off >>= 1) {
        const float ob = __shfl_xor(best, off, HAL_WAVE);
        const int oe = __shfl_xor(best_e, off, HAL_WAVE);
        if (oe < MOE_MAX_EXPERTS && (best_e == MOE_MAX_EXPERTS || ob > best || (ob == best && oe < best_e))) best = ob, best_e = oe;
      }
      float own = 0.f;
#pragma unroll
      for (int u = 0; u < W; ++u)
        if (lane + u * HAL_WAVE == best_e) place[u] = j, own = w[u];  // taken
      sum += lane_value(own, __builtin_amdgcn_readfirstlane(best_e % HAL_WAVE));
    }
    sum += how.norm_eps;
#pragma unroll
    for (int u = 0; u < W; ++u) {
      mine[u] = (how.normalize ? w[u] / sum : w[u]) * how.scale;
      if (place[u] < 0) continue;
      idx[(size_t)t * top + place[u]] = lane + u * HAL_WAVE;
      wgt[(size_t)t * top + place[u]] = mine[u];
    }
  }
}

template <int W>
__global__ void __launch_bounds__(HAL_WAVE) moe_route_kernel(const float* __restrict__ z, int ldz, int E, int top, MoeChoice how,
                                                             int* __restrict__ idx, float* __restrict__ wgt, int n_tokens) {
  moe_route_token<W>(z, ldz, E, top, how, idx, wgt, blockIdx.x, threadIdx.x);
}

static int moe_check_choice(const MoeChoice& how, int E, int top) {
  HAL_REQUIRE(how.c_dtype == HAL_F32 || how.c_dtype == HAL_BF16, "router: a correction of type %d", how.c_dtype);
  HAL_REQUIRE(how.groups >= 0 && (how.groups == 0 || (E % how.groups == 0 && how.keep > 0 && how.keep <= how.groups &&
                                                      top <= E / how.groups * how.keep)),
              "router: %d of %d experts in %d groups of which %d are kept", top, E, how.groups, how.keep);
  return 0;
}

#define MOE_BY_WORDS(LAUNCH_, MOST_)               \
  do {                                             \
    if (E <= HAL_WAVE) LAUNCH_(1);                 \
    else if (E <= 2 * HAL_WAVE) LAUNCH_(2);        \
    else if (E <= 4 * HAL_WAVE) LAUNCH_(4);        \
    else if (MOST_ > 4) LAUNCH_(MOST_);            \
  } while (0)

extern "C" int hal_moe_route(const float* z, int ldz, int E, int top, int softmax, int normalize, float norm_eps,
                             float scale, const void* correction, int c_dtype, int groups, int keep, int* idx,
                             float* wgt, int n_tokens, hipStream_t stream) {
  const MoeChoice how = {softmax, normalize, norm_eps, scale, correction, c_dtype, groups, keep};
  HAL_REQUIRE(n_tokens >= 0 && E > 0 && E <= MOE_MAX_EXPERTS && top > 0 && top <= E && ldz >= E,
              "hal_moe_route: bad sizes T=%d E=%d top=%d", n_tokens, E, top);
  if (int rc = moe_check_choice(how, E, top)) return rc;
  if (n_tokens == 0) return 0;
#define MOE_ROUTE(W_) \
  hipLaunchKernelGGL(moe_route_kernel<W_>, dim3(n_tokens), dim3(HAL_WAVE), 0, stream, z, ldz, E, top, how, idx, wgt, n_tokens)
  MOE_BY_WORDS(MOE_ROUTE, 16);
#undef MOE_ROUTE
  HAL_LAUNCH_CHECK();
  return 0;
}

// ---------------------------------------------------------------------------------
// Counting sort of the n = T * top pairs by expert, one workgroup.  offsets [E + 1]: where
// each expert's pairs begin in `sorted`; tile_offsets [E + 1]: the same counted in tiles of
// `tile` rows, each expert's count rounded up; sorted [n]: pair numbers (token * top +
// choice), expert by expert.  The order inside an expert is not fixed; nothing that is
// computed from it depends on it.
// ---------------------------------------------------------------------------------
// (idx without __restrict__: the kernel that routes and sorts in one has just written it)
__device__ __forceinline__ void moe_sort_pairs(const int* idx, int n, int E, int tile,
                                               int* __restrict__ offsets, int* __restrict__ tile_offsets,
                                               int* __restrict__ sorted, int* count, int* cursor) {
  for (int e = threadIdx.x; e < E; e += blockDim.x) count[e] = 0;
  __syncthreads();
  for (int i = threadIdx.x; i < n; i += blockDim.x) {
    const int e = idx[i];
    if (e >= 0 && e < E) atomicAdd(&count[e], 1);
  }
  __syncthreads();
  if (threadIdx.x < HAL_WAVE) {  // the first wave: running sums, 64 experts at a time
    const int lane = threadIdx.x;
    int at = 0, tiles = 0;
    for (int e0 = 0; e0 < E; e0 += HAL_WAVE) {
      const int e = e0 + lane, c = e < E ? count[e] : 0, ct = (c + tile - 1) / tile;
      int sum = c, sum_t = ct;
#pragma unroll
      for (int off = 1; off < HAL_WAVE; off <<= 1) {
        const int a = __shfl_up(sum, off, HAL_WAVE), b = __shfl_up(sum_t, off, HAL_WAVE);
        if (lane >= off) sum += a, sum_t += b;
      }
      if (e < E) {
        offsets[e] = cursor[e] = at + sum - c;
        tile_offsets[e] = tiles + sum_t - ct;
      }
      at += __shfl(sum, HAL_WAVE - 1, HAL_WAVE);
      tiles += __shfl(sum_t, HAL_WAVE - 1, HAL_WAVE);
    }
    if (lane == 0) {
      offsets[E] = at;
      tile_offsets[E] = tiles;
    }
  }
  __syncthreads();
  for (int i = threadIdx.x; i < n; i += blockDim.x) {
    const int e = idx[i];
    if (e >= 0 && e < E) sorted[atomicAdd(&cursor[e], 1)] = i;
  }
}

__global__ void __launch_bounds__(1024) moe_sort_kernel(const int* __restrict__ idx, int n, int E, int tile,
                                                        int* __restrict__ offsets,
                                                        int* __restrict__ tile_offsets,
                                                        int* __restrict__ sorted) {
  __shared__ int count[MOE_MAX_EXPERTS];
  __shared__ int cursor[MOE_MAX_EXPERTS];
  moe_sort_pairs(idx, n, E, tile, offsets, tile_offsets, sorted, count, cursor);
}

// Both in one workgroup, for steps of few tokens and up to 256 experts: its waves take the tokens in
// turn, then all of it sorts the pairs.
template <int W>
__global__ void __launch_bounds__(1024) moe_route_sort_kernel(const float* __restrict__ z, int ldz, int E, int top,
                                                              MoeChoice how, int* __restrict__ idx,
                                                              float* __restrict__ wgt, int n_tokens, int tile,
                                                              int* __restrict__ offsets, int* __restrict__ tile_offsets,
                                                              int* __restrict__ sorted) {
  __shared__ int count[MOE_MAX_EXPERTS];
  __shared__ int cursor[MOE_MAX_EXPERTS];
  const int wave = threadIdx.x / HAL_WAVE, lane = threadIdx.x % HAL_WAVE;
  for (int t = wave; t < n_tokens; t += blockDim.x / HAL_WAVE)
    moe_route_token<W>(z, ldz, E, top, how, idx, wgt, t, lane);
  __threadfence_block();
  __syncthreads();
  moe_sort_pairs(idx, n_tokens * top, E, tile, offsets, tile_offsets, sorted, count, cursor);
}

extern "C" int hal_moe_route_sort(const float* z, int ldz, int E, int top, int softmax, int normalize, float norm_eps,
                                  float scale, const void* correction, int c_dtype, int groups, int keep,
                                  int* idx, float* wgt, int n_tokens, int tile, int* offsets, int* tile_offsets,
                                  int* sorted, hipStream_t stream) {
  const MoeChoice how = {softmax, normalize, norm_eps, scale, correction, c_dtype, groups, keep};
  HAL_REQUIRE(n_tokens >= 0 && E > 0 && E <= 4 * HAL_WAVE && top > 0 && top <= E && ldz >= E && tile > 0,
              "hal_moe_route_sort: bad sizes T=%d E=%d top=%d", n_tokens, E, top);
  if (int rc = moe_check_choice(how, E, top)) return rc;
  int waves = n_tokens < 4 ? 4 : (n_tokens < 16 ? n_tokens : 16);
#define MOE_ROUTE_SORT(W_)                                                                                                    \
  hipLaunchKernelGGL(moe_route_sort_kernel<W_>, dim3(1), dim3(waves * HAL_WAVE), 0, stream, z, ldz, E, top, how, idx, wgt,    \
                     n_tokens, tile, offsets, tile_offsets, sorted)
  MOE_BY_WORDS(MOE_ROUTE_SORT, 4);
#undef MOE_ROUTE_SORT
  HAL_LAUNCH_CHECK();
  return 0;
}

extern "C" int hal_moe_sort(const int* idx, int n, int E, int tile, int* offsets, int* tile_offsets,
                            int* sorted, hipStream_t stream) {
  HAL_REQUIRE(n >= 0 && E > 0 && E <= MOE_MAX_EXPERTS && tile > 0, "hal_moe_sort: bad sizes n=%d E=%d", n, E);
  hipLaunchKernelGGL(moe_sort_kernel, dim3(1), dim3(1024), 0, stream, idx, n, E, tile, offsets,
                     tile_offsets, sorted);
  HAL_LAUNCH_CHECK();
  return 0;
}

// ---------------------------------------------------------------------------------
// h[t, :] += sum_j wgt[t, j] * y[t * top + j, :] (+ extra[t, :])   (y float32 [T * top, d])
// ---------------------------------------------------------------------------------
__global__ void moe_combine_kernel(float* __restrict__ h, const float* __restrict__ y,
                                   const float* __restrict__ wgt, const float* __restrict__ extra,
                                   const float* __restrict__ extra_gate, int ld_gate, int top, int d, bool overwrite) {
  const int t = blockIdx.x;
  const float eg = extra_gate ? 1.0f / (1.0f + expf(-extra_gate[(size_t)t * ld_gate])) : 1.0f;
  // (a step of few tokens spreads a row over several workgroups: blockIdx.y takes every gridDim.y-th run of columns)
  for (int i = blockIdx.y * blockDim.x + threadIdx.x; i < d; i += blockDim.x * gridDim.y) {
    float s = extra ? eg * extra[(size_t)t * d + i] : 0.f;
    for (int j = 0; j < top; ++j) s += wgt[(size_t)t * top + j] * y[((size_t)t * top + j) * d + i];
    h[(size_t)t * d + i] = overwrite ? s : h[(size_t)t * d + i] + s;
  }
}

extern "C" int hal_moe_combine(float* h, const float* y, const float* wgt, const float* extra,
                               const float* extra_gate, int ld_gate, int top, int d, int n_tokens,
                               int overwrite, hipStream_t stream) {
  HAL_REQUIRE(n_tokens >= 0 && top > 0 && d > 0, "hal_moe_combine: bad sizes");
  if (n_tokens == 0) return 0;
  int threads = (d + 63) / 64 * 64;
  if (threads > 256) threads = 256;
  int parts = 1;  // workgroups a row, so that a decode step has a few hundred of them
  while (parts < 16 && n_tokens * parts < 256 && d / (threads * parts * 2) >= 1) parts *= 2;
  hipLaunchKernelGGL(moe_combine_kernel, dim3(n_tokens, parts), dim3(threads), 0, stream, h, y, wgt, extra, extra_gate, ld_gate, top, d, overwrite != 0);
  HAL_LAUNCH_CHECK();
  return 0;
}
