// What time mixing needs around its projections and its recurrence:
//   shifted_mixes   out[s][t][c] = h[t][c] + (h'[t][c] - h[t][c]) mu[s][c] for S sources s, h' the request's row before t: the row
//                   before in this step, or the last row of the request's last step, kept in its state (zeros for a request
//                   that starts), which is replaced by this step's last row
//   lowrank_tanh    z[t][c] = sum_r W[r][c] tanh(a[t][r]), float sums
// All arithmetic is float.
#include "common.h"

IFX_DEFINE_LAST_ERROR()

typedef __attribute__((__vector_size__(4 * sizeof(__bf16)))) __bf16 tm_bf16x4;
template <typename T> __device__ __forceinline__ void tm_load4(const T* p, float* v);
template <> __device__ __forceinline__ void tm_load4<float>(const float* p, float* v) {
  const float4 t = *(const float4*)p; v[0] = t.x; v[1] = t.y; v[2] = t.z; v[3] = t.w;
}
template <> __device__ __forceinline__ void tm_load4<bf16_t>(const bf16_t* p, float* v) {
  const tm_bf16x4 t = *(const tm_bf16x4*)p;
#pragma unroll
  for (int i = 0; i < 4; ++i) v[i] = (float)t[i];
}
template <typename T> __device__ __forceinline__ void tm_store4(T* p, const float* v);
template <> __device__ __forceinline__ void tm_store4<float>(float* p, const float* v) { *(float4*)p = make_float4(v[0], v[1], v[2], v[3]); }
template <> __device__ __forceinline__ void tm_store4<bf16_t>(bf16_t* p, const float* v) {
  tm_bf16x4 t;
#pragma unroll
  for (int i = 0; i < 4; ++i) t[i] = (__bf16)v[i];
  *(tm_bf16x4*)p = t;
}

struct MixArgs {
  const void* h; const float* mu; float* state; size_t state_stride, state_offset;
  const int* row_req; const int* q_start; const int* q_len; const int* slots;
  void* out; int T, C, S;
};

// V channels a thread (4 where C is a multiple of 4, else 1).  The thread of a request's first row reads the kept row and puts
// the request's last row in its place: nobody else touches those numbers.
template <typename T, int V>
__global__ __launch_bounds__(256) void shifted_mixes_kernel(MixArgs a) {
  const int t = blockIdx.x, c = (blockIdx.y * 256 + threadIdx.x) * V;
  if (c >= a.C) return;
  const int r = a.row_req[t], first = a.q_start[r];
  const T* h = (const T*)a.h;
  float x[V], p[V];
  if (V == 4) tm_load4<T>(h + (size_t)t * a.C + c, x);
  else x[0] = to_f(h[(size_t)t * a.C + c]);
  if (t == first) {
    float* keep = a.state + (size_t)a.slots[r] * a.state_stride + a.state_offset + c;
    const T* last = h + (size_t)(first + a.q_len[r] - 1) * a.C + c;
    float l[V];
    if (V == 4) { tm_load4<float>(keep, p); tm_load4<T>(last, l); tm_store4<float>(keep, l); }
    else { p[0] = *keep; l[0] = to_f(*last); *keep = l[0]; }
  } else {
    if (V == 4) tm_load4<T>(h + (size_t)(t - 1) * a.C + c, p);
    else p[0] = to_f(h[(size_t)(t - 1) * a.C + c]);
  }
  for (int s = 0; s < a.S; ++s) {
    float m[V], y[V];
    if (V == 4) tm_load4<float>(a.mu + (size_t)s * a.C + c, m);
    else m[0] = a.mu[(size_t)s * a.C + c];
#pragma unroll
    for (int i = 0; i < V; ++i) y[i] = fmaf(p[i] - x[i], m[i], x[i]);
    T* o = (T*)a.out + ((size_t)s * a.T + t) * a.C + c;
    if (V == 4) tm_store4<T>(o, y);
    else *o = from_f<T>(y[0]);
  }
}

extern "C" int ifx_shifted_mixes(const void* h, int dtype, const float* mu, float* state, long long state_stride, long long state_offset,
                                 const int* row_req, const int* q_start, const int* q_len, const int* slots, void* out, int T, int C, int S,
                                 void* stream) {
  IFX_REQUIRE(T >= 0 && C > 0 && S > 0, "shifted_mixes: bad sizes T=%d C=%d S=%d", T, C, S);
  IFX_REQUIRE(state_stride >= state_offset + C && state_offset >= 0, "shifted_mixes: a state row of %lld floats is too short", state_stride);
  if (T == 0) return 0;
  MixArgs a{h, mu, state, (size_t)state_stride, (size_t)state_offset, row_req, q_start, q_len, slots, out, T, C, S};
  const bool v4 = C % 4 == 0 && state_offset % 4 == 0 && state_stride % 4 == 0;
  const dim3 grid(T, (C + 256 * (v4 ? 4 : 1) - 1) / (256 * (v4 ? 4 : 1)));
  hipStream_t s = (hipStream_t)stream;
  if (dtype == DT_F32) {
    if (v4) hipLaunchKernelGGL((shifted_mixes_kernel<float, 4>), grid, dim3(256), 0, s, a);
    else hipLaunchKernelGGL((shifted_mixes_kernel<float, 1>), grid, dim3(256), 0, s, a);
  } else if (dtype == DT_BF16) {
    if (v4) hipLaunchKernelGGL((shifted_mixes_kernel<bf16_t, 4>), grid, dim3(256), 0, s, a);
    else hipLaunchKernelGGL((shifted_mixes_kernel<bf16_t, 1>), grid, dim3(256), 0, s, a);
  } else IFX_FAIL("shifted_mixes: unknown dtype %d", dtype);
  IFX_LAUNCH_CHECK();
}

// ``w`` is W transposed, [rank][C], so that neighbouring lanes read neighbouring channels.  A workgroup takes ROWS rows and 128
// output channels, two a lane; tanh of the rows' numbers lies in LDS.  Its four waves share the rank, a quarter each, and their
// sums meet in LDS in wave order.
template <typename T> __device__ __forceinline__ void tm_load2(const T* p, float& a, float& b);
template <> __device__ __forceinline__ void tm_load2<float>(const float* p, float& a, float& b) { const float2 t = *(const float2*)p; a = t.x; b = t.y; }
template <> __device__ __forceinline__ void tm_load2<bf16_t>(const bf16_t* p, float& a, float& b) {
  typedef __attribute__((__vector_size__(2 * sizeof(__bf16)))) __bf16 bf16x2;
  const bf16x2 t = *(const bf16x2*)p;
  a = (float)t[0]; b = (float)t[1];
}

#define LR_WAVES 4
template <typename T, int ROWS>
__global__ __launch_bounds__(LR_WAVES * WAVE) void lowrank_tanh_kernel(const float* __restrict__ a, int lda, const T* __restrict__ w,
                                                                      float* __restrict__ z, int rows, int rank, int C) {
  extern __shared__ __attribute__((aligned(16))) float lr_lds[];       // tanh [rank][ROWS], then the waves' sums [LR_WAVES - 1][ROWS][128]
  float* th = lr_lds;
  float* part = lr_lds + rank * ROWS;
  const int t0 = blockIdx.x * ROWS, n = min(ROWS, rows - t0), wid = threadIdx.x / WAVE, lane = threadIdx.x % WAVE;
  for (int x = threadIdx.x; x < ROWS * rank; x += LR_WAVES * WAVE) {
    const int r = x / ROWS, tt = x % ROWS;
    th[x] = tt < n ? tanhf(a[(size_t)(t0 + tt) * lda + r]) : 0.f;
  }
  __syncthreads();
  const int c = blockIdx.y * 128 + 2 * lane;          // (C is even where two channels are read at once)
  const bool both = c + 1 < C && C % 2 == 0;
  float acc[ROWS][2];
#pragma unroll
  for (int i = 0; i < ROWS; ++i) acc[i][0] = acc[i][1] = 0.f;
  const int per = (rank + LR_WAVES - 1) / LR_WAVES, r0 = wid * per, r1 = min(rank, r0 + per);
  // eight channels' pairs of weights are asked for at once, from places that exist (what they give past the ends is dropped)
  for (int rb = r0; rb < r1; rb += 8) {
    float w0[8], w1[8];
    if (C % 2 == 0) {
      const T* wc = w + min(c, C - 2);
#pragma unroll
      for (int u = 0; u < 8; ++u) tm_load2<T>(wc + (size_t)min(rb + u, rank - 1) * C, w0[u], w1[u]);
    } else {
#pragma unroll
      for (int u = 0; u < 8; ++u) {
        const T* wr = w + (size_t)min(rb + u, rank - 1) * C;
        w0[u] = to_f(wr[min(c, C - 1)]);
        w1[u] = to_f(wr[min(c + 1, C - 1)]);
      }
    }
#pragma unroll
    for (int u = 0; u < 8; ++u) {
      if (rb + u >= r1) break;
#pragma unroll
      for (int i = 0; i < ROWS; ++i) {
        const float t = th[(rb + u) * ROWS + i];
        acc[i][0] = fmaf(w0[u], t, acc[i][0]);
        acc[i][1] = fmaf(w1[u], t, acc[i][1]);
      }
    }
  }
  if (wid > 0)
#pragma unroll
    for (int i = 0; i < ROWS; ++i) *(float2*)(part + ((size_t)(wid - 1) * ROWS + i) * 128 + 2 * lane) = make_float2(acc[i][0], acc[i][1]);
  __syncthreads();
  if (wid > 0) return;
  for (int v = 0; v < LR_WAVES - 1; ++v)
#pragma unroll
    for (int i = 0; i < ROWS; ++i) {
      const float2 p = *(const float2*)(part + ((size_t)v * ROWS + i) * 128 + 2 * lane);
      acc[i][0] += p.x; acc[i][1] += p.y;
    }
#pragma unroll
  for (int i = 0; i < ROWS; ++i) {
    if (i >= n) break;
    float* o = z + (size_t)(t0 + i) * C + c;
    if (both) *(float2*)o = make_float2(acc[i][0], acc[i][1]);
    else {
      if (c < C) o[0] = acc[i][0];
      if (c + 1 < C) o[1] = acc[i][1];
    }
  }
}

extern "C" int ifx_lowrank_tanh(const float* a, int lda, const void* w, int w_dtype, float* z, int T, int rank, int C, void* stream) {
  IFX_REQUIRE(T >= 0 && rank > 0 && C > 0 && lda >= rank, "lowrank_tanh: bad sizes T=%d rank=%d C=%d", T, rank, C);
  const int rows = T <= 16 ? 2 : (T <= 128 ? 4 : 16);         // (few rows: more workgroups)
  const size_t lds = ((size_t)rows * rank + (size_t)(LR_WAVES - 1) * rows * 128) * sizeof(float);
  IFX_REQUIRE(lds <= 64 * 1024, "lowrank_tanh: a rank of %d does not fit a workgroup's LDS", rank);
  if (T == 0) return 0;
  const dim3 grid((T + rows - 1) / rows, (C + 127) / 128);
  hipStream_t s = (hipStream_t)stream;
#define LR(TY, R) hipLaunchKernelGGL((lowrank_tanh_kernel<TY, R>), grid, dim3(LR_WAVES * WAVE), lds, s, a, lda, (const TY*)w, z, T, rank, C)
  if (w_dtype == DT_F32) { if (rows == 2) LR(float, 2); else if (rows == 4) LR(float, 4); else LR(float, 16); }
  else if (w_dtype == DT_BF16) { if (rows == 2) LR(bf16_t, 2); else if (rows == 4) LR(bf16_t, 4); else LR(bf16_t, 16); }
  else IFX_FAIL("lowrank_tanh: unknown dtype %d", w_dtype);
#undef LR
  IFX_LAUNCH_CHECK();
}
