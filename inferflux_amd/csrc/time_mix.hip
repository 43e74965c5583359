// What time mixing needs around its projections and its recurrence:
//   shifted_mixes   out[s][t][c] = h[t][c] + (h'[t][c] - h[t][c]) mu[s][c] for S sources s, h' the request's row before t: the row
//                   before in this step, or the last row of the request's last step, kept in its state (zeros for a request
//                   that starts), which is replaced by this step's last row
//   lowrank_tanh    z[t][c] = sum_r W[c][r] tanh(a[t][r]), float sums
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

// A workgroup takes ROWS rows and 256 output channels: tanh of the rows' numbers in LDS, a channel a thread, whose weights are
// read once for all the rows.
#define LR_ROWS 8
template <typename T>
__global__ __launch_bounds__(256) void lowrank_tanh_kernel(const float* __restrict__ a, int lda, const T* __restrict__ w, float* __restrict__ z,
                                                           int rows, int rank, int C) {
  extern __shared__ float th[];              // [LR_ROWS][rank]
  const int t0 = blockIdx.x * LR_ROWS, n = min(LR_ROWS, rows - t0);
  for (int x = threadIdx.x; x < LR_ROWS * rank; x += 256) {
    const int tt = x / rank, r = x - tt * rank;
    th[x] = tt < n ? tanhf(a[(size_t)(t0 + tt) * lda + r]) : 0.f;
  }
  __syncthreads();
  const int c = blockIdx.y * 256 + threadIdx.x;
  if (c >= C) return;
  float acc[LR_ROWS];
#pragma unroll
  for (int i = 0; i < LR_ROWS; ++i) acc[i] = 0.f;
  const T* wc = w + (size_t)c * rank;
  if (rank % 4 == 0) {
    for (int r = 0; r < rank; r += 4) {
      float wv[4];
      tm_load4<T>(wc + r, wv);
#pragma unroll
      for (int i = 0; i < LR_ROWS; ++i)
#pragma unroll
        for (int e = 0; e < 4; ++e) acc[i] = fmaf(wv[e], th[i * rank + r + e], acc[i]);
    }
  } else {
    for (int r = 0; r < rank; ++r) {
      const float wv = to_f(wc[r]);
#pragma unroll
      for (int i = 0; i < LR_ROWS; ++i) acc[i] = fmaf(wv, th[i * rank + r], acc[i]);
    }
  }
  for (int i = 0; i < n; ++i) z[(size_t)(t0 + i) * C + c] = acc[i];
}

extern "C" int ifx_lowrank_tanh(const float* a, int lda, const void* w, int w_dtype, float* z, int T, int rank, int C, void* stream) {
  IFX_REQUIRE(T >= 0 && rank > 0 && C > 0 && lda >= rank, "lowrank_tanh: bad sizes T=%d rank=%d C=%d", T, rank, C);
  IFX_REQUIRE((size_t)LR_ROWS * rank * sizeof(float) <= 64 * 1024, "lowrank_tanh: a rank of %d does not fit a workgroup's LDS", rank);
  if (T == 0) return 0;
  const dim3 grid((T + LR_ROWS - 1) / LR_ROWS, (C + 255) / 256);
  const size_t lds = (size_t)LR_ROWS * rank * sizeof(float);
  hipStream_t s = (hipStream_t)stream;
  if (w_dtype == DT_F32) hipLaunchKernelGGL(lowrank_tanh_kernel<float>, grid, dim3(256), lds, s, a, lda, (const float*)w, z, T, rank, C);
  else if (w_dtype == DT_BF16) hipLaunchKernelGGL(lowrank_tanh_kernel<bf16_t>, grid, dim3(256), lds, s, a, lda, (const bf16_t*)w, z, T, rank, C);
  else IFX_FAIL("lowrank_tanh: unknown dtype %d", w_dtype);
  IFX_LAUNCH_CHECK();
}
