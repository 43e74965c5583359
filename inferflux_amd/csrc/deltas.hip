// Several additions to the residual stream at once.  A term is a tensor [T, H] (float or bfloat16), a product left as float
// partial sums (slices, added in order), or one vector [H] for all rows, each with a factor.
//   add_terms_rmsnorm   x = stream + sum of the terms (written back unless rows are picked); out = x / sqrt(mean(x^2) + eps) * weight
//   join_stream         out[t] = [stream[t] + sum of the terms | other[t]], rounded to the activation type
// All arithmetic is float; terms are added in their order.
#include "common.h"

IFX_DEFINE_LAST_ERROR()

#define MAX_TERMS 6
#define MAX_PIECES 64        // tensors, vectors and single slices of all terms

// What is added, piece by piece: a slice of a term is a piece of its own, so that the loads of many are on their way at once.
struct Piece { const void* p; int dtype, row_stride; float scale; };
struct Pieces { Piece t[MAX_PIECES]; int n; };

__device__ __forceinline__ float pieces_at(const Pieces& pieces, size_t row, int i, float x) {
  for (int k = 0; k < pieces.n; ++k) x = fmaf(load_dyn(pieces.t[k].p, pieces.t[k].dtype, row * pieces.t[k].row_stride + i), pieces.t[k].scale, x);
  return x;
}
typedef __attribute__((__vector_size__(4 * sizeof(__bf16)))) __bf16 dl_bf16x4;
__device__ __forceinline__ void dl_load4(const void* p, int dtype, size_t at, float* v) {
  if (dtype == DT_F32) {
    const float4 t = *(const float4*)((const float*)p + at);
    v[0] = t.x; v[1] = t.y; v[2] = t.z; v[3] = t.w;
  } else {
    const dl_bf16x4 t = *(const dl_bf16x4*)((const bf16_t*)p + at);
#pragma unroll
    for (int e = 0; e < 4; ++e) v[e] = (float)t[e];
  }
}
__device__ __forceinline__ void dl_store4(float* p, const float* v) { *(float4*)p = make_float4(v[0], v[1], v[2], v[3]); }
__device__ __forceinline__ void dl_store4(bf16_t* p, const float* v) {
  dl_bf16x4 t;
#pragma unroll
  for (int e = 0; e < 4; ++e) t[e] = (__bf16)v[e];
  *(dl_bf16x4*)p = t;
}
// x[v][..] += the pieces at columns 4 (threadIdx.x + 256 v) of ``row``, AT_ONCE of them asked for before the first is added
template <int NV>
__device__ __forceinline__ void add_pieces4(const Pieces& pieces, size_t row, int H, float x[NV][4]) {
  constexpr int AT_ONCE = NV <= 2 ? 8 : (NV <= 4 ? 4 : 2);
  for (int k0 = 0; k0 < pieces.n; k0 += AT_ONCE) {
    float d[AT_ONCE][NV][4];
#pragma unroll
    for (int u = 0; u < AT_ONCE; ++u) {
      const Piece& k = pieces.t[min(k0 + u, pieces.n - 1)];
#pragma unroll
      for (int v = 0; v < NV; ++v) {
        const int i = 4 * (threadIdx.x + 256 * v);
        if (i < H && k0 + u < pieces.n) dl_load4(k.p, k.dtype, row * k.row_stride + i, d[u][v]);
        else d[u][v][0] = d[u][v][1] = d[u][v][2] = d[u][v][3] = 0.f;
      }
    }
#pragma unroll
    for (int u = 0; u < AT_ONCE; ++u) {
      const float scale = pieces.t[min(k0 + u, pieces.n - 1)].scale;
#pragma unroll
      for (int v = 0; v < NV; ++v)
#pragma unroll
        for (int e = 0; e < 4; ++e) x[v][e] = fmaf(d[u][v][e], scale, x[v][e]);
    }
  }
}

template <typename TO, int NV>
__global__ __launch_bounds__(256) void add_terms_rmsnorm4_kernel(float* __restrict__ stream, Pieces pieces, const void* __restrict__ weight,
                                                                 int weight_dtype, TO* __restrict__ out, const int* __restrict__ rows, int H,
                                                                 float eps, int write_back) {
  __shared__ float red[16];
  const size_t src = rows ? (size_t)rows[blockIdx.x] : (size_t)blockIdx.x;
  float x[NV][4];
#pragma unroll
  for (int v = 0; v < NV; ++v) {
    const int i = 4 * (threadIdx.x + 256 * v);
    if (i < H) dl_load4(stream, DT_F32, src * H + i, x[v]);
    else x[v][0] = x[v][1] = x[v][2] = x[v][3] = 0.f;
  }
  add_pieces4<NV>(pieces, src, H, x);
  float ss = 0.f;
#pragma unroll
  for (int v = 0; v < NV; ++v) {
    const int i = 4 * (threadIdx.x + 256 * v);
    if (write_back && i < H) dl_store4(stream + src * H + i, x[v]);
#pragma unroll
    for (int e = 0; e < 4; ++e) ss += x[v][e] * x[v][e];
  }
  const float f = rsqrtf(block_sum(ss, red) / (float)H + eps);
#pragma unroll
  for (int v = 0; v < NV; ++v) {
    const int i = 4 * (threadIdx.x + 256 * v);
    if (i >= H) continue;
    float w[4], y[4];
    dl_load4(weight, weight_dtype, i, w);
#pragma unroll
    for (int e = 0; e < 4; ++e) y[e] = x[v][e] * f * w[e];
    dl_store4(out + (size_t)blockIdx.x * H + i, y);
  }
}

// any width: the sum is formed twice where it is not written back
template <typename TO>
__global__ __launch_bounds__(256) void add_terms_rmsnorm_kernel(float* __restrict__ stream, Pieces pieces, const void* __restrict__ weight,
                                                                int weight_dtype, TO* __restrict__ out, const int* __restrict__ rows, int H,
                                                                float eps, int write_back) {
  __shared__ float red[16];
  const size_t src = rows ? (size_t)rows[blockIdx.x] : (size_t)blockIdx.x;
  float* res = stream + src * H;
  auto at = [&](int i) { return pieces_at(pieces, src, i, res[i]); };
  float ss = 0.f;
  for (int i = threadIdx.x; i < H; i += 256) {
    const float x = at(i);
    if (write_back) res[i] = x;
    ss += x * x;
  }
  const float f = rsqrtf(block_sum(ss, red) / (float)H + eps);
  for (int i = threadIdx.x; i < H; i += 256) {
    const float x = write_back ? res[i] : at(i);
    out[(size_t)blockIdx.x * H + i] = from_f<TO>(x * f * load_dyn(weight, weight_dtype, i));
  }
}

template <typename TO, int NV>
__global__ __launch_bounds__(256) void join_stream4_kernel(const float* __restrict__ stream, Pieces pieces, const float* __restrict__ other,
                                                           TO* __restrict__ out, int H) {
  const size_t t = blockIdx.x;
  float x[NV][4], y[NV][4];
#pragma unroll
  for (int v = 0; v < NV; ++v) {
    const int i = 4 * (threadIdx.x + 256 * v);
    if (i < H) {
      dl_load4(stream, DT_F32, t * H + i, x[v]);
      dl_load4(other, DT_F32, t * H + i, y[v]);
    }
  }
  add_pieces4<NV>(pieces, t, H, x);
#pragma unroll
  for (int v = 0; v < NV; ++v) {
    const int i = 4 * (threadIdx.x + 256 * v);
    if (i < H) {
      dl_store4(out + t * 2 * H + i, x[v]);
      dl_store4(out + t * 2 * H + H + i, y[v]);
    }
  }
}

// any width
template <typename TO>
__global__ __launch_bounds__(256) void join_stream_kernel(const float* __restrict__ stream, Pieces pieces, const float* __restrict__ other,
                                                          TO* __restrict__ out, int H) {
  const size_t t = blockIdx.x;
  const int c = blockIdx.y * 256 + threadIdx.x;
  if (c >= 2 * H) return;
  float x;
  if (c < H) {
    x = pieces_at(pieces, t, c, stream[t * H + c]);
  } else {
    x = other[t * H + c - H];
  }
  out[t * 2 * H + c] = from_f<TO>(x);
}

// The terms as arrays on the host: pointers, element types, slices, elements between slices and rows, factors.
static int gather_terms(Pieces& out, int n, const void* const* p, const int* dtype, const int* n_slices, const long long* slice_stride,
                        const int* row_stride, const float* scale) {
  out.n = 0;
  if (n < 0 || n > MAX_TERMS) return 0;
  for (int k = 0; k < n; ++k) {
    if (!p[k] || n_slices[k] < 1 || (n_slices[k] > 1 && dtype[k] != DT_F32) || (dtype[k] != DT_F32 && dtype[k] != DT_BF16)) return 0;
    if (out.n + n_slices[k] > MAX_PIECES) return 0;
    for (int s = 0; s < n_slices[k]; ++s)
      out.t[out.n++] = Piece{(const char*)p[k] + (size_t)s * slice_stride[k] * sizeof(float), dtype[k], row_stride[k], scale[k]};
  }
  return 1;
}

extern "C" int ifx_add_terms_rmsnorm(float* stream_io, int n_terms, const void* const* p, const int* dtype, const int* n_slices,
                                     const long long* slice_stride, const int* row_stride, const float* scale, const void* weight,
                                     int weight_dtype, void* out, int out_dtype, const int* rows, int n_rows, int H, float eps,
                                     int write_back, void* stream) {
  IFX_REQUIRE(n_rows >= 0 && H > 0, "add_terms_rmsnorm: bad sizes rows=%d H=%d", n_rows, H);
  IFX_REQUIRE(!(rows && write_back), "add_terms_rmsnorm: a row gather cannot write the stream back");
  IFX_REQUIRE(out_dtype == DT_F32 || out_dtype == DT_BF16, "add_terms_rmsnorm: unknown out dtype %d", out_dtype);
  Pieces pieces;
  IFX_REQUIRE(gather_terms(pieces, n_terms, p, dtype, n_slices, slice_stride, row_stride, scale), "add_terms_rmsnorm: bad terms (%d, at most %d, of %d slices together)", n_terms, MAX_TERMS, MAX_PIECES);
  if (n_rows == 0) return 0;
  hipStream_t s = (hipStream_t)stream;
#define GO4(TO, NV) hipLaunchKernelGGL((add_terms_rmsnorm4_kernel<TO, NV>), dim3(n_rows), dim3(256), 0, s, stream_io, pieces, weight, weight_dtype, (TO*)out, rows, H, eps, write_back)
#define GO(TO)                                          \
  do {                                                  \
    if (H % 4 == 0 && H <= 1024) GO4(TO, 1);            \
    else if (H % 4 == 0 && H <= 2048) GO4(TO, 2);       \
    else if (H % 4 == 0 && H <= 4096) GO4(TO, 4);       \
    else if (H % 4 == 0 && H <= 8192) GO4(TO, 8);       \
    else hipLaunchKernelGGL(add_terms_rmsnorm_kernel<TO>, dim3(n_rows), dim3(256), 0, s, stream_io, pieces, weight, weight_dtype, (TO*)out, rows, H, eps, write_back); \
  } while (0)
  if (out_dtype == DT_F32) GO(float);
  else GO(bf16_t);
#undef GO
#undef GO4
  IFX_LAUNCH_CHECK();
}

extern "C" int ifx_join_stream(const float* x, int n_terms, const void* const* p, const int* dtype, const int* n_slices,
                               const long long* slice_stride, const int* row_stride, const float* scale, const float* other, void* out,
                               int out_dtype, int T, int H, void* stream) {
  IFX_REQUIRE(T >= 0 && H > 0, "join_stream: bad sizes T=%d H=%d", T, H);
  Pieces pieces;
  IFX_REQUIRE(gather_terms(pieces, n_terms, p, dtype, n_slices, slice_stride, row_stride, scale), "join_stream: bad terms (%d, at most %d, of %d slices together)", n_terms, MAX_TERMS, MAX_PIECES);
  if (T == 0) return 0;
  const dim3 grid(T, (2 * H + 255) / 256);
  hipStream_t s = (hipStream_t)stream;
  if (H % 4 == 0 && H <= 8192 && (out_dtype == DT_F32 || out_dtype == DT_BF16)) {
#define JOIN(TO, NV) hipLaunchKernelGGL((join_stream4_kernel<TO, NV>), dim3(T), dim3(256), 0, s, x, pieces, other, (TO*)out, H)
#define JOIN_ALL(TO)                 \
  do {                               \
    if (H <= 1024) JOIN(TO, 1);      \
    else if (H <= 2048) JOIN(TO, 2); \
    else if (H <= 4096) JOIN(TO, 4); \
    else JOIN(TO, 8);                \
  } while (0)
    if (out_dtype == DT_F32) JOIN_ALL(float);
    else JOIN_ALL(bf16_t);
#undef JOIN_ALL
#undef JOIN
    IFX_LAUNCH_CHECK();
  }
  if (out_dtype == DT_F32) hipLaunchKernelGGL(join_stream_kernel<float>, grid, dim3(256), 0, s, x, pieces, other, (float*)out, H);
  else if (out_dtype == DT_BF16) hipLaunchKernelGGL(join_stream_kernel<bf16_t>, grid, dim3(256), 0, s, x, pieces, other, (bf16_t*)out, H);
  else IFX_FAIL("join_stream: unknown out dtype %d", out_dtype);
  IFX_LAUNCH_CHECK();
}
