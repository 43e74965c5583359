// Matrix memory with exponential gates: a recurrence per head whose state is a matrix S [d, dv] and a normaliser n [d], both
// decayed and written with one number per token and kept relative to exp(m), m the running maximum of the exponents.
//
// For a request's tokens t = 0, 1, ... and each head:
//
//   i = cap tanh((i_in + i_bias) / cap),  f = log sigmoid(cap tanh((f_in + f_bias) / cap))
//   m_t = max(f + m_(t-1), i),  m_(-1) = 0;  keep = exp(f + m_(t-1) - m_t),  write = exp(i - m_t)
//   S <- keep S + write k v^T;  n <- keep n + write k;  o = S^T q * q_scale / (max(|n . q * q_scale|, exp(-m_t)) + 1e-6)
//   out = o / sqrt(mean(o^2) + eps) * w_norm * sigmoid(gate_in)         (the norm over the head's dv values)
//
// q, k, v and gate_in are columns of projected rows [T, ld] (float or bfloat16), i_in and f_in columns of float rows.  Gates,
// m, S, n, every sum, the norm and the gate are float whatever those types are.
//
// The normaliser is one more column of S: column dv, whose value is 1 for every token.  A request's state is one float row:
// m [H, padded to a multiple of 4], then S laid out [head][column 0 .. dv][d_pad], d_pad = CH * KS >= d (padding stays zero).
// The columns of S never meet, so a head's columns are dealt to several workgroups of ``cols`` columns each.  In a workgroup
// thread (column, run) holds CH consecutive key channels of its column in registers; the KS threads of a column are
// neighbouring lanes and add their parts of S^T q in a fixed order.  Tokens are taken STAGE at a time: all threads load the
// stage's q, k and their columns of v into LDS, one wave forms the gates and the running maximum of the stage (the maximum
// as a scan over its lanes: m after a token is max(m + F, M) of the composed pairs (F, M)), everybody walks the tokens.  Read-outs
// go to ``o_raw`` [T, H, dv + 1] (float); a second kernel, a wave per (token, head), divides, norms and gates them, and
// writes a request's last m into its state (the walk's workgroups all read the old one).
#include "common.h"
#include "lane_sums.h"

IFX_DEFINE_LAST_ERROR()

#define STAGE 16

struct MemoryArgs {
  const void* rows; int ld, q_col, k_col, v_col, g_col;
  const float* gates; int ldg, i_col, f_col;
  const float* i_bias; const float* f_bias; float cap, q_scale;
  const float* norm_w; float eps;              // [H dv]
  float* state; size_t state_stride; int s_off;
  const int* q_start; const int* q_len; const int* slots; const int* row_req;
  float* o_raw;        // [T, H, dv + 1]
  float* floor;        // [T, H]: exp(-m_t)
  float* m_end;        // [R, H]
  void* out;           // [T, H dv]
  int T, R, H, d, dv, KS, cols;
};

__device__ __forceinline__ float log_sigmoid(float x) {      // -softplus(-x), without overflow
  return x >= 0.f ? -log1pf(expf(-x)) : x - log1pf(expf(x));
}
__device__ __forceinline__ float soft_cap(float x, float cap) { return cap * tanhf(x / cap); }

template <typename TI, int CH>
__global__ __launch_bounds__(256) void memory_walk_kernel(MemoryArgs a) {
  extern __shared__ __attribute__((aligned(16))) float lds[];      // q and k of a stage [STAGE][dpad] each, then its v [STAGE][cols]
  __shared__ float keep_s[STAGE], write_s[STAGE];
  const int n_cols = a.dv + 1, n_cb = (n_cols + a.cols - 1) / a.cols;
  const int h = blockIdx.x / n_cb, cb = blockIdx.x % n_cb, j0 = cb * a.cols, r = blockIdx.y;
  const int n = a.q_len[r];
  if (n <= 0) return;
  const int t0 = a.q_start[r], d = a.d, KS = a.KS, dpad = CH * KS;
  const int cols = min(a.cols, n_cols - j0);
  float* q_s = lds;
  float* k_s = lds + STAGE * dpad;
  float* v_s = lds + 2 * STAGE * dpad;
  const int tid = threadIdx.x, nthr = blockDim.x, lane = tid % WAVE;
  const int jl = tid / KS, s = tid % KS;
  const bool owner = jl < cols;
  float* row = a.state + (size_t)a.slots[r] * a.state_stride;
  float* Sp = row + a.s_off + ((size_t)h * n_cols + j0 + (owner ? jl : 0)) * dpad + s * CH;
  float S[CH];
#pragma unroll
  for (int c = 0; c < CH; c += 4) {
    const float4 v = owner ? *(const float4*)(Sp + c) : make_float4(0.f, 0.f, 0.f, 0.f);
    S[c] = v.x; S[c + 1] = v.y; S[c + 2] = v.z; S[c + 3] = v.w;
  }
  float m = row[h];                    // (kept by the first wave)
  const float ib = a.i_bias[h], fb = a.f_bias[h];
  const TI* rows = (const TI*)a.rows;
  const LaneSteps steps = lane_steps(KS);
  const int dshift = __ffs(dpad) - 1;
  for (int base = 0; base < n; base += STAGE) {
    const int cnt = min(STAGE, n - base);
    if (tid < WAVE) {
      // the stage's gates, a token a lane, and the running maximum as a scan of the pairs (F: sum of f, M: the best exponent)
      const bool in = lane < cnt;
      const size_t t = (size_t)(t0 + base + (in ? lane : 0));
      const float li = in ? soft_cap(a.gates[t * a.ldg + a.i_col + h] + ib, a.cap) : -INFINITY;
      const float lf = in ? log_sigmoid(soft_cap(a.gates[t * a.ldg + a.f_col + h] + fb, a.cap)) : 0.f;
      float F = lf, M = li;
#pragma unroll
      for (int o = 1; o < STAGE; o <<= 1) {
        const float Fp = __shfl_up(F, o, WAVE), Mp = __shfl_up(M, o, WAVE);
        if (lane >= o) { M = fmaxf(Mp + F, M); F += Fp; }
      }
      const float mt = fmaxf(m + F, M);
      const float up = __shfl_up(mt, 1, WAVE);
      const float before = lane == 0 ? m : up;
      if (in) {
        keep_s[lane] = expf(lf + before - mt);
        write_s[lane] = expf(li - mt);
        if (cb == 0) a.floor[t * a.H + h] = expf(-mt);
      }
      m = __shfl(mt, cnt - 1, WAVE);
    }
    for (int x = tid; x < cnt * dpad; x += nthr) {
      const int tt = x >> dshift, c = x & (dpad - 1);
      const size_t at = (size_t)(t0 + base + tt) * a.ld + (size_t)h * d + c;
      q_s[x] = c < d ? to_f(rows[at + a.q_col]) * a.q_scale : 0.f;
      k_s[x] = c < d ? to_f(rows[at + a.k_col]) : 0.f;
    }
    for (int x = tid; x < cnt * cols; x += nthr) {
      const int tt = x / cols, c = x - tt * cols;
      v_s[tt * a.cols + c] = j0 + c < a.dv ? to_f(rows[(size_t)(t0 + base + tt) * a.ld + a.v_col + (size_t)h * a.dv + j0 + c]) : 1.f;
    }
    __syncthreads();
    if (owner) {
      for (int tt = 0; tt < cnt; ++tt) {
        const float keep = keep_s[tt], wv = write_s[tt] * v_s[tt * a.cols + jl];
        const float* kp = k_s + tt * dpad + s * CH;
        const float* qp = q_s + tt * dpad + s * CH;
        float o4[4] = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int c = 0; c < CH; ++c) {
          S[c] = fmaf(kp[c], wv, keep * S[c]);
          o4[c & 3] = fmaf(S[c], qp[c], o4[c & 3]);
        }
        const float o = column_sum((o4[0] + o4[1]) + (o4[2] + o4[3]), steps);
        if (s == 0) a.o_raw[((size_t)(t0 + base + tt) * a.H + h) * n_cols + j0 + jl] = o;
      }
    }
    __syncthreads();
  }
  if (owner) {
#pragma unroll
    for (int c = 0; c < CH; c += 4) *(float4*)(Sp + c) = make_float4(S[c], S[c + 1], S[c + 2], S[c + 3]);
  }
  if (cb == 0 && tid == 0) a.m_end[(size_t)r * a.H + h] = m;
}

// A wave per (token, head): o = o_raw / (max(|n . q|, exp(-m)) + 1e-6), its norm, the weight and the gate.
template <typename TI, typename TO>
__global__ __launch_bounds__(256) void memory_finish_kernel(MemoryArgs a) {
  const size_t item = (size_t)blockIdx.x * (256 / WAVE) + threadIdx.x / WAVE;
  const int lane = threadIdx.x % WAVE;
  if (item >= (size_t)a.T * a.H) return;
  const size_t t = item / a.H;
  const int h = (int)(item % a.H), dv = a.dv;
  const float* o = a.o_raw + item * (dv + 1);
  const float inv_den = 1.0f / (fmaxf(fabsf(o[dv]), a.floor[item]) + 1e-6f);
  float ss = 0.f;
  for (int c = lane; c < dv; c += WAVE) { const float v = o[c] * inv_den; ss = fmaf(v, v, ss); }
  const float f = inv_den / sqrtf(wave_sum(ss) / (float)dv + a.eps);
  const TI* rows = (const TI*)a.rows;
  for (int c = lane; c < dv; c += WAVE) {
    const float g = to_f(rows[t * a.ld + a.g_col + (size_t)h * dv + c]);
    ((TO*)a.out)[item * dv + c] = from_f<TO>(o[c] * f * a.norm_w[(size_t)h * dv + c] / (1.0f + expf(-g)));
  }
  const int r = a.row_req[t];
  if (lane == 0 && (int)t == a.q_start[r] + a.q_len[r] - 1)
    a.state[(size_t)a.slots[r] * a.state_stride + h] = a.m_end[(size_t)r * a.H + h];
}

extern "C" int ifx_matrix_memory(const void* rows, int dtype, int ld, int q_col, int k_col, int v_col, int g_col, const float* gates, int ldg,
                                 int i_col, int f_col, const float* i_bias, const float* f_bias, float cap, float q_scale,
                                 const float* norm_w, float eps, float* state, long long state_stride, int s_off, const int* q_start,
                                 const int* q_len, const int* slots, const int* row_req, float* o_raw, float* floor_, float* m_end,
                                 void* out, int out_dtype, int T, int R, int H, int d, int dv, int ch, int ks, int cols, void* stream) {
  IFX_REQUIRE(T >= 0 && R >= 0 && H > 0 && d > 0 && dv > 0 && cap > 0.f, "matrix_memory: bad sizes T=%d R=%d H=%d d=%d dv=%d", T, R, H, d, dv);
  IFX_REQUIRE(ks > 0 && ks <= WAVE && (ks & (ks - 1)) == 0 && ch * ks >= d, "matrix_memory: %d threads of %d channels for heads of %d", ks, ch, d);
  IFX_REQUIRE(cols > 0 && cols * ks <= 256, "matrix_memory: %d columns x %d threads do not fit a workgroup of 256", cols, ks);
  IFX_REQUIRE(s_off >= H && s_off % 4 == 0 && state_stride % 4 == 0, "matrix_memory: S must lie at a multiple of 16 bytes behind the maxima");
  IFX_REQUIRE(state_stride >= s_off + (long long)H * (dv + 1) * ch * ks, "matrix_memory: a state row of %lld floats is too short", state_stride);
  IFX_REQUIRE(R <= 65535, "matrix_memory: too many requests for one launch");
  const size_t lds = (size_t)STAGE * (2 * ch * ks + cols) * sizeof(float);
  IFX_REQUIRE(lds <= 60 * 1024, "matrix_memory: d=%d needs more LDS than a workgroup has", d);
  if (T == 0 || R == 0) return 0;
  MemoryArgs a{rows, ld, q_col, k_col, v_col, g_col, gates, ldg, i_col, f_col, i_bias, f_bias, cap, q_scale, norm_w, eps, state,
               (size_t)state_stride, s_off, q_start, q_len, slots, row_req, o_raw, floor_, m_end, out, T, R, H, d, dv, ks, cols};
  const dim3 grid(H * ((dv + cols) / cols), R);        // (dv + 1 columns)
  const int threads = (cols * ks + WAVE - 1) / WAVE * WAVE;
  const unsigned blocks = (unsigned)(((size_t)T * H + 256 / WAVE - 1) / (256 / WAVE));
  hipStream_t s = (hipStream_t)stream;
#define WALK(TY, C) hipLaunchKernelGGL((memory_walk_kernel<TY, C>), grid, dim3(threads), lds, s, a)
#define BY_CH(TY)                       \
  do {                                  \
    if (ch == 4) WALK(TY, 4);           \
    else if (ch == 8) WALK(TY, 8);      \
    else if (ch == 16) WALK(TY, 16);    \
    else if (ch == 32) WALK(TY, 32);    \
    else IFX_FAIL("matrix_memory: %d channels a thread (4, 8, 16 or 32)", ch); \
  } while (0)
  if (dtype == DT_F32) BY_CH(float);
  else if (dtype == DT_BF16) BY_CH(bf16_t);
  else IFX_FAIL("matrix_memory: unknown dtype %d", dtype);
#undef BY_CH
#undef WALK
#define FINISH(TI, TO) hipLaunchKernelGGL((memory_finish_kernel<TI, TO>), dim3(blocks), dim3(256), 0, s, a)
  if (dtype == DT_F32 && out_dtype == DT_F32) FINISH(float, float);
  else if (dtype == DT_F32 && out_dtype == DT_BF16) FINISH(float, bf16_t);
  else if (dtype == DT_BF16 && out_dtype == DT_BF16) FINISH(bf16_t, bf16_t);
  else IFX_FAIL("matrix_memory: unsupported types rows=%d out=%d", dtype, out_dtype);
#undef FINISH
  IFX_LAUNCH_CHECK();
}
