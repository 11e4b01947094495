// RMSNorm in the forms the post-norm language models need, on a residual stream that is kept in 32 bits:
//
//     n = u * rsqrt(mean(u^2) + eps) * (w_offset + w)        w_offset 1: the weight is stored around zero, 0: a plain weight
//     v = n * sigmoid(gate)                                  with a gate
//     s = residual + mult * v                                with a residual (fp32), written to `sum` (fp32)
//     y = s, or v without a residual                         in the model's dtype: what the next matrix product reads
//
// u is a row of x, or — mixture of experts — the weighted sum of a token's expert outputs: u = sum_j wt_j * Y[pos_j], where a
// choice without a row (pos < 0) is an identity expert whose output is the residual row itself.
// Statistics, sums and the residual are fp32; one work-group per row.  Rows of up to 8 192 elements whose pieces are 16-byte
// aligned stay in registers between the statistics and the output; everything else takes a scalar two-pass form.
#include "common.hpp"

namespace {

constexpr int RX_THREADS = 256;
constexpr int RX_MAXV = 4;         // 8-element pieces a thread keeps
constexpr int RX_MAXTOP = 32;

struct RxArgs {
  const void *x, *w, *gate;
  const float* res;
  float* sum;
  void *y, *y2;          // y2: the same row again, to row y2_rows[row] of another buffer (a cache)
  const int* y2_rows;
  const int* pos;        // [rows][top], mixture of experts only
  const float* wts;      // [rows][top]
  int D, top;
  int64_t xs, gs, rs, ss, ys, y2s;
  float eps, mult, woff;
};

template <typename T> __device__ __forceinline__ void load8(const T* p, float (&o)[8]);
template <> __device__ __forceinline__ void load8<float>(const float* p, float (&o)[8]) {
  const f32x4 a = *(const f32x4*)p, b = *(const f32x4*)(p + 4);
#pragma unroll
  for (int i = 0; i < 4; ++i) { o[i] = a[i]; o[4 + i] = b[i]; }
}
template <> __device__ __forceinline__ void load8<bf16_t>(const bf16_t* p, float (&o)[8]) {
  const bf16x8 a = *(const bf16x8*)p;
#pragma unroll
  for (int i = 0; i < 8; ++i) o[i] = (float)a[i];
}
template <typename T> __device__ __forceinline__ void store8(T* p, const float (&o)[8]);
template <> __device__ __forceinline__ void store8<float>(float* p, const float (&o)[8]) {
  *(f32x4*)p = f32x4{o[0], o[1], o[2], o[3]};
  *(f32x4*)(p + 4) = f32x4{o[4], o[5], o[6], o[7]};
}
template <> __device__ __forceinline__ void store8<bf16_t>(bf16_t* p, const float (&o)[8]) {
  bf16x8 v;
#pragma unroll
  for (int i = 0; i < 8; ++i) v[i] = (bf16_t)o[i];
  *(bf16x8*)p = v;
}

__device__ __forceinline__ float block_total(float v, float* red) {
  v = wave_sum(v);
  if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = v;
  __syncthreads();
  float t = 0.f;
#pragma unroll
  for (int i = 0; i < RX_THREADS / 64; ++i) t += red[i];
  return t;
}

template <typename XT, typename WT, typename YT, bool MOE>
__global__ __launch_bounds__(RX_THREADS) void rmsnorm_ex_kernel(RxArgs a) {
  __shared__ float red[RX_THREADS / 64];
  const int64_t row = blockIdx.x;
  const int nv = a.D / 8;
  const XT* xr = (const XT*)a.x + (MOE ? 0 : row * a.xs);
  const float* rr = a.res ? a.res + row * a.rs : nullptr;
  const WT* gr = a.gate ? (const WT*)a.gate + row * a.gs : nullptr;
  float u[RX_MAXV][8], ssq = 0.f;
#pragma unroll
  for (int k = 0; k < RX_MAXV; ++k) {
    const int iv = threadIdx.x + k * RX_THREADS;
    if (iv < nv) {
      if (MOE) {
#pragma unroll
        for (int i = 0; i < 8; ++i) u[k][i] = 0.f;
        for (int j = 0; j < a.top; ++j) {
          const int p = a.pos[row * a.top + j];
          const float wt = a.wts[row * a.top + j];
          float e[8];
          if (p >= 0) load8<XT>(xr + (int64_t)p * a.xs + 8 * iv, e);
          else load8<float>(rr + 8 * iv, e);
#pragma unroll
          for (int i = 0; i < 8; ++i) u[k][i] = fmaf(wt, e[i], u[k][i]);
        }
      } else {
        load8<XT>(xr + 8 * iv, u[k]);
      }
#pragma unroll
      for (int i = 0; i < 8; ++i) ssq = fmaf(u[k][i], u[k][i], ssq);
    }
  }
  const float rstd = rsqrtf(block_total(ssq, red) / (float)a.D + a.eps);
#pragma unroll
  for (int k = 0; k < RX_MAXV; ++k) {
    const int iv = threadIdx.x + k * RX_THREADS;
    if (iv < nv) {
      float w[8], o[8];
      load8<WT>((const WT*)a.w + 8 * iv, w);
#pragma unroll
      for (int i = 0; i < 8; ++i) o[i] = u[k][i] * rstd * (a.woff + w[i]);
      if (gr) {
        float g[8];
        load8<WT>(gr + 8 * iv, g);
#pragma unroll
        for (int i = 0; i < 8; ++i) o[i] *= sigmoid_f(g[i]);
      }
      if (rr) {
        float r[8];
        load8<float>(rr + 8 * iv, r);
#pragma unroll
        for (int i = 0; i < 8; ++i) o[i] = fmaf(a.mult, o[i], r[i]);
        if (a.sum) store8<float>(a.sum + row * a.ss + 8 * iv, o);
      }
      if (a.y) store8<YT>((YT*)a.y + row * a.ys + 8 * iv, o);
      if (a.y2) store8<YT>((YT*)a.y2 + (int64_t)a.y2_rows[row] * a.y2s + 8 * iv, o);
    }
  }
}

// any width and alignment: the row is read twice
template <typename XT, typename WT, typename YT, bool MOE>
__global__ __launch_bounds__(RX_THREADS) void rmsnorm_ex_scalar_kernel(RxArgs a) {
  __shared__ float red[RX_THREADS / 64];
  const int64_t row = blockIdx.x;
  const XT* xr = (const XT*)a.x + (MOE ? 0 : row * a.xs);
  const float* rr = a.res ? a.res + row * a.rs : nullptr;
  const WT* gr = a.gate ? (const WT*)a.gate + row * a.gs : nullptr;
  auto value = [&](int d) {
    if (!MOE) return to_f32(xr[d]);
    float u = 0.f;
    for (int j = 0; j < a.top; ++j) {
      const int p = a.pos[row * a.top + j];
      const float e = p >= 0 ? to_f32(xr[(int64_t)p * a.xs + d]) : rr[d];
      u = fmaf(a.wts[row * a.top + j], e, u);
    }
    return u;
  };
  float ssq = 0.f;
  for (int d = threadIdx.x; d < a.D; d += RX_THREADS) {
    const float u = value(d);
    ssq = fmaf(u, u, ssq);
  }
  const float rstd = rsqrtf(block_total(ssq, red) / (float)a.D + a.eps);
  for (int d = threadIdx.x; d < a.D; d += RX_THREADS) {
    float o = value(d) * rstd * (a.woff + to_f32(((const WT*)a.w)[d]));
    if (gr) o *= sigmoid_f(to_f32(gr[d]));
    if (rr) {
      o = fmaf(a.mult, o, rr[d]);
      if (a.sum) a.sum[row * a.ss + d] = o;          // (element d of the residual row is read by this thread only)
    }
    if (a.y) ((YT*)a.y)[row * a.ys + d] = from_f32<YT>(o);
    if (a.y2) ((YT*)a.y2)[(int64_t)a.y2_rows[row] * a.y2s + d] = from_f32<YT>(o);
  }
}

// rows of an embedding table times a constant, in fp32 (the residual stream) and in the model's dtype; with a position table
// its row of the token's place in the sequence is added: place = start[b] + row - cu[b], b = seq[row]
template <typename T>
__global__ __launch_bounds__(RX_THREADS) void embed_scaled_kernel(const int64_t* __restrict__ ids, const T* __restrict__ table,
                                                                  float* __restrict__ x, T* __restrict__ h, int D, int64_t vocab,
                                                                  float scale, const T* __restrict__ pos, const int* __restrict__ seq,
                                                                  const int* __restrict__ cu, const int* __restrict__ start,
                                                                  int64_t max_pos, int vec) {
  const int64_t row = blockIdx.x, id = ids[row];
  const bool ok = id >= 0 && id < vocab;             // (callers check on the host; a bad id or place reads nothing)
  int64_t at = -1;
  if (pos) {
    const int b = seq[row];
    at = (int64_t)start[b] + row - cu[b];
    if (at >= max_pos) at = -1;
  }
  if (vec) {
    for (int iv = threadIdx.x; iv < D / 8; iv += RX_THREADS) {
      float v[8] = {0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f}, p[8];
      if (ok) load8<T>(table + id * D + 8 * iv, v);
#pragma unroll
      for (int i = 0; i < 8; ++i) v[i] *= scale;
      if (at >= 0) {
        load8<T>(pos + at * D + 8 * iv, p);
#pragma unroll
        for (int i = 0; i < 8; ++i) v[i] += p[i];
      }
      store8<float>(x + row * D + 8 * iv, v);
      if (h) store8<T>(h + row * D + 8 * iv, v);
    }
    return;
  }
  for (int d = threadIdx.x; d < D; d += RX_THREADS) {
    float v = ok ? to_f32(table[id * D + d]) * scale : 0.f;
    if (at >= 0) v += to_f32(pos[at * D + d]);
    x[row * D + d] = v;
    if (h) h[row * D + d] = from_f32<T>(v);
  }
}

bool al16(const void* p) { return ((uintptr_t)p & 15) == 0; }

template <typename XT, typename WT, typename YT, bool MOE>
int launch(const RxArgs& a, int64_t rows, hipStream_t st) {
  const bool vec = a.D % 8 == 0 && a.D <= 8 * RX_MAXV * RX_THREADS && al16(a.x) && al16(a.w) && al16(a.gate) && al16(a.res) &&
                   al16(a.sum) && al16(a.y) && al16(a.y2) && a.y2s % 8 == 0 && a.xs % 8 == 0 && a.gs % 8 == 0 && a.rs % 4 == 0 && a.ss % 4 == 0 && a.ys % 8 == 0;
  if (vec) rmsnorm_ex_kernel<XT, WT, YT, MOE><<<dim3((unsigned)rows), RX_THREADS, 0, st>>>(a);
  else rmsnorm_ex_scalar_kernel<XT, WT, YT, MOE><<<dim3((unsigned)rows), RX_THREADS, 0, st>>>(a);
  TV_LAUNCH_CHECK();
}

template <bool MOE>
int dispatch(const RxArgs& a, int64_t rows, int x_dtype, int w_dtype, int y_dtype, hipStream_t st) {
  if (w_dtype == TV_BF16) {
    if (x_dtype == TV_BF16 && y_dtype == TV_BF16) return launch<bf16_t, bf16_t, bf16_t, MOE>(a, rows, st);
    if (x_dtype == TV_F32 && y_dtype == TV_BF16) return launch<float, bf16_t, bf16_t, MOE>(a, rows, st);
    if (x_dtype == TV_BF16 && y_dtype == TV_F32) return launch<bf16_t, bf16_t, float, MOE>(a, rows, st);
    if (x_dtype == TV_F32 && y_dtype == TV_F32) return launch<float, bf16_t, float, MOE>(a, rows, st);
  } else if (w_dtype == TV_F32 && x_dtype == TV_F32 && y_dtype == TV_F32) {
    return launch<float, float, float, MOE>(a, rows, st);
  }
  TV_UNSUPPORTED("rmsnorm_ex: dtypes x %d w %d y %d", x_dtype, w_dtype, y_dtype);
}

}  // namespace

extern "C" int tv_rmsnorm_ex_fwd(const void* x, const void* weight, const void* gate, const float* residual, float* sum, void* y,
                                 void* y2, const int* y2_rows, int64_t y2_stride, int64_t rows, int D, int64_t x_stride, int64_t gate_stride, int64_t residual_stride,
                                 int64_t sum_stride, int64_t y_stride, float eps, float mult, float weight_offset, int x_dtype,
                                 int weight_dtype, int y_dtype, void* stream) {
  TV_CHECK_ARG(rows >= 0 && rows < (1ll << 31) && D > 0, "rmsnorm_ex: bad sizes");
  if (rows == 0) return TV_OK;
  TV_CHECK_ARG(x && weight && (y || sum || y2) && (!sum || residual) && (!y2 || y2_rows), "rmsnorm_ex: null pointer");
  RxArgs a{x, weight, gate, residual, sum, y, y2, y2_rows, nullptr, nullptr, D, 0, x_stride, gate_stride, residual_stride, sum_stride,
           y_stride, y2_stride, eps, mult, weight_offset};
  return dispatch<false>(a, rows, x_dtype, weight_dtype, y_dtype, (hipStream_t)stream);
}

extern "C" int tv_moe_combine_norm_fwd(const void* expert_out, const int* pos, const float* weights, int top, const float* residual,
                                       const void* norm_weight, float* sum, void* y, int64_t rows, int D, int64_t out_stride,
                                       int64_t residual_stride, int64_t sum_stride, int64_t y_stride, float eps, float mult,
                                       float weight_offset, int out_dtype, int weight_dtype, int y_dtype, void* stream) {
  TV_CHECK_ARG(rows >= 0 && rows < (1ll << 31) && D > 0 && top > 0 && top <= RX_MAXTOP, "moe_combine_norm: bad sizes");
  if (rows == 0) return TV_OK;
  TV_CHECK_ARG(expert_out && pos && weights && residual && norm_weight && (y || sum), "moe_combine_norm: null pointer");
  RxArgs a{expert_out, norm_weight, nullptr, residual, sum, y, nullptr, nullptr, pos, weights, D, top, out_stride, 0, residual_stride,
           sum_stride, y_stride, 0, eps, mult, weight_offset};
  return dispatch<true>(a, rows, out_dtype, weight_dtype, y_dtype, (hipStream_t)stream);
}

extern "C" int tv_embed_scaled_fwd(const int64_t* ids, const void* table, float* x, void* h, int64_t rows, int D, int64_t vocab,
                                   float scale, const void* pos, const int* seq, const int* cu, const int* start, int64_t max_pos,
                                   int dtype, void* stream) {
  TV_CHECK_ARG(rows >= 0 && rows < (1ll << 31) && D > 0 && vocab > 0, "embed_scaled: bad sizes");
  if (rows == 0) return TV_OK;
  TV_CHECK_ARG(ids && table && x && (!pos || (seq && cu && start && max_pos > 0)), "embed_scaled: null pointer");
  hipStream_t st = (hipStream_t)stream;
  const dim3 grid((unsigned)rows);
  const int vec = D % 8 == 0 && al16(table) && al16(x) && al16(h) && al16(pos);
  if (dtype == TV_F32)
    embed_scaled_kernel<float><<<grid, RX_THREADS, 0, st>>>(ids, (const float*)table, x, (float*)h, D, vocab, scale, (const float*)pos, seq, cu, start, max_pos, vec);
  else if (dtype == TV_BF16)
    embed_scaled_kernel<bf16_t><<<grid, RX_THREADS, 0, st>>>(ids, (const bf16_t*)table, x, (bf16_t*)h, D, vocab, scale, (const bf16_t*)pos, seq, cu, start, max_pos, vec);
  else TV_UNSUPPORTED("embed_scaled: dtype %d", dtype);
  TV_LAUNCH_CHECK();
}
