// Row operators of language models whose two sublayers run in parallel on a 32-bit residual stream:
//
//   residual_add   x' = x + u, fp32, and its rounding to the model's dtype
//   norm_shift     x' = x + y / rms(y) * w        (what waits from the operator in front: its norm and residual add; optional)
//                  h  = x' / rms(x') * g          (one gain for all coordinates)
//                  hs = h + (h_before - h) * s    (token shift: h_before is the h of the sequence's previous token; optional)
//   gated_mul      f(a) * b, the rows of b optionally gathered by token id
//   scatter_rows   rows of a projection to the rows of a cache
//
// norm_shift keeps the h of the last token between steps in fp32: state (slots, 2, D), row p & 1 holds the h of position p, so a
// single token reads one row and writes the other.  Statistics, sums, the shift and the state are fp32.  A group of one or four
// waves walks `run` consecutive rows with the row in registers; the row in front of the first is computed again.  The group that
// holds the FIRST row of a sequence's portion reads the carried h and also writes the new one (it computes the portion's last
// row for that), so nobody overwrites a row that another group still has to read.
#include "common.hpp"

namespace {

constexpr int SO_THREADS = 256;

template <typename T> __device__ __forceinline__ void so_load8(const T* p, float (&o)[8]);
template <> __device__ __forceinline__ void so_load8<float>(const float* p, float (&o)[8]) {
  const f32x4 a = *(const f32x4*)p, b = *(const f32x4*)(p + 4);
#pragma unroll
  for (int i = 0; i < 4; ++i) { o[i] = a[i]; o[4 + i] = b[i]; }
}
template <> __device__ __forceinline__ void so_load8<bf16_t>(const bf16_t* p, float (&o)[8]) {
  const bf16x8 a = *(const bf16x8*)p;
#pragma unroll
  for (int i = 0; i < 8; ++i) o[i] = (float)a[i];
}
template <typename T> __device__ __forceinline__ void so_store8(T* p, const float (&o)[8]);
template <> __device__ __forceinline__ void so_store8<float>(float* p, const float (&o)[8]) {
  *(f32x4*)p = f32x4{o[0], o[1], o[2], o[3]};
  *(f32x4*)(p + 4) = f32x4{o[4], o[5], o[6], o[7]};
}
template <> __device__ __forceinline__ void so_store8<bf16_t>(bf16_t* p, const float (&o)[8]) {
  bf16x8 v;
#pragma unroll
  for (int i = 0; i < 8; ++i) v[i] = (bf16_t)o[i];
  *(bf16x8*)p = v;
}

// ---------------------------------------------------------------- norm, token shift
struct NsArgs {
  const float* x;          // (rows, D) dense
  const void *y, *yw;      // (rows, D) and (D): the waiting sublayer output and its norm weight, or NULL
  float* x_out;            // (rows, D) or NULL
  const void *gain, *shift;
  float* state;            // (slots, 2, D) blocks, `ss` floats apart
  const int *seq, *cu, *start, *slot;
  void *h, *hs;
  int rows, D, run, single;          // single: one row per sequence
  int64_t ys, ss;
  float eps;
};

template <int WAVES>
__device__ __forceinline__ float so_total(float v, float* red) {
  v = wave_sum_dpp(v);
  if constexpr (WAVES == 1) return v;
  __syncthreads();                                   // (red is used again)
  if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = v;
  __syncthreads();
  float t = 0.f;
#pragma unroll
  for (int i = 0; i < WAVES; ++i) t += red[i];
  return t;
}

template <typename T, int NP, int WAVES>
__global__ __launch_bounds__(SO_THREADS) void norm_shift_kernel(NsArgs a) {
  constexpr int G = 64 * WAVES;
  __shared__ float red[4];
  const int lt = threadIdx.x % G;
  const int grp = WAVES == 1 ? __builtin_amdgcn_readfirstlane((int)(blockIdx.x * 4 + (threadIdx.x >> 6))) : (int)blockIdx.x;
  const int t0 = grp * a.run, t1 = min(t0 + a.run, a.rows);
  if (t0 >= a.rows) return;
  const int nv = a.D / 8;
  const float gain = to_f32(*(const T*)a.gain), inv_d = 1.f / (float)a.D;

  auto row_h = [&](int t, float (&o)[NP][8], bool keep) __attribute__((always_inline)) {
    const float* xr = a.x + (int64_t)t * a.D;
    float ssq = 0.f;
#pragma unroll
    for (int k = 0; k < NP; ++k) {
      const int iv = lt + k * G;
      if (iv < nv) so_load8<float>(xr + 8 * iv, o[k]);
    }
    if (a.y) {
      const T* yr = (const T*)a.y + (int64_t)t * a.ys;
      float y[NP][8];
#pragma unroll
      for (int k = 0; k < NP; ++k) {
        const int iv = lt + k * G;
        if (iv < nv) {
          so_load8<T>(yr + 8 * iv, y[k]);
#pragma unroll
          for (int i = 0; i < 8; ++i) ssq = fmaf(y[k][i], y[k][i], ssq);
        }
      }
      const float r = rsqrtf(so_total<WAVES>(ssq, red) * inv_d + a.eps);
      ssq = 0.f;
#pragma unroll
      for (int k = 0; k < NP; ++k) {
        const int iv = lt + k * G;
        if (iv < nv) {
          float w[8];
          so_load8<T>((const T*)a.yw + 8 * iv, w);
#pragma unroll
          for (int i = 0; i < 8; ++i) o[k][i] = fmaf(y[k][i] * r, w[i], o[k][i]);
          if (keep && a.x_out) so_store8<float>(a.x_out + (int64_t)t * a.D + 8 * iv, o[k]);
        }
      }
    }
#pragma unroll
    for (int k = 0; k < NP; ++k)
      if (lt + k * G < nv) {
#pragma unroll
        for (int i = 0; i < 8; ++i) ssq = fmaf(o[k][i], o[k][i], ssq);
      }
    const float r = rsqrtf(so_total<WAVES>(ssq, red) * inv_d + a.eps) * gain;
#pragma unroll
    for (int k = 0; k < NP; ++k)
#pragma unroll
      for (int i = 0; i < 8; ++i) o[k][i] *= r;
  };
  auto put_state = [&](const float (&v)[NP][8], int b, int p) __attribute__((always_inline)) {
    float* sr = a.state + (int64_t)a.slot[b] * a.ss + (int64_t)(p & 1) * a.D;
#pragma unroll
    for (int k = 0; k < NP; ++k)
      if (lt + k * G < nv) so_store8<float>(sr + 8 * (lt + k * G), v[k]);
  };

  float before[NP][8];
  for (int t = t0; t < t1; ++t) {
    float cur[NP][8];
    bool first = false;
    int b = 0, st = 0;
    if (a.shift) {
      b = a.single ? t : a.seq[t];
      first = a.single || t == a.cu[b];
      if (first) {
        st = a.start[b];
        const float* sr = a.state + (int64_t)a.slot[b] * a.ss + (int64_t)((st - 1) & 1) * a.D;
#pragma unroll
        for (int k = 0; k < NP; ++k) {
#pragma unroll
          for (int i = 0; i < 8; ++i) before[k][i] = 0.f;
          if (st > 0 && lt + k * G < nv) so_load8<float>(sr + 8 * (lt + k * G), before[k]);
        }
      } else if (t == t0) {
        row_h(t - 1, before, false);
      }
    }
    row_h(t, cur, true);
#pragma unroll
    for (int k = 0; k < NP; ++k) {
      const int iv = lt + k * G;
      if (iv < nv) {
        if (a.h) so_store8<T>((T*)a.h + (int64_t)t * a.D + 8 * iv, cur[k]);
        if (a.shift) {
          float s[8];
          so_load8<T>((const T*)a.shift + 8 * iv, s);
#pragma unroll
          for (int i = 0; i < 8; ++i) s[i] = fmaf(before[k][i] - cur[k][i], s[i], cur[k][i]);
          so_store8<T>((T*)a.hs + (int64_t)t * a.D + 8 * iv, s);
        }
      }
    }
    if (first) {
      const int last = a.single ? t : a.cu[b + 1] - 1, p = st + last - t;
      if (last == t) {
        put_state(cur, b, p);
      } else {
        row_h(last, before, false);
        put_state(before, b, p);
      }
    }
#pragma unroll
    for (int k = 0; k < NP; ++k)
#pragma unroll
      for (int i = 0; i < 8; ++i) before[k][i] = cur[k][i];
  }
}

// any width and alignment: a work-group per row, the row is read again in every pass
template <typename T>
__global__ __launch_bounds__(SO_THREADS) void norm_shift_scalar_kernel(NsArgs a) {
  __shared__ float red[4];
  const int t = blockIdx.x;
  const float gain = to_f32(*(const T*)a.gain), inv_d = 1.f / (float)a.D;
  float ry = 0.f;
  auto value = [&](int row, float r, int d) {
    const float x = a.x[(int64_t)row * a.D + d];
    return a.y ? fmaf(to_f32(((const T*)a.y)[(int64_t)row * a.ys + d]) * r, to_f32(((const T*)a.yw)[d]), x) : x;
  };
  // (scale of the waiting output, scale of the norm) of a row
  auto stats = [&](int row, float& r1, float& r2) {
    float s = 0.f;
    if (a.y) {
      for (int d = threadIdx.x; d < a.D; d += SO_THREADS) {
        const float y = to_f32(((const T*)a.y)[(int64_t)row * a.ys + d]);
        s = fmaf(y, y, s);
      }
      r1 = rsqrtf(so_total<4>(s, red) * inv_d + a.eps);
    }
    s = 0.f;
    for (int d = threadIdx.x; d < a.D; d += SO_THREADS) {
      const float v = value(row, r1, d);
      s = fmaf(v, v, s);
    }
    r2 = rsqrtf(so_total<4>(s, red) * inv_d + a.eps) * gain;
  };
  float rn, by = 0.f, bn = 0.f, ly = 0.f, ln = 0.f;
  stats(t, ry, rn);
  int b = 0, st = 0, last = t;
  bool first = false;
  if (a.shift) {
    b = a.seq[t];
    first = t == a.cu[b];
    st = a.start[b];
    last = a.cu[b + 1] - 1;
    if (!first) stats(t - 1, by, bn);
    else if (last != t) stats(last, ly, ln);
  }
  float* sl = a.shift ? a.state + (int64_t)a.slot[b] * a.ss : nullptr;
  for (int d = threadIdx.x; d < a.D; d += SO_THREADS) {
    const float x = value(t, ry, d), h = x * rn;
    if (a.x_out) a.x_out[(int64_t)t * a.D + d] = x;
    if (a.h) ((T*)a.h)[(int64_t)t * a.D + d] = from_f32<T>(h);
    if (a.shift) {
      float before = 0.f;
      if (!first) before = value(t - 1, by, d) * bn;
      else if (st > 0) before = sl[(int64_t)((st - 1) & 1) * a.D + d];
      ((T*)a.hs)[(int64_t)t * a.D + d] = from_f32<T>(fmaf(before - h, to_f32(((const T*)a.shift)[d]), h));
      if (first) sl[(int64_t)((st + last - t) & 1) * a.D + d] = last == t ? h : value(last, ly, d) * ln;
    }
  }
}

template <typename T, int NP, int WAVES>
void launch_ns(const NsArgs& a, hipStream_t st) {
  const int groups = (a.rows + a.run - 1) / a.run;
  norm_shift_kernel<T, NP, WAVES><<<dim3((unsigned)(WAVES == 1 ? (groups + 3) / 4 : groups)), SO_THREADS, 0, st>>>(a);
}

bool al16(const void* p) { return ((uintptr_t)p & 15) == 0; }

template <typename T>
int norm_shift(NsArgs a, hipStream_t st) {
  const int np = (a.D + 511) / 512;
  const bool vec = a.D % 8 == 0 && np <= 16 && al16(a.x) && al16(a.y) && al16(a.yw) && al16(a.x_out) && al16(a.shift) && al16(a.state) &&
                   al16(a.h) && al16(a.hs) && a.ys % 8 == 0 && a.ss % 4 == 0;
  if (!vec) {
    norm_shift_scalar_kernel<T><<<dim3((unsigned)a.rows), SO_THREADS, 0, st>>>(a);
  } else {
    a.run = a.shift == nullptr || a.rows < 2048 ? 1 : a.rows < 8192 ? 2 : 4;
    if (np <= 1) launch_ns<T, 1, 1>(a, st);
    else if (np <= 2) launch_ns<T, 2, 1>(a, st);
    else if (np <= 4) launch_ns<T, 1, 4>(a, st);
    else if (np <= 8) launch_ns<T, 2, 4>(a, st);
    else launch_ns<T, 4, 4>(a, st);
  }
  TV_LAUNCH_CHECK();
}

// ---------------------------------------------------------------- elementwise
template <typename T>
__global__ __launch_bounds__(SO_THREADS) void residual_add_kernel(const float* __restrict__ x, const T* __restrict__ u, float* __restrict__ xo,
                                                                  T* __restrict__ h, int64_t n, int D, int64_t us, int vec) {
  const int64_t i = (int64_t)blockIdx.x * SO_THREADS + threadIdx.x;
  if (vec) {
    if (8 * i >= n) return;
    const int64_t row = 8 * i / D, c = 8 * i - row * D;
    float a[8], b[8];
    so_load8<float>(x + 8 * i, a);
    so_load8<T>(u + row * us + c, b);
#pragma unroll
    for (int j = 0; j < 8; ++j) a[j] += b[j];
    so_store8<float>(xo + 8 * i, a);
    if (h) so_store8<T>(h + 8 * i, a);
  } else {
    if (i >= n) return;
    const int64_t row = i / D, c = i - row * D;
    const float v = x[i] + to_f32(u[row * us + c]);
    xo[i] = v;
    if (h) h[i] = from_f32<T>(v);
  }
}

enum { GM_SIGMOID = 0, GM_GELU_TANH = 1 };
template <typename T>
__global__ __launch_bounds__(SO_THREADS) void gated_mul_kernel(const T* __restrict__ a, const T* __restrict__ b, const int64_t* __restrict__ ids,
                                                               T* __restrict__ o, unsigned n, unsigned nc, int64_t as, int64_t bs, int64_t os,
                                                               int64_t b_rows, int act, int vec) {
  const unsigned i = blockIdx.x * SO_THREADS + threadIdx.x;
  if (i >= n) return;
  const unsigned row = i / nc, c = i - row * nc;
  const int64_t rb = ids ? ids[row] : row;
  const bool ok = rb >= 0 && rb < b_rows;            // (callers check ids on the host; a bad one reads nothing)
  if (vec) {
    float u[8], v[8] = {0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f};
    so_load8<T>(a + row * as + 8 * c, u);
    if (ok) so_load8<T>(b + rb * bs + 8 * c, v);
#pragma unroll
    for (int j = 0; j < 8; ++j) u[j] = (act == GM_SIGMOID ? sigmoid_f(u[j]) : gelu_tanh_f(u[j])) * v[j];
    so_store8<T>(o + row * os + 8 * c, u);
  } else {
    const float u = to_f32(a[row * as + c]), v = ok ? to_f32(b[rb * bs + c]) : 0.f;
    o[row * os + c] = from_f32<T>((act == GM_SIGMOID ? sigmoid_f(u) : gelu_tanh_f(u)) * v);
  }
}

template <typename T>
__global__ __launch_bounds__(SO_THREADS) void scatter_rows_kernel(const T* __restrict__ s, const int* __restrict__ rows, T* __restrict__ d,
                                                                  unsigned n, unsigned nc, int64_t ss, int64_t ds, int vec) {
  typedef typename Vec16<T>::type vec_t;
  constexpr int V = Vec16<T>::N;
  const unsigned i = blockIdx.x * SO_THREADS + threadIdx.x;
  if (i >= n) return;
  const unsigned row = i / nc, c = i - row * nc;
  const int64_t to = rows[row];
  if (vec) *(vec_t*)(d + to * ds + (int64_t)V * c) = *(const vec_t*)(s + row * ss + (int64_t)V * c);
  else d[to * ds + c] = s[row * ss + c];
}

bool fits(int64_t n) { return n < (1ll << 31); }

}  // namespace

extern "C" int tv_norm_shift_fwd(const float* x, const void* y, const void* y_weight, float* x_out, const void* gain, const void* shift,
                                 float* state, const int* seq, const int* cu, const int* start, const int* slot, void* h, void* hs,
                                 int64_t rows, int D, int64_t y_stride, int64_t state_stride, float eps, int single, int dtype, void* stream) {
  TV_CHECK_ARG(rows >= 0 && fits(rows) && D > 0, "norm_shift: bad sizes");
  if (rows == 0) return TV_OK;
  TV_CHECK_ARG(x && gain && (h || hs) && (!y || y_weight) && (!x_out || y), "norm_shift: null pointer");
  TV_CHECK_ARG(!shift || (state && seq && cu && start && slot && hs), "norm_shift: the token shift needs its state and the plan of the step");
  TV_CHECK_ARG(x_out != x, "norm_shift: x is not updated in place (rows are read by their neighbours)");
  NsArgs a{x, y, y_weight, x_out, gain, shift, state, seq, cu, start, slot, h, hs, (int)rows, D, 1, single, y_stride, state_stride, eps};
  if (dtype == TV_F32) return norm_shift<float>(a, (hipStream_t)stream);
  if (dtype == TV_BF16) return norm_shift<bf16_t>(a, (hipStream_t)stream);
  TV_UNSUPPORTED("norm_shift: dtype %d", dtype);
}

extern "C" int tv_residual_add_fwd(const float* x, const void* u, float* x_out, void* h, int64_t rows, int D, int64_t u_stride, int dtype,
                                   void* stream) {
  TV_CHECK_ARG(rows >= 0 && D > 0, "residual_add: bad sizes");
  if (rows == 0) return TV_OK;
  TV_CHECK_ARG(x && u && x_out, "residual_add: null pointer");
  const int vec = D % 8 == 0 && u_stride % 8 == 0 && al16(x) && al16(u) && al16(x_out) && al16(h);
  const int64_t n = rows * D, items = vec ? n / 8 : n;
  TV_CHECK_ARG(fits(items), "residual_add: too many elements");
  const dim3 grid((unsigned)((items + SO_THREADS - 1) / SO_THREADS));
  hipStream_t st = (hipStream_t)stream;
  if (dtype == TV_F32) residual_add_kernel<float><<<grid, SO_THREADS, 0, st>>>(x, (const float*)u, x_out, (float*)h, n, D, u_stride, vec);
  else if (dtype == TV_BF16) residual_add_kernel<bf16_t><<<grid, SO_THREADS, 0, st>>>(x, (const bf16_t*)u, x_out, (bf16_t*)h, n, D, u_stride, vec);
  else TV_UNSUPPORTED("residual_add: dtype %d", dtype);
  TV_LAUNCH_CHECK();
}

extern "C" int tv_gated_mul_fwd(const void* a, const void* b, const int64_t* b_ids, void* o, int64_t rows, int cols, int64_t a_stride,
                                int64_t b_stride, int64_t o_stride, int64_t b_rows, int act, int dtype, void* stream) {
  TV_CHECK_ARG(rows >= 0 && cols > 0 && b_rows > 0, "gated_mul: bad sizes");
  if (rows == 0) return TV_OK;
  TV_CHECK_ARG(a && b && o, "gated_mul: null pointer");
  TV_CHECK_ARG(act == GM_SIGMOID || act == GM_GELU_TANH, "gated_mul: activation %d", act);
  const int vec = cols % 8 == 0 && a_stride % 8 == 0 && b_stride % 8 == 0 && o_stride % 8 == 0 && al16(a) && al16(b) && al16(o);
  const int nc = vec ? cols / 8 : cols;
  TV_CHECK_ARG(fits(rows * nc), "gated_mul: too many elements");
  const unsigned n = (unsigned)(rows * nc);
  const dim3 grid((n + SO_THREADS - 1) / SO_THREADS);
  hipStream_t st = (hipStream_t)stream;
  if (dtype == TV_F32)
    gated_mul_kernel<float><<<grid, SO_THREADS, 0, st>>>((const float*)a, (const float*)b, b_ids, (float*)o, n, nc, a_stride, b_stride, o_stride, b_rows, act, vec);
  else if (dtype == TV_BF16)
    gated_mul_kernel<bf16_t><<<grid, SO_THREADS, 0, st>>>((const bf16_t*)a, (const bf16_t*)b, b_ids, (bf16_t*)o, n, nc, a_stride, b_stride, o_stride, b_rows, act, vec);
  else TV_UNSUPPORTED("gated_mul: dtype %d", dtype);
  TV_LAUNCH_CHECK();
}

extern "C" int tv_scatter_rows(const void* src, const int* rows_to, void* dst, int64_t rows, int cols, int64_t src_stride, int64_t dst_stride,
                               int dtype, void* stream) {
  TV_CHECK_ARG(rows >= 0 && cols > 0, "scatter_rows: bad sizes");
  if (rows == 0) return TV_OK;
  TV_CHECK_ARG(src && rows_to && dst, "scatter_rows: null pointer");
  hipStream_t st = (hipStream_t)stream;
  const int V = dtype == TV_F32 ? 4 : 8;
  const int vec = cols % V == 0 && src_stride % V == 0 && dst_stride % V == 0 && al16(src) && al16(dst);
  const int nc = vec ? cols / V : cols;
  TV_CHECK_ARG(fits(rows * nc), "scatter_rows: too many elements");
  const unsigned n = (unsigned)(rows * nc);
  const dim3 grid((n + SO_THREADS - 1) / SO_THREADS);
  if (dtype == TV_F32) scatter_rows_kernel<float><<<grid, SO_THREADS, 0, st>>>((const float*)src, rows_to, (float*)dst, n, nc, src_stride, dst_stride, vec);
  else if (dtype == TV_BF16) scatter_rows_kernel<bf16_t><<<grid, SO_THREADS, 0, st>>>((const bf16_t*)src, rows_to, (bf16_t*)dst, n, nc, src_stride, dst_stride, vec);
  else TV_UNSUPPORTED("scatter_rows: dtype %d", dtype);
  TV_LAUNCH_CHECK();
}
