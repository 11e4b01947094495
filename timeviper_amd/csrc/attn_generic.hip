// Softmax attention for every shape and for 32-bit models: any query / key dimension, any value dimension, fp32 or bf16
// operands, key / value heads shared by groups of query heads, an optional sink per query head, ragged batches.
// One work-group per (query row, head): 256 keys at a time — a thread scores one key — with an online softmax; scores,
// weights and sums are fp32.  The matrix-core kernels (attention.hip, latent_decode.hip) take the shapes they are written
// for; this is the form that has no shape limits beyond 1 024 value dimensions.
//
// Sequence b owns query rows [cu_q[b], cu_q[b + 1]); its keys are rows [0, start[b] + i] of key block slot[b] for its i-th
// query row when causal (start: the tokens that were there before), all start[b] + n_b keys otherwise.
// A sink is a learned logit without key or value: exp(sink_h) is one more term of the denominator, not scaled.
// Causal with a window: position p sees keys (p - window, p] and the first `keep` keys of its sequence; the loop runs over the
// visible keys only.  gate: the output is multiplied by sigmoid(gate), element by element.
#include "common.hpp"

namespace {

constexpr int AG_THREADS = 256;
constexpr int AG_MAXNV = 4;        // value dims per thread: vdim <= 1 024

struct AgArgs {
  const void *q, *k, *v;
  const float* sink;
  void* o;
  const int *cu_q, *start, *slot;
  int nseq, H, gq, dk, dv, causal, window, keep;
  int64_t qsl, qsh, ksb, ksl, ksh, vsb, vsl, vsh, osl, osh;
  float scale;
  const void* gate;
  int64_t gsl, gsh;
};

template <typename T>
__global__ __launch_bounds__(AG_THREADS) void attn_generic_kernel(AgArgs a) {
  extern __shared__ __attribute__((aligned(16))) float ag_smem[];
  float* sq = ag_smem;                         // [dk]
  float* sp = sq + (a.dk + 3) / 4 * 4;         // [256]
  float* sacc = sp + AG_THREADS;               // [256]
  __shared__ float red[AG_THREADS / 64];
  const int tid = threadIdx.x, h = blockIdx.y;
  const int row = blockIdx.x;
  int b = 0;
  while (b + 1 < a.nseq && row >= a.cu_q[b + 1]) ++b;
  const int n_b = a.cu_q[b + 1] - a.cu_q[b], i = row - a.cu_q[b], st = a.start ? a.start[b] : 0;
  const int end = a.causal ? st + i + 1 : st + n_b;
  const int lo = a.causal ? max(0, end - a.window) : 0, kept = min(a.keep, lo);      // keys [0, kept) and [lo, end)
  const int nk = kept + end - lo, skip = lo - kept;                                  // visible key j: j, or j + skip from kept on
  const int64_t blk = a.slot ? a.slot[b] : b;
  const T* kb = (const T*)a.k + blk * a.ksb + (int64_t)(h / a.gq) * a.ksh;
  const T* vb = (const T*)a.v + blk * a.vsb + (int64_t)(h / a.gq) * a.vsh;
  const T* qr = (const T*)a.q + (int64_t)row * a.qsl + (int64_t)h * a.qsh;
  for (int d = tid; d < a.dk; d += AG_THREADS) sq[d] = to_f32(qr[d]);
  // value phase: `wid` threads side by side own the value dims (dims vd, vd + wid, ... when vdim > 256), groups split the keys
  int wid = 1;
  while (wid < a.dv && wid < AG_THREADS) wid <<= 1;
  const int ng = AG_THREADS / wid, grp = tid / wid, vd = tid % wid;
  float acc[AG_MAXNV];
#pragma unroll
  for (int j = 0; j < AG_MAXNV; ++j) acc[j] = 0.f;
  float m_run = a.sink ? a.sink[h] : -INFINITY;
  float l_run = a.sink ? 1.f : 0.f;
  __syncthreads();
  for (int k0 = 0; k0 < nk; k0 += AG_THREADS) {
    const int key = k0 + tid;
    float s = -INFINITY;
    if (key < nk) {
      const T* kr = kb + (int64_t)(key < kept ? key : key + skip) * a.ksl;
      float dot = 0.f;
      for (int d = 0; d < a.dk; ++d) dot = fmaf(sq[d], to_f32(kr[d]), dot);
      s = dot * a.scale;
    }
    const float wm = wave_max(s);
    if ((tid & 63) == 0) red[tid >> 6] = wm;
    __syncthreads();
    float m_new = m_run;
#pragma unroll
    for (int w = 0; w < AG_THREADS / 64; ++w) m_new = fmaxf(m_new, red[w]);
    const float alpha = expf(m_run - m_new);             // (m_new is finite: the step holds a key; m_run = -inf gives 0)
    const float p = key < nk ? expf(s - m_new) : 0.f;
    sp[tid] = p;
    const float ws = wave_sum(p);
    __syncthreads();                                     // red has been read, sp is written
    if ((tid & 63) == 0) red[tid >> 6] = ws;
    __syncthreads();
    float tot = 0.f;
#pragma unroll
    for (int w = 0; w < AG_THREADS / 64; ++w) tot += red[w];
    l_run = l_run * alpha + tot;
    m_run = m_new;
#pragma unroll
    for (int j = 0; j < AG_MAXNV; ++j) acc[j] *= alpha;
    const int kn = min(AG_THREADS, nk - k0);
    for (int kk = grp; kk < kn; kk += ng) {
      const float pk = sp[kk];
      const T* vr = vb + (int64_t)(k0 + kk < kept ? k0 + kk : k0 + kk + skip) * a.vsl;
#pragma unroll
      for (int j = 0; j < AG_MAXNV; ++j) {
        const int d = vd + j * wid;
        if (d < a.dv) acc[j] = fmaf(pk, to_f32(vr[d]), acc[j]);
      }
    }
    __syncthreads();                                     // sp and red are written again in the next step
  }
  const float inv = l_run > 0.f ? 1.f / l_run : 0.f;
  T* orow = (T*)a.o + (int64_t)row * a.osl + (int64_t)h * a.osh;
#pragma unroll
  for (int j = 0; j < AG_MAXNV; ++j) {
    if (j * wid < a.dv) {                                // (uniform over the work-group)
      sacc[tid] = acc[j];
      __syncthreads();
      if (grp == 0) {
        float t = 0.f;
        for (int g = 0; g < ng; ++g) t += sacc[g * wid + vd];
        const int d = vd + j * wid;
        if (d < a.dv) {
          t *= inv;
          if (a.gate) t *= sigmoid_f(to_f32(((const T*)a.gate)[(int64_t)row * a.gsl + (int64_t)h * a.gsh + d]));
          orow[d] = from_f32<T>(t);
        }
      }
      __syncthreads();
    }
  }
}

}  // namespace

extern "C" int tv_attn_generic_fwd(const void* q, const void* k, const void* v, const float* sink, void* o, const int* cu_q,
                                   const int* start, const int* slot, int nseq, int64_t rows, int nheads_q, int nheads_kv,
                                   int qk_dim, int v_dim, int64_t q_stride_l, int64_t q_stride_h, int64_t k_stride_b,
                                   int64_t k_stride_l, int64_t k_stride_h, int64_t v_stride_b, int64_t v_stride_l,
                                   int64_t v_stride_h, int64_t o_stride_l, int64_t o_stride_h, float softmax_scale, int causal,
                                   int window, int keep_first, const void* gate, int64_t gate_stride_l, int64_t gate_stride_h,
                                   int dtype, void* stream) {
  TV_CHECK_ARG(nseq > 0 && rows >= 0 && rows < (1ll << 31) && nheads_q > 0 && nheads_kv > 0 && nheads_q % nheads_kv == 0 &&
                   qk_dim > 0 && v_dim > 0 && window > 0 && keep_first >= 0, "attn_generic: bad sizes");
  if (rows == 0) return TV_OK;
  TV_CHECK_ARG(q && k && v && o && cu_q, "attn_generic: null pointer");
  if (dtype != TV_F32 && dtype != TV_BF16) TV_UNSUPPORTED("attn_generic: dtype must be fp32 or bf16");
  if (v_dim > AG_THREADS * AG_MAXNV || qk_dim > 4096) TV_UNSUPPORTED("attn_generic: qk_dim %d / v_dim %d", qk_dim, v_dim);
  AgArgs a{q, k, v, sink, o, cu_q, start, slot, nseq, nheads_q, nheads_q / nheads_kv, qk_dim, v_dim, causal, window, keep_first,
           q_stride_l, q_stride_h, k_stride_b, k_stride_l, k_stride_h, v_stride_b, v_stride_l, v_stride_h, o_stride_l, o_stride_h,
           softmax_scale, gate, gate_stride_l, gate_stride_h};
  const size_t lds = ((qk_dim + 3) / 4 * 4 + 2 * AG_THREADS) * sizeof(float);
  const dim3 grid((unsigned)rows, (unsigned)nheads_q);
  if (dtype == TV_F32) attn_generic_kernel<float><<<grid, AG_THREADS, lds, (hipStream_t)stream>>>(a);
  else attn_generic_kernel<bf16_t><<<grid, AG_THREADS, lds, (hipStream_t)stream>>>(a);
  TV_LAUNCH_CHECK();
}
