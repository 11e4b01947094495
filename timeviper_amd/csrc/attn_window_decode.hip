// One query token per sequence against a slot cache, with a sliding window and kept first keys (bf16, any head counts, query / key
// and value dims of their own): position p sees keys (p - window, p] and the first `keep` keys of its sequence.
//
// A cache row holds a token's keys and values side by side, [kv heads x dim | kv heads x vdim].  The VISIBLE keys of a sequence
// (kept ones, then the window) are numbered 0 .. n - 1 and split over `nsplit` work-groups per key / value head; a work-group
// serves up to GQ query heads of its key / value head, so a row is read once per GQ heads.  64 keys a round: L lanes hold a key's
// row in 16-byte pieces (keys and values of a round are requested together, ahead of the first product), scores are dot products
// reduced over the L lanes, every wave keeps its own running maximum and sums, and the four waves meet once at the end.  Scores,
// weights and sums are fp32, the weights are not rounded.  With one split the result is written directly; else a second kernel
// merges the splits.  The output gate (o *= sigmoid(gate)) is applied where the result is written.
//
// `fresh`: the step's own keys and values (a projection output).  The work-group that meets the newest key takes it from there and
// writes it to the cache.  Layers that read another layer's cache leave it out: the row is in the cache already.
#include "ssd_common.hpp"

namespace {
using namespace ssdk;

constexpr int WD_THREADS = 256;
constexpr int WD_KEYS = 64;          // keys of a round
constexpr int WD_MAX_SPLIT = 128;
typedef __bf16 bf16x2 __attribute__((ext_vector_type(2)));

struct WdArgs {
  const bf16_t *q, *fresh, *gate;
  bf16_t *cache, *o;
  float *part_o, *part_ml;           // (B, H, nsplit, e) and (B, H, nsplit, 2)
  const int *keys, *slot;
  int H, G, gq, d, e, cap, window, keep, nsplit, hblocks;
  int64_t qs, fs, gs, os;
  float scale_log2;
};

__device__ __forceinline__ float wd_dot8(bf16x8 a, bf16x8 b) {
  float acc = 0.f;
#pragma unroll
  for (int j = 0; j < 4; ++j)
    acc = __builtin_amdgcn_fdot2_f32_bf16(bf16x2{a[2 * j], a[2 * j + 1]}, bf16x2{b[2 * j], b[2 * j + 1]}, acc, false);
  return acc;
}

// visible keys of a sequence that holds nk keys, and the share of a split (whole rounds of a quarter: 16 keys)
struct Visible { int n, kept, skip, chunk; };
__device__ __forceinline__ Visible visible_of(const WdArgs& a, int nk) {
  Visible v;
  const int lo = max(0, nk - a.window);
  v.kept = min(a.keep, lo);
  v.skip = lo - v.kept;
  v.n = nk - v.skip;
  v.chunk = ((v.n + a.nsplit - 1) / a.nsplit + 15) / 16 * 16;
  return v;
}

template <int GQ, int L>
__global__ __launch_bounds__(WD_THREADS) void attn_window_decode_kernel(WdArgs a) {
  constexpr int KPP = WD_THREADS / L;          // keys of a pass over the work-group
  constexpr int NP = WD_KEYS / KPP;            // passes of a round
  constexpr int E = 8 * L;                     // widest value row
  __shared__ float sO[4][GQ][E];
  __shared__ float sM[4][GQ], sL[4][GQ];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int c = tid % L, g = tid / L;          // 16-byte piece of a row, key of a pass
  const int split = blockIdx.x, b = blockIdx.z;
  const int hk = blockIdx.y / a.hblocks, hb = blockIdx.y % a.hblocks;
  const int head0 = hk * a.gq + GQ * hb, nh = min(GQ, a.gq - GQ * hb);
  const int nk = min(a.keys[b], a.cap);
  const Visible vis = visible_of(a, nk);
  const int r0 = split * vis.chunk, r1 = min(vis.n, r0 + vis.chunk);
  if (r0 >= r1) return;                        // (the merge kernel leaves the same splits out)
  const int W = a.G * (a.d + a.e), ko = hk * a.d, vo = a.G * a.d + hk * a.e;
  bf16_t* base = a.cache + (int64_t)a.slot[b] * a.cap * W;
  const bf16_t* fresh = a.fresh ? a.fresh + (int64_t)b * a.fs : nullptr;
  const bool kd = 8 * c < a.d, ve = 8 * c < a.e;
  const bf16x8 zero = {};

  bf16x8 qf[GQ];
#pragma unroll
  for (int h = 0; h < GQ; ++h)
    qf[h] = kd && h < nh ? *(const bf16x8*)(a.q + (int64_t)b * a.qs + (int64_t)(head0 + h) * a.d + 8 * c) : zero;

  float m_run[GQ], l_run[GQ], acc[GQ][8];
#pragma unroll
  for (int h = 0; h < GQ; ++h) {
    m_run[h] = -INFINITY;
    l_run[h] = 0.f;
#pragma unroll
    for (int j = 0; j < 8; ++j) acc[h][j] = 0.f;
  }

  for (int k0 = r0; k0 < r1; k0 += WD_KEYS) {
    bf16x8 kf[NP], vf[NP];
#pragma unroll
    for (int p = 0; p < NP; ++p) {
      const int j = k0 + p * KPP + g, key = j < vis.kept ? j : j + vis.skip;
      kf[p] = zero;
      vf[p] = zero;
      if (j < r1) {
        const bf16_t* row = fresh && key == nk - 1 ? fresh : base + (int64_t)key * W;
        if (kd) kf[p] = *(const bf16x8*)(row + ko + 8 * c);
        if (ve) vf[p] = *(const bf16x8*)(row + vo + 8 * c);
      }
    }
    float s[NP][GQ];
#pragma unroll
    for (int p = 0; p < NP; ++p)
#pragma unroll
      for (int h = 0; h < GQ; ++h) {
        float x = wd_dot8(kf[p], qf[h]);
#pragma unroll
        for (int o = 1; o < L; o <<= 1) x += __shfl_xor(x, o, 64);
        s[p][h] = k0 + p * KPP + g < r1 ? x * a.scale_log2 : -INFINITY;
      }
#pragma unroll
    for (int h = 0; h < GQ; ++h) {
      float m = s[0][h];
#pragma unroll
      for (int p = 1; p < NP; ++p) m = fmaxf(m, s[p][h]);
#pragma unroll
      for (int o = L; o < 64; o <<= 1) m = fmaxf(m, __shfl_xor(m, o, 64));
      const float m_new = fmaxf(m_run[h], m), m_use = m_new == -INFINITY ? 0.f : m_new;      // (a wave may have met no key yet)
      const float alpha = __builtin_amdgcn_exp2f(m_run[h] - m_use);
      m_run[h] = m_new;
      l_run[h] *= alpha;
#pragma unroll
      for (int j = 0; j < 8; ++j) acc[h][j] *= alpha;
#pragma unroll
      for (int p = 0; p < NP; ++p) {
        const float w = __builtin_amdgcn_exp2f(s[p][h] - m_use);
        l_run[h] += w;
#pragma unroll
        for (int j = 0; j < 8; ++j) acc[h][j] = fmaf(w, (float)vf[p][j], acc[h][j]);
      }
    }
    if (fresh && hb == 0 && r1 == vis.n && k0 + WD_KEYS >= r1) {       // the round that holds the newest key
#pragma unroll
      for (int p = 0; p < NP; ++p)
        if (k0 + p * KPP + g == vis.n - 1) {
          bf16_t* row = base + (int64_t)(nk - 1) * W;
          if (kd) *(bf16x8*)(row + ko + 8 * c) = kf[p];
          if (ve) *(bf16x8*)(row + vo + 8 * c) = vf[p];
        }
    }
  }

  // the keys of a wave, then the four waves
#pragma unroll
  for (int h = 0; h < GQ; ++h) {
#pragma unroll
    for (int o = L; o < 64; o <<= 1) {
      l_run[h] += __shfl_xor(l_run[h], o, 64);
#pragma unroll
      for (int j = 0; j < 8; ++j) acc[h][j] += __shfl_xor(acc[h][j], o, 64);
    }
    if (lane < L) {
#pragma unroll
      for (int j = 0; j < 8; ++j) sO[wave][h][8 * lane + j] = acc[h][j];
      if (lane == 0) { sM[wave][h] = m_run[h]; sL[wave][h] = l_run[h]; }
    }
  }
  __syncthreads();
  for (int i = tid; i < nh * a.e; i += WD_THREADS) {
    const int h = i / a.e, x = i - h * a.e;
    float M = sM[0][h];
#pragma unroll
    for (int w = 1; w < 4; ++w) M = fmaxf(M, sM[w][h]);    // (finite: the range holds a key)
    float Lt = 0.f, O = 0.f;
#pragma unroll
    for (int w = 0; w < 4; ++w) {
      const float f = __builtin_amdgcn_exp2f(sM[w][h] - M);
      Lt = fmaf(f, sL[w][h], Lt);
      O = fmaf(f, sO[w][h][x], O);
    }
    const int head = head0 + h;
    if (a.nsplit == 1) {
      float r = O / Lt;
      if (a.gate) r *= sigmoid_f((float)a.gate[(int64_t)b * a.gs + (int64_t)head * a.e + x]);
      a.o[(int64_t)b * a.os + (int64_t)head * a.e + x] = (bf16_t)r;
    } else {
      const int64_t at = ((int64_t)b * a.H + head) * a.nsplit + split;
      a.part_o[at * a.e + x] = O;
      if (x == 0) { a.part_ml[2 * at] = M; a.part_ml[2 * at + 1] = Lt; }
    }
  }
}

// merge of the splits, output gate: a work-group per (head, sequence), a thread per value dim; 8 splits' loads at a time
__global__ __launch_bounds__(WD_THREADS) void attn_window_merge_kernel(WdArgs a) {
  constexpr int U = 8;
  typedef float f32x2 __attribute__((ext_vector_type(2)));
  const int h = blockIdx.x, b = blockIdx.y, x = threadIdx.x;
  if (x >= a.e) return;
  const Visible vis = visible_of(a, min(a.keys[b], a.cap));
  const int n = (vis.n + vis.chunk - 1) / vis.chunk;
  const int64_t at = ((int64_t)b * a.H + h) * a.nsplit;
  const float gt = a.gate ? (float)a.gate[(int64_t)b * a.gs + (int64_t)h * a.e + x] : 0.f;
  float M = -INFINITY, Lt = 0.f, O = 0.f;
  for (int s0 = 0; s0 < n; s0 += U) {
    f32x2 ml[U];
    float o[U];
#pragma unroll
    for (int u = 0; u < U; ++u) {
      const int s = min(s0 + u, n - 1);                    // (past the end: the last split again, weighted 0)
      ml[u] = *(const f32x2*)(a.part_ml + 2 * (at + s));
      o[u] = a.part_o[(at + s) * a.e + x];
    }
    float m = M;
#pragma unroll
    for (int u = 0; u < U; ++u) m = s0 + u < n ? fmaxf(m, ml[u][0]) : m;
    const float sc = __builtin_amdgcn_exp2f(M - m);        // (M = -inf: 0)
    Lt *= sc;
    O *= sc;
#pragma unroll
    for (int u = 0; u < U; ++u) {
      const float w = s0 + u < n ? __builtin_amdgcn_exp2f(ml[u][0] - m) : 0.f;
      Lt = fmaf(w, ml[u][1], Lt);
      O = fmaf(w, o[u], O);
    }
    M = m;
  }
  float r = O / Lt;
  if (a.gate) r *= sigmoid_f(gt);
  a.o[(int64_t)b * a.os + (int64_t)h * a.e + x] = (bf16_t)r;
}

int cu_count() {
  static const int n = [] {
    int dev = 0, cus = 0;
    if (hipGetDevice(&dev) != hipSuccess ||
        hipDeviceGetAttribute(&cus, hipDeviceAttributeMultiprocessorCount, dev) != hipSuccess || cus < 8)
      cus = 256;                               // MI355X
    return cus;
  }();
  return n;
}

int heads_per_group(int gq) { return gq >= 8 ? 8 : gq > 2 ? 4 : gq; }

// work-groups for every compute unit, but a round of keys for each
int pick_splits(int batch, int nheads_kv, int gq, int capacity, int window, int keep) {
  const int hpg = heads_per_group(gq), per = batch * nheads_kv * ((gq + hpg - 1) / hpg);
  const int64_t vis = (int64_t)window + keep < capacity ? (int64_t)window + keep : capacity;
  int want = (2 * cu_count() + per - 1) / per;
  const int64_t most = (vis + WD_KEYS - 1) / WD_KEYS;
  if (want > most) want = (int)most;
  if (want > WD_MAX_SPLIT) want = WD_MAX_SPLIT;
  return want < 1 ? 1 : want;
}

template <int GQ>
void launch_wd(const WdArgs& a, int L, dim3 grid, hipStream_t st) {
  if (L <= 8) attn_window_decode_kernel<GQ, 8><<<grid, WD_THREADS, 0, st>>>(a);
  else if (L <= 16) attn_window_decode_kernel<GQ, 16><<<grid, WD_THREADS, 0, st>>>(a);
  else attn_window_decode_kernel<GQ, 32><<<grid, WD_THREADS, 0, st>>>(a);
}

}  // namespace

extern "C" size_t tv_attn_window_decode_workspace_bytes(int batch, int nheads_q, int nheads_kv, int v_dim, int capacity, int window,
                                                        int keep_first) {
  if (batch <= 0 || nheads_kv <= 0 || nheads_q <= 0 || nheads_q % nheads_kv || v_dim <= 0 || capacity <= 0 || window <= 0 || keep_first < 0) return 0;
  const int ns = pick_splits(batch, nheads_kv, nheads_q / nheads_kv, capacity, window, keep_first);
  return ns == 1 ? 0 : (size_t)batch * nheads_q * ns * (v_dim + 2) * sizeof(float);
}

extern "C" int tv_attn_window_decode_fwd(const void* q, void* cache, const void* fresh, const void* gate, void* o, const int* keys,
                                         const int* slot, int batch, int nheads_q, int nheads_kv, int dim, int v_dim, int capacity,
                                         int window, int keep_first, int64_t q_stride, int64_t fresh_stride, int64_t gate_stride,
                                         int64_t o_stride, float scale, void* workspace, size_t workspace_bytes, void* stream) {
  TV_CHECK_ARG(q && cache && o && keys && slot, "attn_window_decode: null pointer");
  TV_CHECK_ARG(batch > 0 && batch < 65536 && nheads_q > 0 && nheads_kv > 0 && nheads_q % nheads_kv == 0 && dim > 0 && v_dim > 0 && capacity > 0 &&
                   window > 0 && keep_first >= 0 && keep_first < (1 << 30), "attn_window_decode: bad sizes");
  if (dim % 8 || v_dim % 8 || dim > 256 || v_dim > 256) TV_UNSUPPORTED("attn_window_decode: dims %d / %d (multiples of 8, at most 256)", dim, v_dim);
  if (q_stride % 8 || fresh_stride % 8 || ((uintptr_t)q & 15) || ((uintptr_t)cache & 15) || ((uintptr_t)fresh & 15))
    TV_UNSUPPORTED("attn_window_decode: q, cache and new rows must be 16-byte aligned");
  const int gq = nheads_q / nheads_kv, hpg = heads_per_group(gq);
  WdArgs a;
  a.q = (const bf16_t*)q; a.fresh = (const bf16_t*)fresh; a.gate = (const bf16_t*)gate; a.cache = (bf16_t*)cache; a.o = (bf16_t*)o;
  a.keys = keys; a.slot = slot;
  a.H = nheads_q; a.G = nheads_kv; a.gq = gq; a.d = dim; a.e = v_dim; a.cap = capacity; a.window = window; a.keep = keep_first;
  a.hblocks = (gq + hpg - 1) / hpg;
  a.nsplit = pick_splits(batch, nheads_kv, gq, capacity, window, keep_first);
  a.qs = q_stride; a.fs = fresh_stride; a.gs = gate_stride; a.os = o_stride;
  a.scale_log2 = scale * 1.4426950408889634f;
  a.part_o = a.part_ml = nullptr;
  if (a.nsplit > 1) {
    const size_t need = tv_attn_window_decode_workspace_bytes(batch, nheads_q, nheads_kv, v_dim, capacity, window, keep_first);
    TV_CHECK_ARG(workspace && workspace_bytes >= need && ((uintptr_t)workspace & 15) == 0,
                 "attn_window_decode: workspace of %zu bytes (16-byte aligned) needed, got %zu", need, workspace_bytes);
    // (max, sum) pairs first: 8-byte aligned whatever v_dim is
    a.part_ml = (float*)workspace;
    a.part_o = a.part_ml + (size_t)2 * batch * nheads_q * a.nsplit;
  }
  hipStream_t st = (hipStream_t)stream;
  const dim3 grid((unsigned)a.nsplit, (unsigned)(nheads_kv * a.hblocks), (unsigned)batch);
  const int L = (dim > v_dim ? dim : v_dim) / 8;
  if (hpg == 1) launch_wd<1>(a, L, grid, st);
  else if (hpg == 2) launch_wd<2>(a, L, grid, st);
  else if (hpg == 4) launch_wd<4>(a, L, grid, st);
  else launch_wd<8>(a, L, grid, st);
  if (a.nsplit > 1) attn_window_merge_kernel<<<dim3((unsigned)nheads_q, (unsigned)batch), WD_THREADS, 0, st>>>(a);
  TV_LAUNCH_CHECK();
}
