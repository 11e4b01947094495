// One query token per sequence against a slot cache, with a sliding window and kept first keys (bf16, any head counts, query / key
// and value dims of their own): position p sees keys (p - window, p] and the first `keep` keys of its sequence.
//
// A cache row holds a token's keys and values side by side, [kv heads x dim | kv heads x vdim].  The VISIBLE keys of a sequence
// (kept ones, then the window) are numbered 0 .. n - 1 and split over `nsplit` work-groups per key / value head; a work-group
// serves up to GQ query heads of its key / value head, so a row is read once per GQ heads.  64 keys a round, everything the
// round needs requested at once:
//   scores    S^T[key][head] = K . Q^T, v_mfma_f32_16x16x32_bf16: a wave's 16 keys come from memory in the A operand's layout
//             (lane = key % 16 and a quarter of 32 dims), the heads are the columns
//   softmax   a wave per head, a lane per key, through LDS; one running maximum per head for the whole work-group
//   values    through LDS; a lane owns two columns of every head, a wave 16 keys, fp32 weights times bf16 values on the vector pipe
//             (no cross-lane sums: the four waves meet once at the end)
// (Scores as dot products over lanes and weights applied in place took 1 400 vector instructions a wave and 64 keys, 4 cycles
// each: the kernel was bound by them.)  Scores, weights and sums are fp32, the weights are not rounded.  With one split the
// result is written directly; else a second kernel merges the splits.  The output gate (o *= sigmoid(gate)) is applied where
// the result is written.
//
// `fresh`: the step's own keys and values (a projection output).  The work-group that meets the newest key takes it from there and
// writes it to the cache.  Layers that read another layer's cache leave it out: the row is in the cache already.
#include "ssd_common.hpp"

namespace {
using namespace ssdk;

constexpr int WD_THREADS = 256;
constexpr int WD_KEYS = 64;          // keys of a round
constexpr int WD_MAX_SPLIT = 256;
constexpr int WD_MERGE = 1024;       // threads of a merging work-group
struct WdArgs {
  const bf16_t *q, *fresh, *gate;
  bf16_t *cache, *o;
  float *part_o, *part_ml;           // (B, H, nsplit, e) and (B, H, nsplit, 2)
  const int *keys, *slot;
  int H, G, gq, d, e, cap, window, keep, nsplit, hblocks;
  int64_t qs, fs, gs, os;
  float scale_log2;
};

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

// GQ query heads a work-group (<= 16), KS >= dim / 32 k-steps, EC x 128 >= value columns
template <int GQ, int KS, int EC>
__global__ __launch_bounds__(WD_THREADS) void attn_window_decode_kernel(WdArgs a) {
  constexpr int VP = 16 * EC;                  // 16-byte pieces of a value row
  constexpr int NV = WD_KEYS * VP / WD_THREADS;
  constexpr int OW = 128 * EC;
  union Tile {
    bf16_t v[WD_KEYS][OW];
    float o[4][GQ][OW];
  };
  __shared__ __attribute__((aligned(16))) Tile t;
  __shared__ __attribute__((aligned(16))) float sP[WD_KEYS][GQ];
  __shared__ float sA[GQ], sM[GQ], sL[GQ];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int n = lane & 15, kq = lane >> 4;     // key of the wave's 16 (and head column), quarter of a k-step
  const int split = blockIdx.x, b = blockIdx.z;
  const int hk = blockIdx.y / a.hblocks, hb = blockIdx.y % a.hblocks;
  const int head0 = hk * a.gq + GQ * hb, nh = min(GQ, a.gq - GQ * hb);

  // Q^T fragments: lane (n, kq) holds Q[head0 + n][32 ks + 8 kq .. + 7], zeros past dim (columns past nh are not used)
  bf16x8 qf[KS];
#pragma unroll
  for (int ks = 0; ks < KS; ++ks) {
    const int d0 = 32 * ks + 8 * kq;
    qf[ks] = *(const bf16x8*)(a.q + (int64_t)b * a.qs + (int64_t)(head0 + min(n, nh - 1)) * a.d + (d0 < a.d ? d0 : 0));
  }
  const int slot = a.slot[b], nk = min(a.keys[b], a.cap);
  const Visible vis = visible_of(a, nk);
  const int r0 = split * vis.chunk, r1 = min(vis.n, r0 + vis.chunk);
  if (r0 >= r1) return;                        // (the merge kernel leaves the same splits out)
  const int W = a.G * (a.d + a.e), ko = hk * a.d, vo = a.G * a.d + hk * a.e;
  bf16_t* base = a.cache + (int64_t)slot * a.cap * W;
  const bf16_t* fresh = a.fresh ? a.fresh + (int64_t)b * a.fs : nullptr;
  auto row_of = [&](int j) __attribute__((always_inline)) {
    const int key = j < vis.kept ? j : j + vis.skip;
    return fresh && key == nk - 1 ? fresh : base + (int64_t)key * W;
  };

  float m_run[(GQ + 3) / 4], l_run[(GQ + 3) / 4], acc[GQ][2 * EC];
#pragma unroll
  for (int i = 0; i < (GQ + 3) / 4; ++i) { m_run[i] = -INFINITY; l_run[i] = 0.f; }
#pragma unroll
  for (int h = 0; h < GQ; ++h)
#pragma unroll
    for (int i = 0; i < 2 * EC; ++i) acc[h][i] = 0.f;

  for (int k0 = r0; k0 < r1; k0 += WD_KEYS) {
    // no branch around a load (where two paths join, the value is waited for): keys past the range repeat its last one with weight 0,
    // pieces past a row's end take its first one (the query is 0 there; the output columns do not exist)
    bf16x8 kf[KS], vf[NV];
    const int jk = k0 + 16 * wave + n;
    const bf16_t* kr = row_of(min(jk, r1 - 1)) + ko;
#pragma unroll
    for (int ks = 0; ks < KS; ++ks) kf[ks] = *(const bf16x8*)(kr + (32 * ks + 8 * kq < a.d ? 32 * ks + 8 * kq : 0));
#pragma unroll
    for (int i = 0; i < NV; ++i) {
      const int p = tid + i * WD_THREADS, c = p % VP;
      vf[i] = *(const bf16x8*)(row_of(min(k0 + p / VP, r1 - 1)) + vo + (8 * c < a.e ? 8 * c : 0));
    }
    f32x4 s = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int ks = 0; ks < KS; ++ks) {
      const bf16x8 zero = {};
      s = mfma16(kf[ks], 32 * ks + 8 * kq < a.d ? qf[ks] : zero, s);
    }
    if (n < GQ) {                              // rows 4 kq + i of the wave's keys, column n
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int j = 16 * wave + 4 * kq + i;
        sP[j][n] = k0 + j < r1 ? s[i] * a.scale_log2 : -INFINITY;
      }
    }
#pragma unroll
    for (int i = 0; i < NV; ++i) {
      const int p = tid + i * WD_THREADS;
      *(bf16x8*)&t.v[p / VP][8 * (p % VP)] = vf[i];
    }
    if (fresh && hb == 0 && r1 == vis.n && k0 + WD_KEYS >= r1) {       // the round that holds the newest key
      bf16_t* row = base + (int64_t)(nk - 1) * W;
      if (jk == r1 - 1) {
#pragma unroll
        for (int ks = 0; ks < KS; ++ks)
          if (32 * ks + 8 * kq < a.d) *(bf16x8*)(row + ko + 32 * ks + 8 * kq) = kf[ks];
      }
#pragma unroll
      for (int i = 0; i < NV; ++i) {
        const int p = tid + i * WD_THREADS, c = p % VP;
        if (k0 + p / VP == r1 - 1 && 8 * c < a.e) *(bf16x8*)(row + vo + 8 * c) = vf[i];
      }
    }
    __syncthreads();
#pragma unroll
    for (int i = 0; i < (GQ + 3) / 4; ++i) {
      const int h = wave + 4 * i;
      if (h < GQ) {
        const float x = sP[lane][h], m_new = fmaxf(m_run[i], wave_max_dpp(x));      // (finite: every round holds a key)
        const float p = __builtin_amdgcn_exp2f(x - m_new), alpha = __builtin_amdgcn_exp2f(m_run[i] - m_new);
        l_run[i] = fmaf(l_run[i], alpha, wave_sum_dpp(p));
        m_run[i] = m_new;
        sP[lane][h] = p;
        if (lane == 0) { sA[h] = alpha; sM[h] = m_new; sL[h] = l_run[i]; }
      }
    }
    __syncthreads();
    if (k0 != r0) {
#pragma unroll
      for (int h = 0; h < GQ; ++h)
#pragma unroll
        for (int i = 0; i < 2 * EC; ++i) acc[h][i] *= sA[h];
    }
#pragma unroll
    for (int j = 0; j < 16; ++j) {
      const int key = 16 * wave + j;
#pragma unroll
      for (int ec = 0; ec < EC; ++ec) {
        const unsigned u = *(const unsigned*)&t.v[key][128 * ec + 2 * lane];
        const float v0 = __uint_as_float(u << 16), v1 = __uint_as_float(u & 0xffff0000u);
#pragma unroll
        for (int h = 0; h < GQ; ++h) {
          const float p = sP[key][h];
          acc[h][2 * ec] = fmaf(p, v0, acc[h][2 * ec]);
          acc[h][2 * ec + 1] = fmaf(p, v1, acc[h][2 * ec + 1]);
        }
      }
    }
    __syncthreads();                           // the tile and the weights are written again
  }

  // the four waves' keys
  typedef float f32x2 __attribute__((ext_vector_type(2)));
#pragma unroll
  for (int h = 0; h < GQ; ++h)
#pragma unroll
    for (int ec = 0; ec < EC; ++ec) *(f32x2*)&t.o[wave][h][128 * ec + 2 * lane] = f32x2{acc[h][2 * ec], acc[h][2 * ec + 1]};
  __syncthreads();
  for (int i = tid; i < nh * a.e; i += WD_THREADS) {
    const int h = i / a.e, x = i - h * a.e, head = head0 + h;
    const float O = (t.o[0][h][x] + t.o[1][h][x]) + (t.o[2][h][x] + t.o[3][h][x]);
    if (a.nsplit == 1) {
      float r = O / sL[h];
      if (a.gate) r *= sigmoid_f((float)a.gate[(int64_t)b * a.gs + (int64_t)head * a.e + x]);
      a.o[(int64_t)b * a.os + (int64_t)head * a.e + x] = (bf16_t)r;
    } else {
      const int64_t at = ((int64_t)b * a.H + head) * a.nsplit + split;
      a.part_o[at * a.e + x] = O;
      if (x == 0) { a.part_ml[2 * at] = sM[h]; a.part_ml[2 * at + 1] = sL[h]; }
    }
  }
}

// merge of the splits, output gate: a work-group per (head, sequence); groups of threads as wide as a value row take 8 splits each
// per round
__global__ __launch_bounds__(WD_MERGE) void attn_window_merge_kernel(WdArgs a) {
  constexpr int U = 8;
  typedef float f32x2 __attribute__((ext_vector_type(2)));
  __shared__ float sO[WD_MERGE];
  __shared__ float sM[WD_MERGE / 8], sL[WD_MERGE / 8];
  const int h = blockIdx.x, b = blockIdx.y;
  const int ng = WD_MERGE / a.e, grp = threadIdx.x / a.e, x = threadIdx.x - grp * a.e;      // (e <= 256: two groups at least)
  const float gt = a.gate ? (float)a.gate[(int64_t)b * a.gs + (int64_t)h * a.e + x] : 0.f;
  const int nk = min(a.keys[b], a.cap);
  const int64_t at = ((int64_t)b * a.H + h) * a.nsplit;
  float M = -INFINITY, Lt = 0.f, O = 0.f;
  int n = a.nsplit;
  if (grp < ng) {
    for (int s0 = grp * U; s0 < n; s0 += ng * U) {
      f32x2 ml[U];
      float o[U];
#pragma unroll
      for (int u = 0; u < U; ++u) {
        const int s = min(s0 + u, a.nsplit - 1);           // (requested beside the key count: splits without keys are weighted 0 below)
        ml[u] = *(const f32x2*)(a.part_ml + 2 * (at + s));
        o[u] = a.part_o[(at + s) * a.e + x];
      }
      const Visible vis = visible_of(a, nk);
      n = (vis.n + vis.chunk - 1) / vis.chunk;
      float m = M;
#pragma unroll
      for (int u = 0; u < U; ++u) m = s0 + u < n ? fmaxf(m, ml[u][0]) : m;
      const float sc = M == -INFINITY ? 0.f : __builtin_amdgcn_exp2f(M - m);
      Lt *= sc;
      O *= sc;
#pragma unroll
      for (int u = 0; u < U; ++u) {
        if (s0 + u < n) {
          const float w = __builtin_amdgcn_exp2f(ml[u][0] - m);
          Lt = fmaf(w, ml[u][1], Lt);
          O = fmaf(w, o[u], O);
        }
      }
      M = m;
    }
    sO[threadIdx.x] = O;
    if (x == 0) { sM[grp] = M; sL[grp] = Lt; }
  }
  __syncthreads();
  if (grp == 0) {
    for (int g = 1; g < ng; ++g) {                         // (group 0 has a split with keys, others may have none)
      if (sM[g] == -INFINITY) continue;
      const float m = fmaxf(M, sM[g]), f0 = __builtin_amdgcn_exp2f(M - m), f1 = __builtin_amdgcn_exp2f(sM[g] - m);
      Lt = Lt * f0 + sL[g] * f1;
      O = O * f0 + sO[g * a.e + x] * f1;
      M = m;
    }
    float r = O / Lt;
    if (a.gate) r *= sigmoid_f(gt);
    a.o[(int64_t)b * a.os + (int64_t)h * a.e + x] = (bf16_t)r;
  }
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

// query heads a work-group serves (16 fill the columns of a product; at wide values their sums would not fit the LDS)
int heads_per_group(int gq, int v_dim) { return gq > 8 && v_dim <= 128 ? 16 : gq > 4 ? 8 : gq > 2 ? 4 : gq; }

// a round of keys a work-group; more than one when the chip is full many times over
int pick_splits(int batch, int nheads_kv, int gq, int v_dim, int capacity, int window, int keep) {
  const int hpg = heads_per_group(gq, v_dim);
  const int64_t per = (int64_t)batch * nheads_kv * ((gq + hpg - 1) / hpg);
  const int64_t vis = (int64_t)window + keep < capacity ? (int64_t)window + keep : capacity;
  int64_t rounds = vis * per / (WD_KEYS * 8ll * cu_count());
  const int64_t least = (vis + (int64_t)WD_KEYS * WD_MAX_SPLIT - 1) / ((int64_t)WD_KEYS * WD_MAX_SPLIT);
  if (rounds < least) rounds = least;
  return (int)((vis + WD_KEYS * rounds - 1) / (WD_KEYS * rounds));
}

template <int GQ, int KS>
void launch_wd_e(const WdArgs& a, dim3 grid, hipStream_t st) {
  if (a.e <= 128) attn_window_decode_kernel<GQ, KS, 1><<<grid, WD_THREADS, 0, st>>>(a);
  else if constexpr (GQ <= 8) attn_window_decode_kernel<GQ, KS, 2><<<grid, WD_THREADS, 0, st>>>(a);
}
template <int GQ>
void launch_wd(const WdArgs& a, dim3 grid, hipStream_t st) {
  if (a.d <= 64) launch_wd_e<GQ, 2>(a, grid, st);
  else if (a.d <= 128) launch_wd_e<GQ, 4>(a, grid, st);
  else launch_wd_e<GQ, 8>(a, grid, st);
}

}  // namespace

extern "C" size_t tv_attn_window_decode_workspace_bytes(int batch, int nheads_q, int nheads_kv, int v_dim, int capacity, int window,
                                                        int keep_first) {
  if (batch <= 0 || nheads_kv <= 0 || nheads_q <= 0 || nheads_q % nheads_kv || v_dim <= 0 || capacity <= 0 || window <= 0 || keep_first < 0) return 0;
  const int ns = pick_splits(batch, nheads_kv, nheads_q / nheads_kv, v_dim, capacity, window, keep_first);
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
  const int gq = nheads_q / nheads_kv, hpg = heads_per_group(gq, v_dim);
  WdArgs a;
  a.q = (const bf16_t*)q; a.fresh = (const bf16_t*)fresh; a.gate = (const bf16_t*)gate; a.cache = (bf16_t*)cache; a.o = (bf16_t*)o;
  a.keys = keys; a.slot = slot;
  a.H = nheads_q; a.G = nheads_kv; a.gq = gq; a.d = dim; a.e = v_dim; a.cap = capacity; a.window = window; a.keep = keep_first;
  a.hblocks = (gq + hpg - 1) / hpg;
  a.nsplit = pick_splits(batch, nheads_kv, gq, v_dim, capacity, window, keep_first);
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
  switch (hpg) {
    case 1: launch_wd<1>(a, grid, st); break;
    case 2: launch_wd<2>(a, grid, st); break;
    case 4: launch_wd<4>(a, grid, st); break;
    case 8: launch_wd<8>(a, grid, st); break;
    default: launch_wd<16>(a, grid, st);
  }
  if (a.nsplit > 1) attn_window_merge_kernel<<<dim3((unsigned)nheads_q, (unsigned)batch), WD_MERGE, 0, st>>>(a);
  TV_LAUNCH_CHECK();
}
