// seq_attn_mc.hip -- windowed sink-softmax attention over the paged latent cache on the matrix cores (bf16 cache).
//
// All heads of a sequence share the cached latent rows C [keys, R]: they are keys AND (their first RV elements) values.  A workgroup
// owns 64 or 128 consecutive (row, head) pairs of one portion -- one or two tiles of 16 per wave -- and walks the key tiles of 32
// cached rows its pairs can see.  Per tile: S^T = C . Q^T (A = the tile's rows as they lie in LDS, B = the wave's query fragments,
// held in registers for the whole walk), mask + running softmax on the accumulator lanes (a pair's 32 scores sit in the four 16-lane
// groups of one lane column: permlane swaps reduce them), then O^T += C^T . P^T with P taken straight from those lanes and C^T read
// from the same LDS tile through the transposing LDS read.  The next tile's rows are in flight meanwhile (registers, then the other
// of two LDS tiles: one barrier per tile).
// The loops over the row are fully unrolled for the row's size class (a multiple of 64; no run-time condition inside, which would
// put a wait behind every LDS read): the columns between R and the class hold some finite cached values against zero query elements.
// The key walk can be split over gridDim.z workgroups (few rows: decoding); the partial (maximum, denominator, sums)
// records are merged by a second launch.  The sink joins split 0 as the running softmax's start (maximum = sink,
// denominator = 1).  A pair's own instructions and their order do not depend on how many tiles its wave owns.
#include "seq_common.h"

namespace dihip {
namespace {

struct McArgs {
  float* out; long ldo;
  const float* q; long ldq;
  void* const* spans; int span_stride, span_len;
  const void* sink; int wdt;
  const int32_t* tok_pos; const int32_t* ent_slot; const int32_t* ent_row0; const int32_t* ent_count;
  int H, R, RV, window; float scale;   // RV: the row's first RV elements are the value (multiple of 16)
  float* ws; int rows_total;
};

__device__ __forceinline__ f32x4_t mfma_bf16x(const u32x4_t& a, const u32x4_t& b, const f32x4_t& c) {
  return __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8_t, a), __builtin_bit_cast(bf16x8_t, b), c, 0, 0, 0);
}

// (two waves per SIMD where the state of a wave fits 256 registers: the sums then live in vector registers, not accumulation
// registers, and are scaled in place)
template <int RM, int VM, int QT>
__global__ __launch_bounds__(256, ((RM + VM) * QT <= 900 ? 2 : 1)) void latent_attn_mc_kernel(McArgs a) {
  constexpr int KS = RM / 32, DT = VM / 16, UN = RM / 64, UPR = RM / 8;   // k steps, value tiles, 16-byte units per thread and per tile row
  constexpr int PB = RM * 2 + 16, TILE = 32 * PB;                         // bytes of an LDS row (padded: conflict-free fragments) and tile
  extern __shared__ __attribute__((aligned(16))) unsigned char smem[];
  __shared__ const char* tabs[128];
  const int e = blockIdx.y, split = blockIdx.z, nsplit = gridDim.z;
  const int H = a.H, R = a.R, RV = a.RV;
  const int cnt = a.ent_count[e], row0 = a.ent_row0[e];
  const int nrows = cnt * H, r0 = (gridDim.x - 1 - blockIdx.x) * (64 * QT);      // the longest walks start first
  if (r0 >= nrows) return;
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, ni = lane & 15, kb = lane >> 4;
  const int pos0 = a.tok_pos[row0];
  const int p_lo = pos0 + r0 / H, p_hi = pos0 + min(r0 + 64 * QT - 1, nrows - 1) / H;
  const int k_begin = a.window > 0 ? max(0, p_lo - a.window + 1) : 0;
  const int tile_lo = k_begin >> 5, tile_hi = p_hi >> 5;
  const int per = (tile_hi - tile_lo + nsplit) / nsplit;
  const int my_lo = tile_lo + split * per, my_hi = min(tile_hi, my_lo + per - 1);

  // the span pointers of the walk, staged once: a tile's loads then depend on nothing that is still in flight
  void* const* gtab = a.spans + (size_t)a.ent_slot[e] * a.span_stride;
  const int span_lo = (my_lo * 32) / a.span_len;
  for (int i = tid; i < 128; i += 256) {
    const int sp = span_lo + i;
    tabs[i] = (sp * a.span_len <= p_hi) ? (const char*)gtab[sp] : nullptr;
  }
  int p[QT], h[QT], tq[QT];
  bool row_ok[QT];
  u32x4_t qf[QT][KS];
#pragma unroll
  for (int t = 0; t < QT; ++t) {
    const int myrow = r0 + (wave * QT + t) * 16 + ni;
    row_ok[t] = myrow < nrows;
    const int rr = row_ok[t] ? myrow : nrows - 1;
    tq[t] = rr / H;
    h[t] = rr - tq[t] * H;
    p[t] = pos0 + tq[t];
    const float* qrow = a.q + (size_t)(row0 + tq[t]) * a.ldq + (size_t)h[t] * R + kb * 8;
#pragma unroll
    for (int ks = 0; ks < KS; ++ks) {
      const bool in = ks < KS - 1 || ks * 32 < R;      // (R is a multiple of 32: only the class's last step can lie past it)
      const float* src = qrow + (in ? ks * 32 : 0);
      const f32x4_t lo = *reinterpret_cast<const f32x4_t*>(src), hi = *reinterpret_cast<const f32x4_t*>(src + 4);
      qf[t][ks] = u32x4_t{pack_bf16x2(lo[0], lo[1]), pack_bf16x2(lo[2], lo[3]), pack_bf16x2(hi[0], hi[1]), pack_bf16x2(hi[2], hi[3])};
      if (ks == KS - 1 && !in) qf[t][ks] = u32x4_t{0u, 0u, 0u, 0u};
    }
  }
  const f32x4_t z4 = {0.f, 0.f, 0.f, 0.f};
  float m[QT], l[QT];
  f32x4_t oacc[QT][DT];
#pragma unroll
  for (int t = 0; t < QT; ++t) {
    const bool with_sink = a.sink != nullptr && split == 0;
    m[t] = with_sink ? ld_any(a.sink, h[t], a.wdt) : -1e30f;
    l[t] = with_sink ? 1.f : 0.f;
#pragma unroll
    for (int d = 0; d < DT; ++d) oacc[t][d] = z4;
  }
  // a thread's 16-byte units of a tile: (key inside the tile, column) fixed for the whole walk.  A tile of 32 keys lies inside one
  // span (span_len % 32 == 0): its span and offset are wave-uniform.
  int goff[UN], loff[UN];
#pragma unroll
  for (int j = 0; j < UN; ++j) {
    const int u = tid + 256 * j, kin = u / UPR, c = u - kin * UPR;
    goff[j] = (kin * R + min(c, (R >> 3) - 1) * 8) * 2;
    loff[j] = kin * PB + c * 16;
  }
  __syncthreads();
  u32x4_t pre[UN];
  auto fetch = [&](int tile) {
    const int key0 = tile * 32, sp = key0 / a.span_len;
    const char* sb = (sp - span_lo < 128 ? tabs[sp - span_lo] : (const char*)gtab[sp]) + (size_t)(key0 - sp * a.span_len) * R * 2;
#pragma unroll
    for (int j = 0; j < UN; ++j) pre[j] = gload<u32x4_t>(sb + goff[j]);
  };
  auto stage = [&](unsigned char* buf) {
#pragma unroll
    for (int j = 0; j < UN; ++j) *reinterpret_cast<u32x4_t*>(buf + loff[j]) = pre[j];
  };
  if (my_lo <= my_hi) {
    fetch(my_lo);
    stage(smem);
  }
  __syncthreads();
  for (int tile = my_lo; tile <= my_hi; ++tile) {
    const unsigned char* buf = smem + ((tile - my_lo) & 1) * TILE;
    const bool more = tile < my_hi;
    fetch(more ? tile + 1 : tile);
    f32x4_t sacc[QT][2];
#pragma unroll
    for (int t = 0; t < QT; ++t) sacc[t][0] = sacc[t][1] = z4;
    const unsigned char* kr = buf + ni * PB + kb * 16;
#pragma unroll
    for (int ks = 0; ks < KS; ++ks)
#pragma unroll
      for (int nt = 0; nt < 2; ++nt) {
        const u32x4_t kf = *reinterpret_cast<const u32x4_t*>(kr + nt * 16 * PB + ks * 64);
#pragma unroll
        for (int t = 0; t < QT; ++t) sacc[t][nt] = mfma_bf16x(kf, qf[t][ks], sacc[t][nt]);
      }
    u32x4_t pf[QT];
#pragma unroll
    for (int t = 0; t < QT; ++t) {
      float sv[2][4], mx = -INFINITY;
#pragma unroll
      for (int nt = 0; nt < 2; ++nt)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const int key = tile * 32 + nt * 16 + kb * 4 + r;
          const bool vis = key <= p[t] && (a.window <= 0 || key > p[t] - a.window);
          sv[nt][r] = vis ? sacc[t][nt][r] * a.scale : -INFINITY;
          mx = fmaxf(mx, sv[nt][r]);
        }
      mx = rows_max(mx);
      const float mn = fmaxf(m[t], mx);
      const float corr = __expf(m[t] - mn);
      m[t] = mn;
      float psum = 0.f, ev[2][4];
#pragma unroll
      for (int nt = 0; nt < 2; ++nt)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          ev[nt][r] = __expf(sv[nt][r] - mn);
          psum += ev[nt][r];
        }
      l[t] = l[t] * corr + rows_sum(psum);
      pf[t] = u32x4_t{pack_bf16x2(ev[0][0], ev[0][1]), pack_bf16x2(ev[0][2], ev[0][3]), pack_bf16x2(ev[1][0], ev[1][1]),
                      pack_bf16x2(ev[1][2], ev[1][3])};
      if (__builtin_amdgcn_ballot_w64(corr != 1.f) != 0ull) {
#pragma unroll
        for (int d = 0; d < DT; ++d)
#pragma unroll
          for (int r = 0; r < 4; ++r) oacc[t][d][r] *= corr;
      }
    }
    const unsigned char* tr0 = buf + (kb * 4 + (ni >> 2)) * PB + (ni & 3) * 8;
#pragma unroll
    for (int d = 0; d < DT; ++d) {
      const u32x2_t lo2 = lds_read_tr16(tr0 + d * 32);
      const u32x2_t hi2 = lds_read_tr16(tr0 + d * 32 + 16 * PB);
      const u32x4_t vf = {lo2[0], lo2[1], hi2[0], hi2[1]};
#pragma unroll
      for (int t = 0; t < QT; ++t) oacc[t][d] = mfma_bf16x(vf, pf[t], oacc[t][d]);
    }
    if (more) stage(smem + ((tile + 1 - my_lo) & 1) * TILE);      // (its readers passed the barrier before this tile)
    __syncthreads();
  }
  asm volatile("s_nop 15\n\ts_nop 7" ::: "memory");
#pragma unroll
  for (int t = 0; t < QT; ++t) {
    if (!row_ok[t]) continue;
    if (nsplit == 1) {
      const float inv = 1.f / l[t];
      float* o = a.out + (size_t)(row0 + tq[t]) * a.ldo + (size_t)h[t] * RV + kb * 4;
#pragma unroll
      for (int d = 0; d < DT; ++d)
        if (d * 16 < RV)
          *reinterpret_cast<f32x4_t*>(o + d * 16) = f32x4_t{oacc[t][d][0] * inv, oacc[t][d][1] * inv, oacc[t][d][2] * inv, oacc[t][d][3] * inv};
    } else {
      float* o = a.ws + ((size_t)split * a.rows_total + (size_t)(row0 + tq[t]) * H + h[t]) * (RV + 4);
#pragma unroll
      for (int d = 0; d < DT; ++d)
        if (d * 16 < RV) *reinterpret_cast<f32x4_t*>(o + d * 16 + kb * 4) = oacc[t][d];
      if (kb == 0) { o[RV] = m[t]; o[RV + 1] = l[t]; }
    }
  }
}

// Wide rows (RM > 320): 512 threads own 64 pairs and walk tiles of 64 keys.  The scores are split by pairs and keys -- wave w scores
// pairs (w / 2) * 16 .. + 16 against keys (w % 2) * 32 .. + 32 -- and the value product by columns: every wave holds the sums of ALL 64
// pairs for its value columns (tiles w, w + 8, ..), so that a value fragment read from LDS serves four products.  Maxima and weights
// go through LDS (two barriers per tile).  The state of a wave (queries, sums, the next tile's rows) fits 256 registers: two waves per
// SIMD.  The rows of a tile lie unpadded in LDS, their 16-byte units permuted inside blocks of 8 or 16 (wide_swizzle): the fragment reads
// and the transposing reads are free of bank conflicts.  A maximum moves only when it grows by more than GROW: the weights stay below exp(GROW) with the same relative rounding,
// and the sums are rarely scaled.
template <int RM>
__device__ __forceinline__ int wide_swizzle(int row) {      // unit c of the row lies at unit c ^ wide_swizzle(row)
  const int q = (row >> 1) & 7, s = q < 4 ? 2 * q : (2 * q - 3) & 7;
  return RM % 128 == 0 ? (row & 1) << 3 | s : s;            // (a row of an odd number of 8-unit blocks moves every other row by half the banks)
}

template <int RM, int VM>
__global__ __launch_bounds__(512) void latent_attn_wide_kernel(McArgs a) {
  constexpr int KS = RM / 32, DT = VM / 16, DW = (DT + 7) / 8, UN = RM / 64;
  constexpr int PB = RM * 2, TILE = 64 * PB;
  constexpr float GROW = 8.f;
  extern __shared__ __attribute__((aligned(16))) unsigned char smem[];      // two tiles
  __shared__ __attribute__((aligned(16))) unsigned char wts[2 * 64 * 64];    // weights (bf16): [key half][pair][16-lane group][8 keys]
  __shared__ float stat[2][64];
  __shared__ const char* tabs[64];
  const int e = blockIdx.y, split = blockIdx.z, nsplit = gridDim.z;
  const int H = a.H, R = a.R, RV = a.RV;
  const int cnt = a.ent_count[e], row0 = a.ent_row0[e];
  const int nrows = cnt * H, r0 = (gridDim.x - 1 - blockIdx.x) * 64;      // the longest walks start first
  if (r0 >= nrows) return;
  const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6), ni = lane & 15, kb = lane >> 4;
  const int qg = wave >> 1, kh = wave & 1;
  const int pos0 = a.tok_pos[row0];
  const int p_lo = pos0 + r0 / H, p_hi = pos0 + min(r0 + 63, nrows - 1) / H;
  const int k_begin = a.window > 0 ? max(0, p_lo - a.window + 1) : 0;
  const int tile_lo = k_begin >> 6, tile_hi = p_hi >> 6;
  const int per = (tile_hi - tile_lo + nsplit) / nsplit;
  const int my_lo = tile_lo + split * per, my_hi = min(tile_hi, my_lo + per - 1);

  void* const* gtab = a.spans + (size_t)a.ent_slot[e] * a.span_stride;
  const int span_lo = (my_lo * 64) / a.span_len;
  if (tid < 64) {
    const int sp = span_lo + tid;
    tabs[tid] = (sp * a.span_len <= p_hi) ? (const char*)gtab[sp] : nullptr;
  }
  const int myrow = min(r0 + qg * 16 + ni, nrows - 1), tq = myrow / H, hq = myrow - tq * H, p = pos0 + tq;      // the pair this lane scores
  u32x4_t qf[KS];
  {
    const float* qrow = a.q + (size_t)(row0 + tq) * a.ldq + (size_t)hq * R + kb * 8;
#pragma unroll
    for (int ks = 0; ks < KS; ++ks) {
      const bool in = ks < KS - 1 || ks * 32 < R;
      const float* src = qrow + (in ? ks * 32 : 0);
      const f32x4_t lo = *reinterpret_cast<const f32x4_t*>(src), hi = *reinterpret_cast<const f32x4_t*>(src + 4);
      qf[ks] = u32x4_t{pack_bf16x2(lo[0], lo[1]), pack_bf16x2(lo[2], lo[3]), pack_bf16x2(hi[0], hi[1]), pack_bf16x2(hi[2], hi[3])};
      if (ks == KS - 1 && !in) qf[ks] = u32x4_t{0u, 0u, 0u, 0u};
    }
  }
  const f32x4_t z4 = {0.f, 0.f, 0.f, 0.f};
  const bool with_sink = a.sink != nullptr && split == 0;
  float mq = with_sink ? ld_any(a.sink, hq, a.wdt) : -1e30f;      // the scored pair's maximum; l: its denominator over this wave's keys
  float l = with_sink && kh == 0 ? 1.f : 0.f;
  float m[4];                                                      // the maxima of all pairs (lane column ni of four tiles)
  f32x4_t oacc[4][DW];
#pragma unroll
  for (int t = 0; t < 4; ++t) {
    const int rr = min(r0 + t * 16 + ni, nrows - 1);
    m[t] = with_sink ? ld_any(a.sink, rr % H, a.wdt) : -1e30f;
#pragma unroll
    for (int d = 0; d < DW; ++d) oacc[t][d] = z4;
  }
  // eight threads stage a row of the tile, units (tid % 8) + 8 j: one offset into the page and two into LDS (even and odd j)
  const int srow = tid >> 3, scol = tid & 7, ssw = wide_swizzle<RM>(srow);
  const unsigned goff = (unsigned)(srow * R * 2 + scol * 16);
  const unsigned glast = (unsigned)(srow * R * 2 + min(scol + 8 * (UN - 1), (R >> 3) - 1) * 16);      // (R may end inside the class's last block)
  const int loff0 = srow * PB + (scol ^ ssw) * 16, loff1 = srow * PB + ((scol + 8) ^ ssw) * 16 - 128;
  // the lane's fragment reads: four k steps span 16 units, so four offsets cover every step; its transposing reads: tiles 8 apart, one
  const int sw = wide_swizzle<RM>(ni), vrow = kb * 4 + (ni >> 2), vsw = wide_swizzle<RM>(vrow);
  int koff[4];
#pragma unroll
  for (int i = 0; i < 4; ++i) koff[i] = (kh * 32 + ni) * PB + ((i * 4 + kb) ^ sw) * 16;
  const int voff = vrow * PB + ((wave * 2 + ((ni & 3) >> 1)) ^ vsw) * 16 + (ni & 1) * 8;
  __syncthreads();
  u32x4_t pre[UN];
  auto fetch = [&](int tile) {      // a tile of 64 keys lies inside one span (span_len % 64 == 0)
    const int key0 = tile * 64, sp = key0 / a.span_len;
    const uintptr_t at = (uintptr_t)(sp - span_lo < 64 ? tabs[sp - span_lo] : (const char*)gtab[sp]);
    const uintptr_t ua = (uintptr_t)__builtin_amdgcn_readfirstlane((unsigned)(at >> 32)) << 32 | (unsigned)__builtin_amdgcn_readfirstlane((unsigned)at);
    const char* sb = (const char*)ua + (size_t)(key0 - sp * a.span_len) * R * 2;      // wave-uniform
#pragma unroll
    for (int j = 0; j < UN; ++j) pre[j] = gload<u32x4_t>(sb + (j < UN - 1 ? goff + j * 128u : glast));
  };
  auto stage = [&](unsigned char* buf) {
#pragma unroll
    for (int j = 0; j < UN; ++j) *reinterpret_cast<u32x4_t*>(buf + ((j & 1) ? loff1 : loff0) + j * 128) = pre[j];
  };
  if (my_lo <= my_hi) {
    fetch(my_lo);
    stage(smem);
  }
  __syncthreads();
  for (int tile = my_lo; tile <= my_hi; ++tile) {
    const unsigned char* buf = smem + ((tile - my_lo) & 1) * TILE;
    fetch(min(tile + 1, my_hi));
    f32x4_t sacc[2] = {z4, z4};
    // two k steps at a time, the next two steps' fragments in flight (left alone, the scheduler puts a wait behind every read)
    u32x4_t kf[2][4];
    auto kload = [&](int b) {
#pragma unroll
      for (int i = 0; i < 4; ++i)
        kf[b & 1][i] = *reinterpret_cast<const u32x4_t*>(buf + koff[(2 * b + (i >> 1)) & 3] + (i & 1) * 16 * PB + ((2 * b + (i >> 1)) >> 2) * 256);
    };
    kload(0);
#pragma unroll
    for (int b = 0; b < KS / 2; ++b) {
      if (b + 1 < KS / 2) kload(b + 1);
      __builtin_amdgcn_sched_barrier(0);
#pragma unroll
      for (int i = 0; i < 4; ++i) sacc[i & 1] = mfma_bf16x(kf[b & 1][i], qf[2 * b + (i >> 1)], sacc[i & 1]);
      __builtin_amdgcn_sched_barrier(0);
    }
    float sv[2][4], mx = -INFINITY;
    if (tile * 64 + 63 > p_lo || (a.window > 0 && tile * 64 <= p_hi - a.window)) {      // some pair does not see the whole tile
#pragma unroll
      for (int nt = 0; nt < 2; ++nt)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const int key = tile * 64 + kh * 32 + nt * 16 + kb * 4 + r;
          const bool vis = key <= p && (a.window <= 0 || key > p - a.window);
          sv[nt][r] = vis ? sacc[nt][r] * a.scale : -INFINITY;
          mx = fmaxf(mx, sv[nt][r]);
        }
    } else {
#pragma unroll
      for (int nt = 0; nt < 2; ++nt)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          sv[nt][r] = sacc[nt][r] * a.scale;
          mx = fmaxf(mx, sv[nt][r]);
        }
    }
    mx = rows_max(mx);
    if (kb == 0) stat[kh][qg * 16 + ni] = mx;
    __syncthreads();
    float corr[4];
    bool grown = false;
#pragma unroll
    for (int t = 0; t < 4; ++t) {
      const float x = fmaxf(stat[0][t * 16 + ni], stat[1][t * 16 + ni]);
      const float mn = x > m[t] + GROW ? x : m[t];
      corr[t] = __expf(m[t] - mn);
      grown |= mn != m[t];
      m[t] = mn;
    }
    {
      const float x = fmaxf(stat[0][qg * 16 + ni], stat[1][qg * 16 + ni]);
      const float mn = x > mq + GROW ? x : mq;
      l *= __expf(mq - mn);
      mq = mn;
      float psum = 0.f, ev[2][4];
#pragma unroll
      for (int nt = 0; nt < 2; ++nt)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          ev[nt][r] = __expf(sv[nt][r] - mn);
          psum += ev[nt][r];
        }
      l += rows_sum(psum);
      *reinterpret_cast<u32x4_t*>(wts + ((kh * 64 + qg * 16 + ni) * 4 + kb) * 16) =
          u32x4_t{pack_bf16x2(ev[0][0], ev[0][1]), pack_bf16x2(ev[0][2], ev[0][3]), pack_bf16x2(ev[1][0], ev[1][1]), pack_bf16x2(ev[1][2], ev[1][3])};
    }
    if (__builtin_amdgcn_ballot_w64(grown) != 0ull) {
#pragma unroll
      for (int t = 0; t < 4; ++t)
#pragma unroll
        for (int d = 0; d < DW; ++d)
#pragma unroll
          for (int r = 0; r < 4; ++r) oacc[t][d][r] *= corr[t];
    }
    if (tile < my_hi) stage(smem + ((tile + 1 - my_lo) & 1) * TILE);      // (its readers passed the barrier above)
    __syncthreads();
#pragma unroll
    for (int half = 0; half < 2; ++half) {
      u32x4_t pf[4];
#pragma unroll
      for (int t = 0; t < 4; ++t) pf[t] = *reinterpret_cast<const u32x4_t*>(wts + ((half * 64 + t * 16 + ni) * 4 + kb) * 16);
#pragma unroll
      for (int d = 0; d < DW; ++d) {
        const unsigned char* tr0 = buf + (8 * d + 7 < DT || wave + 8 * d < DT ? voff + d * 256 : voff) + half * 32 * PB;      // (past the value: any tile, not stored)
        const u32x2_t lo2 = lds_read_tr16(tr0), hi2 = lds_read_tr16(tr0 + 16 * PB);
        const u32x4_t vf = {lo2[0], lo2[1], hi2[0], hi2[1]};
#pragma unroll
        for (int t = 0; t < 4; ++t) oacc[t][d] = mfma_bf16x(vf, pf[t], oacc[t][d]);
      }
    }
  }
  __syncthreads();      // the last maxima are no longer read
  if (kb == 0) stat[kh][qg * 16 + ni] = l;
  __syncthreads();
#pragma unroll
  for (int t = 0; t < 4; ++t) {
    const int rr = r0 + t * 16 + ni;
    if (rr >= nrows) continue;
    const int row = row0 + rr / H, h = rr % H;
    const float den = stat[0][t * 16 + ni] + stat[1][t * 16 + ni];
    float* o = nsplit == 1 ? a.out + (size_t)row * a.ldo + (size_t)h * RV : a.ws + ((size_t)split * a.rows_total + (size_t)row * H + h) * (RV + 4);
    const float inv = nsplit == 1 ? 1.f / den : 1.f;
#pragma unroll
    for (int d = 0; d < DW; ++d) {
      const int col = (wave + 8 * d) * 16;
      if (col < RV)
        *reinterpret_cast<f32x4_t*>(o + col + kb * 4) = f32x4_t{oacc[t][d][0] * inv, oacc[t][d][1] * inv, oacc[t][d][2] * inv, oacc[t][d][3] * inv};
    }
    if (nsplit > 1 && wave == 0 && kb == 0) { o[RV] = m[t]; o[RV + 1] = den; }
  }
}

__global__ __launch_bounds__(256) void latent_attn_merge_kernel(float* __restrict__ out, long ldo, const float* __restrict__ ws, int nsplit,
                                                                int rows_total, int H, int RV) {
  __shared__ float wgt[1024];
  __shared__ float red[4];
  const int g = blockIdx.x, t = g / H, h = g - t * H;
  const size_t rec = (size_t)RV + 4, stride = (size_t)rows_total * rec;
  const float* base = ws + (size_t)g * rec;
  float mloc[4], lloc[4], mx = -INFINITY;
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const int s = threadIdx.x + i * 256;
    mloc[i] = s < nsplit ? base[s * stride + RV] : -INFINITY;
    lloc[i] = s < nsplit ? base[s * stride + RV + 1] : 0.f;
    mx = fmaxf(mx, mloc[i]);
  }
  mx = wave_max(mx);
  if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = mx;
  __syncthreads();
  mx = fmaxf(fmaxf(red[0], red[1]), fmaxf(red[2], red[3]));
  float den = 0.f;
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const int s = threadIdx.x + i * 256;
    const float w = s < nsplit ? expf(mloc[i] - mx) : 0.f;
    if (s < nsplit) wgt[s] = w;
    den = __builtin_fmaf(w, lloc[i], den);
  }
  den = block256_sum(den, red);      // (its barriers publish wgt)
  const float inv = 1.f / den;
  for (int r = threadIdx.x; r < RV; r += 256) {
    float acc = 0.f;
#pragma unroll 8
    for (int s = 0; s < nsplit; ++s) acc = __builtin_fmaf(wgt[s], base[s * stride + r], acc);
    out[(size_t)t * ldo + (size_t)h * RV + r] = acc * inv;
  }
}

}  // namespace
}  // namespace dihip

using namespace dihip;

extern "C" {

int dihip_latent_window_attn_mc_supported(int R, int span_len, int cache_dtype) {
  return cache_dtype == DIHIP_BF16 && R % 32 == 0 && R >= 32 && R <= 640 && span_len % 32 == 0;
}

size_t dihip_latent_window_attn_mc_workspace_bytes(int T, int H, int RV, int nsplit) {
  return nsplit > 1 ? (size_t)nsplit * T * H * (RV + 4) * sizeof(float) : 0;
}

int dihip_latent_window_attn_mc(void* stream, float* out, long ldo, const float* q, long ldq, void* const* spans, int span_stride,
                                int span_len, const void* sink, int w_dtype, const int32_t* tok_pos, const int32_t* ent_slot,
                                const int32_t* ent_row0, const int32_t* ent_count, int E, int max_count, int T, int H, int R, int RV, int window,
                                float scale, int nsplit, void* ws, size_t ws_bytes) {
  DIHIP_REQUIRE(dihip_latent_window_attn_mc_supported(R, span_len, DIHIP_BF16), DIHIP_PARAM_ERROR,
                "latent_window_attn_mc: R %d (a multiple of 32 up to 640) / span_len %d (a multiple of 32) not served", R, span_len);
  DIHIP_REQUIRE(RV > 0 && RV <= R && RV <= 512 && RV % 16 == 0, DIHIP_PARAM_ERROR,
                "latent_window_attn_mc: a value of %d elements (a multiple of 16 up to 512 inside the row) not served", RV);
  DIHIP_REQUIRE(E >= 0 && T >= 0 && H > 0 && max_count >= 0 && out && q && spans && tok_pos && ent_slot && ent_row0 && ent_count &&
                    span_stride > 0 && ldo >= (long)H * RV && ldq >= (long)H * R && ldo % 4 == 0 && ldq % 4 == 0 && seq_dtype_ok(w_dtype),
                DIHIP_PARAM_ERROR, "latent_window_attn_mc: bad argument");
  DIHIP_REQUIRE((reinterpret_cast<uintptr_t>(out) & 15u) == 0 && (reinterpret_cast<uintptr_t>(q) & 15u) == 0, DIHIP_PARAM_ERROR,
                "latent_window_attn_mc: q / out must be 16-byte aligned");
  DIHIP_REQUIRE(nsplit >= 1 && nsplit <= 1024 && E <= 65535, DIHIP_PARAM_ERROR, "latent_window_attn_mc: bad split / portion count");
  DIHIP_REQUIRE(ws_bytes >= dihip_latent_window_attn_mc_workspace_bytes(T, H, RV, nsplit) && (nsplit == 1 || ws), DIHIP_PARAM_ERROR,
                "latent_window_attn_mc: workspace too small");
  if (E == 0 || max_count == 0) return DIHIP_SUCCESS;
  hipStream_t s = reinterpret_cast<hipStream_t>(stream);
  McArgs a{out, ldo, q, ldq, spans, span_stride, span_len, sink, w_dtype, tok_pos, ent_slot, ent_row0, ent_count, H, R, RV, window, scale,
           (float*)ws, T * H};
  // two 16-pair tiles per wave halve the LDS traffic per pair: when the pairs fill the chip anyway
  const long pairs = (long)max_count * H;
  const bool two = (pairs + 127) / 128 * E * nsplit >= 256;
  int status = DIHIP_SUCCESS;
  auto go = [&](auto rm, auto vm) {
    constexpr int RM = decltype(rm)::value, VM = decltype(vm)::value;
    const size_t lds = 2 * 32 * (size_t)(RM * 2 + 16);
    auto launch = [&](auto kern, int threads, int per_block, size_t bytes) {
      if (bytes > 64 * 1024 && hipFuncSetAttribute(reinterpret_cast<const void*>(kern), hipFuncAttributeMaxDynamicSharedMemorySize, (int)bytes) != hipSuccess) {
        status = DIHIP_RUNTIME_ERROR;
        return;
      }
      hipLaunchKernelGGL(kern, dim3((unsigned)((pairs + per_block - 1) / per_block), E, nsplit), dim3(threads), bytes, s, a);
    };
    if constexpr (RM > 320 && RM <= 576) {
      if (span_len % 64 == 0) return launch(latent_attn_wide_kernel<RM, VM>, 512, 64, 2 * 64 * (size_t)RM * 2);
    }
    if constexpr (RM <= 320) {      // (a wider row's queries and sums of two tiles do not fit the registers)
      if (two) return launch(latent_attn_mc_kernel<RM, VM, 2>, 256, 128, lds);
    }
    launch(latent_attn_mc_kernel<RM, VM, 1>, 256, 64, lds);
  };
  auto by_v = [&](auto rm) {      // the value is the whole row, or lies within the class below (a rotated part behind it)
    constexpr int RM = decltype(rm)::value, VLOW = RM > 64 ? (RM - 64 > 512 ? 512 : RM - 64) : 64;
    if (RM > 512 || RV <= VLOW) go(rm, std::integral_constant<int, VLOW>{});
    else go(rm, std::integral_constant<int, (RM > 512 ? 512 : RM)>{});
  };
  switch ((R + 63) / 64) {
    case 1: by_v(std::integral_constant<int, 64>{}); break;
    case 2: by_v(std::integral_constant<int, 128>{}); break;
    case 3: by_v(std::integral_constant<int, 192>{}); break;
    case 4: by_v(std::integral_constant<int, 256>{}); break;
    case 5: by_v(std::integral_constant<int, 320>{}); break;
    case 6: by_v(std::integral_constant<int, 384>{}); break;
    case 7: by_v(std::integral_constant<int, 448>{}); break;
    case 8: by_v(std::integral_constant<int, 512>{}); break;
    case 9: by_v(std::integral_constant<int, 576>{}); break;
    default: by_v(std::integral_constant<int, 640>{}); break;
  }
  DIHIP_REQUIRE(status == DIHIP_SUCCESS, DIHIP_RUNTIME_ERROR, "latent_window_attn_mc: the device refuses the workgroup's LDS size");
  if (nsplit > 1) hipLaunchKernelGGL(latent_attn_merge_kernel, dim3(T * H), dim3(256), 0, s, out, ldo, (const float*)ws, nsplit, T * H, H, RV);
  return launch_status();
}

}  // extern "C"
