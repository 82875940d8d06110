// seq_moe.hip -- routing and glue of the mixture-of-experts feed-forward (the expert products are dihip_linear_segmented):
//   moe_route      per token, f32: the `top` experts of largest choice score and their weights (RouteRule below: scores = logits,
//                  their softmax or their sigmoids; a correction for the choice alone; a choice limited to the best groups)
//   moe_sort       the (token, choice) pairs grouped by expert in a fixed order: segment bounds per expert, the token each
//                  sorted row reads, and where each pair went
//   moe_glu        the experts' activation on [gate | up] rows (clamped sigmoid unit, or silu(gate) * up)
//   moe_combine    out[t] = sum over the token's choices, in order, of weight * the expert's output row -- the token's own input
//                  row for the experts past the real ones (identity experts) -- plus an optional row added for every token
#include "seq_common.h"

namespace dihip {
namespace {

// How a token's experts are chosen and weighted.
//   scoring 0  scores = the logits, weights = softmax over the chosen logits alone
//   scoring 1  scores = softmax over all E logits;  scoring 2  scores = sigmoid of every logit
//              the choice goes by score + correction; weights = the chosen scores (over their sum with renorm) * factor
//   ngroups    the experts form equal groups of neighbours; only experts of the `keep` best groups can be chosen (the others count as
//              minus infinity).  A group counts by its largest score, or (group_top2) by the sum of its two largest choice scores
// Ties: the lower index, in groups and experts.
struct RouteRule {
  const void* corr; int cdt;
  int E, top, ngroups, keep, group_top2, renorm;
  float factor;
};

// what one lane wrote to LDS is read by other lanes of the same wave
__device__ __forceinline__ void wave_lds_sync() {
  __builtin_amdgcn_fence(__ATOMIC_RELEASE, "wavefront");
  __builtin_amdgcn_wave_barrier();
  __builtin_amdgcn_fence(__ATOMIC_ACQUIRE, "wavefront");
}

// One token per wave: lane l holds the experts l, l + 64, .. (NE of them), a choice is a maximum over the wave and the lowest index
// that has it.  vals: E floats of LDS of this wave.  Afterwards lane k < top holds choice k and its weight.
template <int SCORING, int NE>
__device__ __forceinline__ void route_wave(const float* __restrict__ z, const RouteRule& r, float* vals, int& id, float& wt) {
  constexpr float NONE = 16777216.f;     // an index beyond every expert
  const int lane = threadIdx.x & 63;
  float s[NE], c[NE];
  float zmax = -INFINITY;
#pragma unroll
  for (int i = 0; i < NE; ++i) {
    const int e = lane + 64 * i;
    s[i] = e < r.E ? z[e] : -INFINITY;
    zmax = fmaxf(zmax, s[i]);
  }
  if (SCORING == 1) {
    zmax = wave_max(zmax);
    float den = 0.f;
#pragma unroll
    for (int i = 0; i < NE; ++i) {
      s[i] = lane + 64 * i < r.E ? expf(s[i] - zmax) : 0.f;
      den += s[i];
    }
    den = wave_sum(den);
#pragma unroll
    for (int i = 0; i < NE; ++i) s[i] /= den;
  }
  if (SCORING == 2) {
#pragma unroll
    for (int i = 0; i < NE; ++i) s[i] = 1.f / (1.f + expf(-s[i]));
  }
#pragma unroll
  for (int i = 0; i < NE; ++i) {
    const int e = lane + 64 * i;
    c[i] = e < r.E ? s[i] + (r.corr ? ld_any(r.corr, e, r.cdt) : 0.f) : -INFINITY;
  }
  if (r.ngroups > 1 && r.keep < r.ngroups) {
    const int gsz = r.E / r.ngroups;
    wave_lds_sync();      // the token before is no longer read
#pragma unroll
    for (int i = 0; i < NE; ++i)
      if (lane + 64 * i < r.E) vals[lane + 64 * i] = r.group_top2 ? c[i] : s[i];
    wave_lds_sync();
    float gv = -INFINITY;
    if (lane < r.ngroups) {
      float m1 = -INFINITY, m2 = -INFINITY;
      for (int e = lane * gsz; e < (lane + 1) * gsz; ++e) {
        const float v = vals[e];
        m2 = fmaxf(m2, fminf(m1, v));
        m1 = fmaxf(m1, v);
      }
      gv = r.group_top2 && gsz > 1 ? m1 + m2 : m1;
    }
    unsigned long long open = 0ull;
    for (int k = 0; k < r.keep; ++k) {
      const float m = wave_max(gv);
      const float g = wave_min(lane < r.ngroups && gv == m ? (float)lane : NONE);
      open |= 1ull << min((int)g, r.ngroups - 1);
      if (lane == (int)g) gv = -INFINITY;
    }
#pragma unroll
    for (int i = 0; i < NE; ++i) {
      const int e = lane + 64 * i;
      if (e < r.E && !(open >> (e / gsz) & 1ull)) c[i] = -INFINITY;
    }
  }
  id = 0;
  wt = SCORING == 0 ? -INFINITY : 0.f;
  for (int k = 0; k < r.top; ++k) {
    float m = c[0];
#pragma unroll
    for (int i = 1; i < NE; ++i) m = fmaxf(m, c[i]);
    m = wave_max(m);
    float x = NONE;
#pragma unroll
    for (int i = NE - 1; i >= 0; --i)
      if (lane + 64 * i < r.E && c[i] == m) x = (float)(lane + 64 * i);
    const int best = min((int)wave_min(x), r.E - 1);
    float sv = -INFINITY;
#pragma unroll
    for (int i = 0; i < NE; ++i)
      if (lane + 64 * i == best) { sv = s[i]; c[i] = -INFINITY; }
    sv = wave_max(sv);
    if (lane == k) { id = best; wt = sv; }
  }
  if (SCORING == 0) {
    wt = expf(wt - __shfl(wt, 0));      // lanes past the choices: 0
    wt = wt / wave_sum(wt);
  } else {
    if (r.renorm) wt = wt / (wave_sum(wt) + 1e-20f);
    wt *= r.factor;
  }
}

template <int SCORING, int NE>
__global__ __launch_bounds__(256) void moe_route_kernel(const float* __restrict__ logits, long ldl, RouteRule r, int32_t* __restrict__ ids,
                                                        float* __restrict__ wts, int T) {
  extern __shared__ float route_vals[];
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, t = blockIdx.x * 4 + wave;
  if (t >= T) return;
  int id;
  float wt;
  route_wave<SCORING, NE>(logits + (size_t)t * ldl, r, route_vals + (size_t)wave * r.E, id, wt);
  if (lane < r.top) {
    ids[(size_t)t * r.top + lane] = id;
    wts[(size_t)t * r.top + lane] = wt;
  }
}

// Few rows (T <= 64, T * top <= 1024, E <= 256; decoding): the choice, the counts and the places in ONE workgroup -- the same ids,
// weights and row order as the three launches below.
template <int SCORING, int NE>
__global__ __launch_bounds__(1024) void moe_route_small_kernel(const float* __restrict__ logits, long ldl, RouteRule r, int32_t* __restrict__ ids,
                                                               float* __restrict__ wts, int32_t* __restrict__ counts, int32_t* __restrict__ seg,
                                                               int32_t* __restrict__ src_row, int32_t* __restrict__ dst, int T) {
  extern __shared__ float route_vals[];
  __shared__ int ids_s[1024];
  __shared__ int cnt_s[256];
  const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63, E = r.E, top = r.top, R = T * top;
  for (int t = wave; t < T; t += 16) {
    int id;
    float wt;
    route_wave<SCORING, NE>(logits + (size_t)t * ldl, r, route_vals + (size_t)wave * E, id, wt);
    if (lane < top) {
      ids[(size_t)t * top + lane] = ids_s[t * top + lane] = id;
      wts[(size_t)t * top + lane] = wt;
    }
  }
  __syncthreads();
  int c = 0;
  if (tid < E) {
    for (int x = 0; x < R; ++x) c += ids_s[x] == tid;
    cnt_s[tid] = c;
    counts[tid] = c;
  }
  __syncthreads();
  if (tid < E) {
    int pos = 0;
    for (int x = 0; x < tid; ++x) pos += cnt_s[x];
    seg[tid] = pos;
    if (tid == E - 1) seg[E] = pos + c;
    for (int x = 0; x < R; ++x)
      if (ids_s[x] == tid) {
        src_row[pos] = x / top;
        dst[x] = pos;
        ++pos;
      }
  }
}

// block e: how many pairs chose expert e
__global__ __launch_bounds__(256) void moe_count_kernel(const int32_t* __restrict__ ids, int R, int32_t* __restrict__ counts) {
  __shared__ int red[4];
  const int e = blockIdx.x;
  int c = 0;
  for (int r = threadIdx.x; r < R; r += 256) c += ids[r] == e;
  for (int o = 32; o > 0; o >>= 1) c += __shfl_xor(c, o);
  if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = c;
  __syncthreads();
  if (threadIdx.x == 0) counts[e] = red[0] + red[1] + red[2] + red[3];
}

// block e: its pairs in ascending pair order -> sorted rows seg[e] ..; thread i scans the pairs [i * per, (i + 1) * per)
__global__ __launch_bounds__(256) void moe_place_kernel(const int32_t* __restrict__ ids, int R, int top, int E, const int32_t* __restrict__ counts,
                                                        int32_t* __restrict__ seg, int32_t* __restrict__ src_row, int32_t* __restrict__ dst) {
  __shared__ int scan[256];
  const int e = blockIdx.x, tid = threadIdx.x;
  const int per = (R + 255) / 256, lo = min(R, tid * per), hi = min(R, lo + per);
  int c = 0;
  for (int r = lo; r < hi; ++r) c += ids[r] == e;
  scan[tid] = c;
  __syncthreads();
  int base = 0;
  for (int x = 0; x < e; ++x) base += counts[x];
  if (tid == 0) {
    seg[e] = base;
    if (e == E - 1) seg[E] = base + counts[e];
  }
  int before = 0;
  for (int x = 0; x < tid; ++x) before += scan[x];
  int pos = base + before;
  for (int r = lo; r < hi; ++r)
    if (ids[r] == e) {
      src_row[pos] = r / top;
      dst[r] = pos;
      ++pos;
    }
}

__global__ __launch_bounds__(256) void moe_glu_kernel(void* __restrict__ y, int ydt, long ldy, const float* __restrict__ gu, long ldgu, int F,
                                                      float limit, float slope, int unit) {
  const int r = blockIdx.x;
  for (int c = blockIdx.y * 256 + threadIdx.x; c < F; c += 256 * gridDim.y) {
    if (unit == 1) {      // silu(gate) * up
      const float g = gu[(size_t)r * ldgu + c], u = gu[(size_t)r * ldgu + F + c];
      st_any(y, (size_t)r * ldy + c, ydt, g / (1.f + expf(-g)) * u);
      continue;
    }
    const float g = fminf(gu[(size_t)r * ldgu + c], limit);
    const float u = fminf(fmaxf(gu[(size_t)r * ldgu + F + c], -limit), limit);
    st_any(y, (size_t)r * ldy + c, ydt, g * (1.f / (1.f + expf(-slope * g))) * (u + 1.f));
  }
}

__global__ __launch_bounds__(256) void moe_combine_kernel(float* __restrict__ out, long ldo, const float* __restrict__ rows, long ldr,
                                                          const int32_t* __restrict__ dst, const float* __restrict__ wts, int top, int K,
                                                          const int32_t* __restrict__ ids, int n_real, const void* __restrict__ own, int odt,
                                                          long ldown, const float* __restrict__ add, long ldadd) {
  const int t = blockIdx.x;
  for (int c = blockIdx.y * 256 + threadIdx.x; c < K; c += 256 * gridDim.y) {
    float acc = 0.f;
    for (int k = 0; k < top; ++k) {
      const size_t pr = (size_t)t * top + k;
      const float v = ids && ids[pr] >= n_real ? ld_any(own, (size_t)t * ldown + c, odt) : rows[(size_t)dst[pr] * ldr + c];
      acc = __builtin_fmaf(wts[pr], v, acc);
    }
    if (add) acc += add[(size_t)t * ldadd + c];
    out[(size_t)t * ldo + c] = acc;
  }
}

}  // namespace
}  // namespace dihip

using namespace dihip;

extern "C" {

int dihip_seq_moe_route(void* stream, const float* logits, long ldl, int32_t* ids, float* wts, int32_t* counts, int32_t* seg, int32_t* src_row,
                        int32_t* dst, int T, int E, int top, int scoring, const void* correction, int w_dtype, int ngroups, int keep,
                        int group_top2, int renorm, float factor) {
  DIHIP_REQUIRE(ngroups >= 1 && ngroups <= 64 && E % ngroups == 0 && keep >= 1 && keep <= ngroups && (long)keep * (E / ngroups) >= top,
                DIHIP_PARAM_ERROR, "moe_route: at most 64 equal groups, of which the kept ones must hold the choices");
  DIHIP_REQUIRE(scoring >= 0 && scoring <= 2 && (!correction || scoring > 0) && seq_dtype_ok(w_dtype), DIHIP_PARAM_ERROR,
                "moe_route: unknown scoring (a correction goes with scoring 1 and 2)");
  DIHIP_REQUIRE(T >= 0 && E > 0 && top > 0 && top <= E && top <= 32 && E <= 1024 && logits && ids && wts && counts && seg && src_row && dst &&
                    ldl >= E, DIHIP_PARAM_ERROR, "moe_route: bad argument (at most 1024 experts, 32 choices per token)");
  if (T == 0) return DIHIP_SUCCESS;
  hipStream_t s = reinterpret_cast<hipStream_t>(stream);
  const RouteRule r{correction, w_dtype, E, top, ngroups, keep, group_top2, renorm, factor};
  const bool small = T <= 64 && T * top <= 1024 && E <= 256;
  auto go = [&](auto sc, auto ne) {
    constexpr int SC = decltype(sc)::value, NE = decltype(ne)::value;
    if (small) hipLaunchKernelGGL((moe_route_small_kernel<SC, NE>), dim3(1), dim3(1024), (size_t)16 * E * 4, s, logits, ldl, r, ids, wts, counts, seg, src_row, dst, T);
    else hipLaunchKernelGGL((moe_route_kernel<SC, NE>), dim3((T + 3) / 4), dim3(256), (size_t)4 * E * 4, s, logits, ldl, r, ids, wts, T);
  };
  auto by_e = [&](auto sc) {
    if (E <= 64) go(sc, std::integral_constant<int, 1>{});
    else if (E <= 256) go(sc, std::integral_constant<int, 4>{});
    else go(sc, std::integral_constant<int, 16>{});
  };
  if (scoring == 2) by_e(std::integral_constant<int, 2>{});
  else if (scoring == 1) by_e(std::integral_constant<int, 1>{});
  else by_e(std::integral_constant<int, 0>{});
  if (small) return launch_status();
  hipLaunchKernelGGL(moe_count_kernel, dim3(E), dim3(256), 0, s, ids, T * top, counts);
  hipLaunchKernelGGL(moe_place_kernel, dim3(E), dim3(256), 0, s, ids, T * top, top, E, counts, seg, src_row, dst);
  return launch_status();
}

int dihip_seq_moe_glu(void* stream, void* y, int y_dtype, long ldy, const float* gu, long ldgu, int R, int F, float limit, float slope, int unit) {
  DIHIP_REQUIRE((unit == 0 || unit == 1) && R >= 0 && F > 0 && y && gu && ldy >= F && ldgu >= 2 * (long)F && seq_dtype_ok(y_dtype), DIHIP_PARAM_ERROR, "moe_glu: bad argument");
  if (R == 0) return DIHIP_SUCCESS;
  hipLaunchKernelGGL(moe_glu_kernel, dim3(R, R >= 256 ? 1 : (F + 1023) / 1024), dim3(256), 0, reinterpret_cast<hipStream_t>(stream), y, y_dtype, ldy, gu, ldgu, F, limit, slope, unit);
  return launch_status();
}

int dihip_seq_moe_combine(void* stream, float* out, long ldo, const float* rows, long ldr, const int32_t* dst, const float* wts, int T, int top,
                      int K, const int32_t* ids, int n_real, const void* own, int own_dtype, long ldown, const float* add, long ldadd) {
  DIHIP_REQUIRE(T >= 0 && top > 0 && K > 0 && out && rows && dst && wts && ldo >= K && ldr >= K, DIHIP_PARAM_ERROR, "moe_combine: bad argument");
  DIHIP_REQUIRE((!ids || (own && ldown >= K && seq_dtype_ok(own_dtype) && n_real >= 0)) && (!add || ldadd >= K), DIHIP_PARAM_ERROR,
                "moe_combine: identity experts need the tokens' own rows; added rows at least K wide");
  if (T == 0) return DIHIP_SUCCESS;
  hipLaunchKernelGGL(moe_combine_kernel, dim3(T, T >= 256 ? 1 : (K + 1023) / 1024), dim3(256), 0, reinterpret_cast<hipStream_t>(stream), out, ldo, rows, ldr, dst, wts, top, K, ids, n_real, own, own_dtype, ldown, add, ldadd);
  return launch_status();
}

}  // extern "C"
