// seq_decay.hip -- linear attention with ONE decay per head (the same for all key channels) and a matrix state per head, everything in f32:
//   S <- a S + w k v^T,   o = S^T q
// in two uses:
//   retention        a is a constant of the head, w = 1;  queries and keys carry rotary positions
//   matrix memory    (xLSTM) a and w come from a log input gate i and a log forget gate f, both capped, through a running maximum m that
//                    keeps the exponentials in range: m' = max(f + m, i), a = exp(f + m - m'), w = exp(i - m'); a second state
//                    n <- a n + w k gives the output's divisor max(|n . q|, exp(-m')) + 1e-6
// S [H, D, DV], n [H, D] and m live per state slot and are carried from portion to portion.
// Because the decay is one number per row, a chunk of rows collapses into matrix products.  With L_t the sum of log a over the chunk's
// rows up to t:
//   o_t = exp(L_t) S_in^T q_t + sum_{s <= t} exp(L_t - L_s) w_s (k_s . q_t) v_s,     S_out = exp(L) S_in + sum_s exp(L - L_s) w_s k_s v_s^T
// Long portions are cut into chunks of 64 rows that run side by side on the f32 matrix instructions (true f32 products and sums):
// (1) every chunk's own contribution to the state, (2) the states the chunks start from, carried over the chunks, (3) the outputs.
// Differences of L are taken in f64: the sums grow with the chunk while the differences that matter are small.
// Few rows run one after the other from a state in registers (decay_rows_kernel), rotation and gates computed on the way.
#include "seq_common.h"

namespace dihip {
namespace {

constexpr int CHUNK = 64;           // rows per chunk
constexpr int RB = 8;               // rows per batch of the row-by-row kernel

struct DecayArgs {
  float* out; long ldo;                                    // [T][H * DV]
  const float* q; long ldq; const float* k; long ldk;      // rows [H * D]
  const float* v; long ldv;                                // rows [H * DV]
  float q_scale, k_scale;
  const double* log_decay;                                 // [H] constant decays (NULL: gates)
  const float* gi; const float* gf; long ldg; float cap;   // rows [H] of raw gates (row kernel and gates kernel)
  float* la; float* gain; float* floor_;                   // [T][H]: log a, w, exp(-m) (gates kernel -> chunk kernels)
  float* den;                                              // [T][H]: 1 / divisor (NULL: none)
  const float* freq; int rot_dims, pairs; const int32_t* tok_pos;    // rotation inside the row kernel (rot_dims 0: none)
  float* S; float* N; float* M;                            // state; M: one copy of m per 64-column block [slots][H][mcopies]
  int mcopies;
  const int32_t* ent_slot; const int32_t* ent_row0; const int32_t* ent_count;
  int H, D, DV;
  float* ws; int max_chunks;                               // [E][max_chunks][H] records: D * DV (state), D (n), exp(L), padding
};
__host__ __device__ inline size_t chunk_rec(int D, int DV) { return ((size_t)D * DV + D + 1 + 3) & ~(size_t)3; }

__device__ __forceinline__ float log_sigmoid(float z) { return -(log1pf(expf(-fabsf(z))) + fmaxf(-z, 0.f)); }
__device__ __forceinline__ void log_gates(float zi, float zf, float cap, float& i, float& f) {
  i = cap * tanhf(zi / cap);
  f = log_sigmoid(cap * tanhf(zf / cap));
}

// ------------------------------------------------------------------------------------------------ rotation in place
// heads of D elements at x[t][off0 ..] (n0 of them) and x[t][off1 ..] (n1); rot_dims leading dimensions of each
__global__ __launch_bounds__(256) void rope_rows_kernel(float* __restrict__ x, long ld, int off0, int n0, int off1, int n1, int D, int rot_dims,
                                                        int pairs, const float* __restrict__ freq, const int32_t* __restrict__ tok_pos) {
  __shared__ float cs[256], sn[256];
  const int t = blockIdx.x, half = rot_dims >> 1;
  for (int i = threadIdx.x; i < half; i += 256) rope_sincos((uint32_t)tok_pos[t], freq[i], &sn[i], &cs[i]);
  __syncthreads();
  float* row = x + (size_t)t * ld;
  for (int c = blockIdx.y * 256 + threadIdx.x; c < (n0 + n1) * half; c += 256 * gridDim.y) {
    const int h = c / half, i = c - h * half;
    float* p = row + (h < n0 ? off0 + h * D : off1 + (h - n0) * D);
    const int iu = pairs ? 2 * i : i, iv = pairs ? 2 * i + 1 : half + i;
    const float u = p[iu], w = p[iv];
    p[iu] = u * cs[i] - w * sn[i];
    p[iv] = w * cs[i] + u * sn[i];
  }
}

// ------------------------------------------------------------------------------------------------ row by row
// A workgroup of 4 waves owns 64 columns of one head: wave sl keeps rows sl * DPT .. + DPT of the state for its 64 columns.  Queries and
// keys of RB rows at a time are staged in LDS (rotated, scaled); the workgroup of the first columns also keeps n and writes the divisor.
template <int DPT>
__global__ __launch_bounds__(256) void decay_rows_kernel(DecayArgs a) {
  constexpr int DP = 4 * DPT, NPT = (DP + 255) / 256;
  __shared__ __attribute__((aligned(16))) float qs[RB][DP];
  __shared__ __attribute__((aligned(16))) float ks[RB][DP];
  __shared__ float part[RB][4][64];
  __shared__ float gi_s[RB], gf_s[RB], nred[RB][4];
  extern __shared__ float rot_s[];                          // [RB][rot_dims / 2] cosines, then sines
  const int tid = threadIdx.x, lane = tid & 63, sl = tid >> 6;
  const int D = a.D, DV = a.DV, H = a.H, half = a.rot_dims >> 1;
  const int cbs = (DV + 63) / 64, h = blockIdx.x / cbs, cb = blockIdx.x - h * cbs, e = blockIdx.y;
  const int cnt = a.ent_count[e], row0 = a.ent_row0[e], slot = a.ent_slot[e];
  if (cnt <= 0) return;
  const int j = cb * 64 + lane;
  const bool col = j < DV, gated = a.log_decay == nullptr, with_n = gated && cb == 0;
  float* sp = a.S + ((size_t)slot * H + h) * D * DV;
  float* np = gated ? a.N + ((size_t)slot * H + h) * D : nullptr;
  float* mp = gated ? a.M + ((size_t)slot * H + h) * a.mcopies + cb : nullptr;
  float S[DPT], n[NPT];
#pragma unroll
  for (int ii = 0; ii < DPT; ++ii) {
    const int i = sl * DPT + ii;
    S[ii] = col && i < D ? sp[(size_t)i * DV + j] : 0.f;
  }
#pragma unroll
  for (int x = 0; x < NPT; ++x) n[x] = with_n && tid + 256 * x < D ? np[tid + 256 * x] : 0.f;
  float m = gated ? *mp : 0.f;
  const float decay = gated ? 0.f : (float)exp(a.log_decay[h]);
  for (int b0 = 0; b0 < cnt; b0 += RB) {
    const int nb = min(RB, cnt - b0);
    const size_t r0 = (size_t)(row0 + b0);
    float vr[RB];
#pragma unroll
    for (int r = 0; r < RB; ++r) vr[r] = r < nb && col ? a.v[(r0 + r) * a.ldv + (size_t)h * DV + j] : 0.f;
    __syncthreads();   // the batch before is no longer read
    for (int c = tid; c < nb * half; c += 256) {
      const int r = c / half, i = c - r * half;
      rope_sincos((uint32_t)a.tok_pos[r0 + r], a.freq[i], &rot_s[(RB + r) * half + i], &rot_s[r * half + i]);
    }
    if (gated && tid < nb) log_gates(a.gi[(r0 + tid) * a.ldg + h], a.gf[(r0 + tid) * a.ldg + h], a.cap, gi_s[tid], gf_s[tid]);
    if (half) __syncthreads();
    for (int c = tid; c < nb * DP; c += 256) {
      const int r = c / DP, i = c - r * DP;
      float qv = 0.f, kv = 0.f;
      if (i < D) {
        const float* qr = a.q + (r0 + r) * a.ldq + (size_t)h * D;
        const float* kr = a.k + (r0 + r) * a.ldk + (size_t)h * D;
        qv = qr[i];
        kv = kr[i];
        if (i < a.rot_dims) {
          const int p = a.pairs ? i >> 1 : (i < half ? i : i - half);
          const bool first = a.pairs ? (i & 1) == 0 : i < half;
          const int o = a.pairs ? i ^ 1 : (first ? i + half : i - half);
          const float c_ = rot_s[r * half + p], s_ = rot_s[(RB + r) * half + p];
          qv = first ? qv * c_ - qr[o] * s_ : qv * c_ + qr[o] * s_;
          kv = first ? kv * c_ - kr[o] * s_ : kv * c_ + kr[o] * s_;
        }
      }
      qs[r][i] = qv * a.q_scale;
      ks[r][i] = kv * a.k_scale;
    }
    __syncthreads();
    float fl[RB];
#pragma unroll
    for (int r = 0; r < RB; ++r) {
      fl[r] = 0.f;
      if (r < nb) {
        float av = decay, w = 1.f;
        if (gated) {
          const float f = gf_s[r], i = gi_s[r], mn = fmaxf(f + m, i);
          av = expf(f - (mn - m));
          w = expf(i - mn);
          fl[r] = expf(-mn);
          m = mn;
        }
        const float wv = w * vr[r];
        float po = 0.f;
#pragma unroll
        for (int i0 = 0; i0 < DPT; i0 += 4) {
          const f32x4_t q4 = *reinterpret_cast<const f32x4_t*>(&qs[r][sl * DPT + i0]);
          const f32x4_t k4 = *reinterpret_cast<const f32x4_t*>(&ks[r][sl * DPT + i0]);
#pragma unroll
          for (int x = 0; x < 4; ++x) {
            S[i0 + x] = __builtin_fmaf(av, S[i0 + x], k4[x] * wv);
            po = __builtin_fmaf(S[i0 + x], q4[x], po);
          }
        }
        part[r][sl][lane] = po;
        if (with_n) {
          float d = 0.f;
#pragma unroll
          for (int x = 0; x < NPT; ++x) {
            if (tid + 256 * x < DP) {
              n[x] = __builtin_fmaf(av, n[x], w * ks[r][tid + 256 * x]);
              d = __builtin_fmaf(n[x], qs[r][tid + 256 * x], d);
            }
          }
          d = wave_sum(d);
          if (lane == 0) nred[r][sl] = d;
        }
      }
    }
    __syncthreads();
    for (int u = tid; u < nb * 64; u += 256) {
      const int r = u >> 6, c = u & 63;
      if (cb * 64 + c < DV)
        a.out[(r0 + r) * a.ldo + (size_t)h * DV + cb * 64 + c] = (part[r][0][c] + part[r][1][c]) + (part[r][2][c] + part[r][3][c]);
    }
    if (with_n) {
#pragma unroll
      for (int r = 0; r < RB; ++r)
        if (tid == r && r < nb) {
          const float nq = (nred[r][0] + nred[r][1]) + (nred[r][2] + nred[r][3]);
          a.den[(r0 + r) * H + h] = 1.f / (fmaxf(fabsf(nq), fl[r]) + 1e-6f);
        }
    }
  }
#pragma unroll
  for (int ii = 0; ii < DPT; ++ii) {
    const int i = sl * DPT + ii;
    if (col && i < D) sp[(size_t)i * DV + j] = S[ii];
  }
  if (with_n) {
#pragma unroll
    for (int x = 0; x < NPT; ++x)
      if (tid + 256 * x < D) np[tid + 256 * x] = n[x];
  }
  if (gated && tid == 0) *mp = m;
}

// ------------------------------------------------------------------------------------------------ gates of a whole portion
// m_t = max(f_t + m_(t-1), i_t) is a composition of maps m -> max(m + F, M); a workgroup scans 1024 rows of one head at a time.  log a is
// taken as f - (m_t - m_(t-1)): the difference of neighbouring maxima is exact where the decay follows f, so sums of log a stay accurate.
__device__ __forceinline__ void compose(float F1, float M1, float& F2, float& M2) {      // first map 1, then map 2
  M2 = fmaxf(M1 + F2, M2);
  F2 = F1 + F2;
}
__global__ __launch_bounds__(1024) void memory_gates_kernel(DecayArgs a) {
  __shared__ float tF[16], tM[16], m_last;
  const int h = blockIdx.x, e = blockIdx.y, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, H = a.H;
  const int cnt = a.ent_count[e], row0 = a.ent_row0[e];
  if (cnt <= 0) return;
  float* mp = a.M + ((size_t)a.ent_slot[e] * H + h) * a.mcopies;
  float m_in = mp[0];
  for (int b0 = 0; b0 < cnt; b0 += 1024) {
    const int t = b0 + tid;
    const size_t r = (size_t)(row0 + t);
    float i = -INFINITY, f = 0.f;
    if (t < cnt) log_gates(a.gi[r * a.ldg + h], a.gf[r * a.ldg + h], a.cap, i, f);
    float F = f, M = i;
#pragma unroll
    for (int o = 1; o < 64; o <<= 1) {
      const float F1 = __shfl_up(F, o), M1 = __shfl_up(M, o);
      if (lane >= o) compose(F1, M1, F, M);
    }
    __syncthreads();            // totals and m_last of the rows before are no longer read
    if (lane == 63) { tF[wave] = F; tM[wave] = M; }
    __syncthreads();
    float Fw = 0.f, Mw = -INFINITY;
    for (int w = 0; w < wave; ++w) {
      float F2 = tF[w], M2 = tM[w];
      compose(Fw, Mw, F2, M2);
      Fw = F2;
      Mw = M2;
    }
    const float m_wave = fmaxf(m_in + Fw, Mw);                // m before this wave's first row
    const float m = fmaxf(m_wave + F, M);
    float m_prev = __shfl_up(m, 1);
    if (lane == 0) m_prev = m_wave;
    if (t < cnt) {
      a.la[r * H + h] = f - (m - m_prev);
      a.gain[r * H + h] = expf(i - m);
      a.floor_[r * H + h] = expf(-m);
    }
    if (t == min(cnt, b0 + 1024) - 1) m_last = m;
    __syncthreads();
    m_in = m_last;
  }
  if (tid < a.mcopies) mp[tid] = m_in;
}

// ------------------------------------------------------------------------------------------------ chunks on the f32 matrix instructions
// v_mfma_f32_16x16x4: lane l holds A[l & 15][l >> 4], B[l >> 4][l & 15] and C[(l >> 4) * 4 + r][l & 15], r < 4
__device__ __forceinline__ f32x4_t mfma_f32(float a, float b, const f32x4_t& c) { return __builtin_amdgcn_mfma_f32_16x16x4f32(a, b, c, 0, 0, 0); }

// the chunk's running sums of log a (f64, inclusive) and its row weights w -> LDS, by the first wave
__device__ __forceinline__ void chunk_logs(const DecayArgs& a, int h, size_t r0, int n, double* Ls, float* gs) {
  if (threadIdx.x < 64) {
    const int t = threadIdx.x;
    if (a.log_decay) {
      Ls[t] = a.log_decay[h] * (double)min(t + 1, n);
      gs[t] = t < n ? 1.f : 0.f;
    } else {
      double L = t < n ? (double)a.la[(r0 + t) * a.H + h] : 0.0;
#pragma unroll
      for (int o = 1; o < 64; o <<= 1) {
        const double p = __shfl_up(L, o);
        if (t >= o) L += p;
      }
      Ls[t] = L;
      gs[t] = t < n ? a.gain[(r0 + t) * a.H + h] : 0.f;
    }
  }
}

// 4 consecutive elements of a row, zeros past `left` (VEC: the row is 16-byte aligned and its length a multiple of 4)
template <bool VEC>
__device__ __forceinline__ f32x4_t load4(const float* p, int left, bool ok) {
  f32x4_t r = {0.f, 0.f, 0.f, 0.f};
  if (!ok || left <= 0) return r;
  if constexpr (VEC) r = *reinterpret_cast<const f32x4_t*>(p);
  else {
#pragma unroll
    for (int i = 0; i < 4; ++i)
      if (i < left) r[i] = p[i];
  }
  return r;
}

// (1) U = sum_s exp(L - L_s) w_s k_s v_s^T of one chunk: a workgroup owns 64 key channels (16 per wave) and 16 * NV value columns
template <int NV, bool VEC>
__global__ __launch_bounds__(256) void decay_chunk_state_kernel(DecayArgs a) {
  constexpr int CB = 16 * NV, PK = 68, PV = CB + 4;
  __shared__ __attribute__((aligned(16))) float ks[CHUNK * PK];
  __shared__ __attribute__((aligned(16))) float vs[CHUNK * PV];
  __shared__ double Ls[CHUNK];
  __shared__ float gs[CHUNK];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, ni = lane & 15, kb = lane >> 4;
  const int D = a.D, DV = a.DV, H = a.H, cbs = (DV + CB - 1) / CB, dbs = (D + 63) / 64;
  const int e = blockIdx.z, ch = blockIdx.x;
  int y = blockIdx.y;
  const int h = y / (cbs * dbs);
  y -= h * cbs * dbs;
  const int cb = y / dbs, d0 = (y - cb * dbs) * 64;
  const int cnt = a.ent_count[e], lo = ch * CHUNK;
  if (lo >= cnt) return;
  const int n = min(CHUNK, cnt - lo);
  const size_t r0 = (size_t)(a.ent_row0[e] + lo);
  chunk_logs(a, h, r0, n, Ls, gs);
  f32x4_t kreg[4], vreg[NV];
#pragma unroll
  for (int u = 0; u < 4; ++u) {
    const int s = (tid + 256 * u) >> 4, c = ((tid + 256 * u) & 15) * 4;
    kreg[u] = load4<VEC>(a.k + (r0 + s) * a.ldk + (size_t)h * D + d0 + c, D - d0 - c, s < n);
  }
#pragma unroll
  for (int u = 0; u < NV; ++u) {
    const int i = tid + 256 * u, s = i / (CB / 4), c = (i - s * (CB / 4)) * 4;
    vreg[u] = load4<VEC>(a.v + (r0 + s) * a.ldv + (size_t)h * DV + cb * CB + c, DV - cb * CB - c, s < n);
  }
  __syncthreads();
  const double Ltot = Ls[CHUNK - 1];
#pragma unroll
  for (int u = 0; u < 4; ++u) {
    const int s = (tid + 256 * u) >> 4, c = ((tid + 256 * u) & 15) * 4;
    const float w = gs[s] * a.k_scale * expf((float)(Ltot - Ls[s]));
    *reinterpret_cast<f32x4_t*>(&ks[s * PK + c]) = f32x4_t{kreg[u][0] * w, kreg[u][1] * w, kreg[u][2] * w, kreg[u][3] * w};
  }
#pragma unroll
  for (int u = 0; u < NV; ++u) {
    const int i = tid + 256 * u, s = i / (CB / 4), c = (i - s * (CB / 4)) * 4;
    *reinterpret_cast<f32x4_t*>(&vs[s * PV + c]) = vreg[u];
  }
  __syncthreads();
  float* rec = a.ws + (((size_t)e * a.max_chunks + ch) * H + h) * chunk_rec(D, DV);
  if (cb == 0) {
    if (a.den && tid < 64 && d0 + tid < D) {
      float s_ = 0.f;
      for (int s = 0; s < CHUNK; ++s) s_ += ks[s * PK + tid];
      rec[(size_t)D * DV + d0 + tid] = s_;
    }
    if (d0 == 0 && tid == 64) rec[(size_t)D * DV + D] = expf((float)Ltot);
  }
  if (d0 + wave * 16 >= D) return;
  f32x4_t acc[NV];
#pragma unroll
  for (int v = 0; v < NV; ++v) acc[v] = f32x4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll
  for (int g = 0; g < CHUNK / 16; ++g) {
    if (g * 16 >= n) break;
#pragma unroll
    for (int x = 0; x < 4; ++x) {
      const int s = g * 16 + kb * 4 + x;
      const float av = ks[s * PK + wave * 16 + ni];
#pragma unroll
      for (int v = 0; v < NV; ++v) acc[v] = mfma_f32(av, vs[s * PV + v * 16 + ni], acc[v]);
    }
  }
#pragma unroll
  for (int v = 0; v < NV; ++v)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int d = d0 + wave * 16 + kb * 4 + r, c = cb * CB + v * 16 + ni;
      if (d < D && c < DV) rec[(size_t)d * DV + c] = acc[v][r];
    }
}

// (2) per element of S (and n), chunks in order: record <- the state the chunk starts from;  S <- exp(L) S + record
__global__ __launch_bounds__(256) void decay_carry_kernel(DecayArgs a) {
  const int e = blockIdx.z, h = blockIdx.y, idx = blockIdx.x * 256 + threadIdx.x;
  const int cnt = a.ent_count[e], slot = a.ent_slot[e], DDV = a.D * a.DV;
  if (cnt <= 0 || idx >= DDV + (a.den ? a.D : 0)) return;
  const int chunks = (cnt + CHUNK - 1) / CHUNK;
  const size_t rec = chunk_rec(a.D, a.DV), step = (size_t)a.H * rec;
  float* home = idx < DDV ? a.S + ((size_t)slot * a.H + h) * DDV + idx : a.N + ((size_t)slot * a.H + h) * a.D + (idx - DDV);
  float S = *home;
  float* w0 = a.ws + ((size_t)e * a.max_chunks * a.H + h) * rec;
  constexpr int U8 = 8;       // eight chunks' records in flight: the chain itself is eight dependent multiply-adds
  for (int c0 = 0; c0 < chunks; c0 += U8) {
    float U[U8], A[U8];
#pragma unroll
    for (int x = 0; x < U8; ++x) {
      const int ch = min(c0 + x, chunks - 1);
      U[x] = w0[ch * step + idx];
      A[x] = w0[ch * step + DDV + a.D];
    }
#pragma unroll
    for (int x = 0; x < U8; ++x)
      if (c0 + x < chunks) {
        w0[(c0 + x) * step + idx] = S;
        S = __builtin_fmaf(A[x], S, U[x]);
      }
  }
  *home = S;
}

// (3) the outputs of one chunk: a workgroup owns 16 * NV value columns of one head, wave w the rows 16 w .. + 16 (lane ni: row 16 w + ni).
// Transposed throughout: P^T = K Q^T leaves its accumulators exactly as the B operand of O^T += V^T P^T wants them.
template <int NV, bool VEC>
__global__ __launch_bounds__(256) void decay_chunk_out_kernel(DecayArgs a) {
  constexpr int CB = 16 * NV, DB = 32, PQ = DB + 4, PS = CB + 4;
  __shared__ __attribute__((aligned(16))) float qs[CHUNK * PQ];
  __shared__ __attribute__((aligned(16))) float ks[CHUNK * PQ];
  __shared__ __attribute__((aligned(16))) float ss[DB * PS];      // a block of the start state, later 32 rows of v
  __shared__ double Ls[CHUNK];
  __shared__ float gs[CHUNK], ns[DB];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, ni = lane & 15, kb = lane >> 4;
  const int D = a.D, DV = a.DV, H = a.H, cbs = (DV + CB - 1) / CB;
  const int e = blockIdx.z, ch = blockIdx.x, h = blockIdx.y / cbs, cb = blockIdx.y - h * cbs;
  const int cnt = a.ent_count[e], lo = ch * CHUNK;
  if (lo >= cnt) return;
  const int n = min(CHUNK, cnt - lo);
  const size_t r0 = (size_t)(a.ent_row0[e] + lo);
  const float* rec = a.ws + (((size_t)e * a.max_chunks + ch) * H + h) * chunk_rec(D, DV);
  const bool with_n = a.den != nullptr && cb == 0;
  chunk_logs(a, h, r0, n, Ls, gs);
  constexpr int SU = DB * CB / 4 / 256;      // start-state units of 4 per thread and block (2 or 4)
  f32x4_t qreg[2], kreg[2], sreg[SU];
  auto fetch = [&](int d0) {
#pragma unroll
    for (int u = 0; u < 2; ++u) {
      const int t = (tid + 256 * u) >> 3, c = ((tid + 256 * u) & 7) * 4;
      qreg[u] = load4<VEC>(a.q + (r0 + t) * a.ldq + (size_t)h * D + d0 + c, D - d0 - c, t < n);
      kreg[u] = load4<VEC>(a.k + (r0 + t) * a.ldk + (size_t)h * D + d0 + c, D - d0 - c, t < n);
    }
#pragma unroll
    for (int u = 0; u < SU; ++u) {
      const int i = tid + 256 * u, d = d0 + i / (CB / 4), c = cb * CB + (i % (CB / 4)) * 4;
      sreg[u] = load4<VEC>(rec + (size_t)d * DV + c, DV - c, d < D);
    }
  };
  const f32x4_t z4 = {0.f, 0.f, 0.f, 0.f};
  f32x4_t P[4] = {z4, z4, z4, z4}, O[NV];
#pragma unroll
  for (int v = 0; v < NV; ++v) O[v] = z4;
  float nq = 0.f;
  fetch(0);
  for (int d0 = 0; d0 < D; d0 += DB) {
    __syncthreads();       // the block before is no longer read (first: publishes nothing yet)
#pragma unroll
    for (int u = 0; u < 2; ++u) {
      const int t = (tid + 256 * u) >> 3, c = ((tid + 256 * u) & 7) * 4;
      *reinterpret_cast<f32x4_t*>(&qs[t * PQ + c]) = qreg[u] * a.q_scale;
      *reinterpret_cast<f32x4_t*>(&ks[t * PQ + c]) = kreg[u];
    }
#pragma unroll
    for (int u = 0; u < SU; ++u) {
      const int i = tid + 256 * u;
      *reinterpret_cast<f32x4_t*>(&ss[(i / (CB / 4)) * PS + (i % (CB / 4)) * 4]) = sreg[u];
    }
    if (with_n && tid < DB) ns[tid] = d0 + tid < D ? rec[(size_t)D * DV + d0 + tid] : 0.f;
    __syncthreads();
    if (d0 + DB < D) fetch(d0 + DB);
#pragma unroll
    for (int dd = 0; dd < DB / 16; ++dd) {
      const f32x4_t qf = *reinterpret_cast<const f32x4_t*>(&qs[(wave * 16 + ni) * PQ + dd * 16 + kb * 4]);
#pragma unroll
      for (int st = 0; st < 4; ++st) {
        if (st <= wave) {
          const f32x4_t kf = *reinterpret_cast<const f32x4_t*>(&ks[(st * 16 + ni) * PQ + dd * 16 + kb * 4]);
#pragma unroll
          for (int x = 0; x < 4; ++x) P[st] = mfma_f32(kf[x], qf[x], P[st]);
        }
      }
#pragma unroll
      for (int x = 0; x < 4; ++x) {
        const float* sr = &ss[(dd * 16 + kb * 4 + x) * PS + ni];
#pragma unroll
        for (int v = 0; v < NV; ++v) O[v] = mfma_f32(sr[v * 16], qf[x], O[v]);
      }
      if (with_n) {
#pragma unroll
        for (int x = 0; x < 4; ++x) nq = __builtin_fmaf(qf[x], ns[dd * 16 + kb * 4 + x], nq);
      }
    }
  }
  // weights of the chunk's own rows, and the start state's share scaled by its decay
  const int t = wave * 16 + ni;
  const double Lt = Ls[t];
  const float et = expf((float)Lt);
  nq *= et;
#pragma unroll
  for (int v = 0; v < NV; ++v) O[v] = O[v] * et;
#pragma unroll
  for (int st = 0; st < 4; ++st)
#pragma unroll
    for (int x = 0; x < 4; ++x) {
      const int s = st * 16 + kb * 4 + x;
      float p = 0.f;
      if (s <= t) p = P[st][x] * (expf((float)(Lt - Ls[s])) * (gs[s] * a.k_scale));
      P[st][x] = p;
      nq += p;
    }
  // + V^T P^T, 32 rows of v at a time
  for (int s0 = 0; s0 < n; s0 += 32) {
    __syncthreads();
#pragma unroll
    for (int u = 0; u < SU; ++u) {
      const int i = tid + 256 * u, s = i / (CB / 4), c = (i % (CB / 4)) * 4;
      *reinterpret_cast<f32x4_t*>(&ss[s * PS + c]) =
          load4<VEC>(a.v + (r0 + s0 + s) * a.ldv + (size_t)h * DV + cb * CB + c, DV - cb * CB - c, s0 + s < n);
    }
    __syncthreads();
#pragma unroll
    for (int st = 0; st < 4; ++st) {
      if (st * 16 >= s0 && st * 16 < s0 + 32 && st <= wave) {
#pragma unroll
        for (int x = 0; x < 4; ++x) {
          const float* vr = &ss[(st * 16 - s0 + kb * 4 + x) * PS + ni];
#pragma unroll
          for (int v = 0; v < NV; ++v) O[v] = mfma_f32(vr[v * 16], P[st][x], O[v]);
        }
      }
    }
  }
  if (t >= n) return;
  float* o = a.out + (r0 + t) * a.ldo + (size_t)h * DV + cb * CB + kb * 4;
#pragma unroll
  for (int v = 0; v < NV; ++v) {
    const int c = cb * CB + v * 16 + kb * 4;
    if constexpr (VEC) {
      if (c < DV) *reinterpret_cast<f32x4_t*>(o + v * 16) = O[v];
    } else {
#pragma unroll
      for (int r = 0; r < 4; ++r)
        if (c + r < DV) o[v * 16 + r] = O[v][r];
    }
  }
  if (with_n) {
    nq = rows_sum(nq);        // over kb: the four lanes that share row t (all active or none: t is theirs)
    if (kb == 0) a.den[(r0 + t) * H + h] = 1.f / (fmaxf(fabsf(nq), a.floor_[(r0 + t) * H + h]) + 1e-6f);
  }
}

}  // namespace
}  // namespace dihip

using namespace dihip;

static size_t decay_gate_floats(int T, int H) { return ((size_t)3 * T * H + 3) & ~(size_t)3; }

// rope_rows: the rows that hold q and k at q_off and k_off (chunked retention rotates them in place first; NULL: no rotation)
static int decay_run(hipStream_t s, DecayArgs a, int T, int E, int max_count, int chunked, float* rope_rows, long rope_ld, int q_off, int k_off, void* ws) {
  const int H = a.H, D = a.D, DV = a.DV, cbs64 = (DV + 63) / 64;
  if (!chunked) {
    const size_t lds = (size_t)RB * a.rot_dims * sizeof(float);
    const dim3 grid(H * cbs64, E);
    auto go = [&](auto dpt) { hipLaunchKernelGGL((decay_rows_kernel<decltype(dpt)::value>), grid, dim3(256), lds, s, a); };
    if (D <= 64) go(std::integral_constant<int, 16>{});
    else if (D <= 128) go(std::integral_constant<int, 32>{});
    else if (D <= 256) go(std::integral_constant<int, 64>{});
    else go(std::integral_constant<int, 128>{});
    return launch_status();
  }
  const int chunks = (max_count + CHUNK - 1) / CHUNK;
  a.max_chunks = chunks;
  float* w = (float*)ws;
  if (!a.log_decay) {
    a.la = w;
    a.gain = w + (size_t)T * H;
    a.floor_ = w + (size_t)2 * T * H;
    w += decay_gate_floats(T, H);
    hipLaunchKernelGGL(memory_gates_kernel, dim3(H, E), dim3(1024), 0, s, a);
  }
  a.ws = w;
  if (a.rot_dims) {
    const int work = 2 * H * (a.rot_dims >> 1);
    hipLaunchKernelGGL(rope_rows_kernel, dim3(T, T >= 256 ? 1 : (work + 255) / 256), dim3(256), 0, s, rope_rows, rope_ld, q_off, H, k_off, H, D, a.rot_dims,
                       a.pairs, a.freq, a.tok_pos);
  }
  const auto al = [](const void* p) { return (reinterpret_cast<uintptr_t>(p) & 15u) == 0; };
  const bool vec = D % 4 == 0 && DV % 4 == 0 && al(a.q) && al(a.k) && al(a.v) && al(a.out) && al(a.ws) && a.ldq % 4 == 0 && a.ldk % 4 == 0 &&
                   a.ldv % 4 == 0 && a.ldo % 4 == 0;
  auto go = [&](auto nv, auto ve) {
    constexpr int NV = decltype(nv)::value;
    constexpr bool VEC = decltype(ve)::value;
    const int cbs = (DV + 16 * NV - 1) / (16 * NV);
    hipLaunchKernelGGL((decay_chunk_state_kernel<NV, VEC>), dim3(chunks, H * cbs * ((D + 63) / 64), E), dim3(256), 0, s, a);
    hipLaunchKernelGGL(decay_carry_kernel, dim3((D * DV + (a.den ? D : 0) + 255) / 256, H, E), dim3(256), 0, s, a);
    hipLaunchKernelGGL((decay_chunk_out_kernel<NV, VEC>), dim3(chunks, H * cbs, E), dim3(256), 0, s, a);
  };
  auto by_v = [&](auto ve) {
    if (DV <= 64) go(std::integral_constant<int, 4>{}, ve);
    else go(std::integral_constant<int, 8>{}, ve);
  };
  if (vec) by_v(std::true_type{});
  else by_v(std::false_type{});
  return launch_status();
}

static int decay_check(const char* what, int T, int E, int max_count, int H, int D, int DV, int chunked, int gated, const void* ws, size_t ws_bytes) {
  DIHIP_REQUIRE(T >= 0 && E >= 0 && max_count >= 0 && max_count <= T && H > 0 && D > 0 && DV > 0, DIHIP_PARAM_ERROR, "%s: bad shape", what);
  DIHIP_REQUIRE(D <= 512, DIHIP_EXCEED_LIMIT_ERROR, "%s: more than 512 key channels per head (%d)", what, D);
  DIHIP_REQUIRE((long)H * ((DV + 63) / 64) * ((D + 63) / 64) <= 65535 && E <= 65535, DIHIP_PARAM_ERROR, "%s: too many heads or portions for one launch", what);
  const size_t need = dihip_decay_attn_workspace_bytes(T, E, max_count, H, D, DV, gated, chunked);
  DIHIP_REQUIRE(need == 0 || (ws && ws_bytes >= need && (reinterpret_cast<uintptr_t>(ws) & 15u) == 0), DIHIP_PARAM_ERROR, "%s: workspace too small", what);
  return DIHIP_SUCCESS;
}

extern "C" {

size_t dihip_decay_attn_workspace_bytes(int T, int E, int max_count, int H, int D, int DV, int gated, int chunked) {
  if (!chunked) return 0;
  return ((gated ? decay_gate_floats(T, H) : 0) + (size_t)E * ((max_count + CHUNK - 1) / CHUNK) * H * chunk_rec(D, DV)) * sizeof(float);
}

int dihip_retention(void* stream, float* out, long ldo, float* rows, long ld, int q_off, int k_off, int v_off, float k_scale, const double* log_decay,
                    const float* freq, int rot_dims, int layout, float* state, const int32_t* tok_pos, const int32_t* ent_slot,
                    const int32_t* ent_row0, const int32_t* ent_count, int T, int E, int max_count, int H, int D, int DV, int chunked, void* ws,
                    size_t ws_bytes) {
  if (int rc = decay_check("retention", T, E, max_count, H, D, DV, chunked, 0, ws, ws_bytes)) return rc;
  DIHIP_REQUIRE(out && rows && log_decay && state && tok_pos && ent_slot && ent_row0 && ent_count && ldo >= (long)H * DV && q_off >= 0 && k_off >= 0 &&
                    v_off >= 0 && ld >= (long)q_off + (long)H * D && ld >= (long)k_off + (long)H * D && ld >= (long)v_off + (long)H * DV,
                DIHIP_PARAM_ERROR, "retention: bad argument");
  DIHIP_REQUIRE(rot_dims >= 0 && rot_dims <= D && rot_dims % 2 == 0 && (rot_dims == 0 || freq) && (layout == 0 || layout == 1), DIHIP_PARAM_ERROR,
                "retention: bad rotation (an even number of dimensions up to the head size, layout 0 / 1)");
  if (T == 0 || E == 0 || max_count == 0) return DIHIP_SUCCESS;
  DecayArgs a{};
  a.out = out; a.ldo = ldo;
  a.q = rows + q_off; a.k = rows + k_off; a.v = rows + v_off; a.ldq = a.ldk = a.ldv = ld;
  a.q_scale = 1.f; a.k_scale = k_scale; a.log_decay = log_decay;
  a.freq = freq; a.rot_dims = rot_dims; a.pairs = layout == 0; a.tok_pos = tok_pos;
  a.S = state; a.ent_slot = ent_slot; a.ent_row0 = ent_row0; a.ent_count = ent_count;
  a.H = H; a.D = D; a.DV = DV;
  return decay_run(reinterpret_cast<hipStream_t>(stream), a, T, E, max_count, chunked, rows, ld, q_off, k_off, ws);
}

int dihip_matrix_memory(void* stream, float* out, long ldo, float* den, const float* q, long ldq, const float* k, long ldk, const float* v, long ldv,
                        const float* gate_i, const float* gate_f, long ldg, float cap, float q_scale, float* state_s, float* state_n, float* state_m,
                        int m_copies, const int32_t* ent_slot, const int32_t* ent_row0, const int32_t* ent_count, int T, int E, int max_count,
                        int H, int D, int DV, int chunked, void* ws, size_t ws_bytes) {
  if (int rc = decay_check("matrix_memory", T, E, max_count, H, D, DV, chunked, 1, ws, ws_bytes)) return rc;
  DIHIP_REQUIRE(out && den && q && k && v && gate_i && gate_f && state_s && state_n && state_m && ent_slot && ent_row0 && ent_count &&
                    ldo >= (long)H * DV && ldq >= (long)H * D && ldk >= (long)H * D && ldv >= (long)H * DV && ldg >= H && cap > 0.f,
                DIHIP_PARAM_ERROR, "matrix_memory: bad argument");
  DIHIP_REQUIRE(m_copies == (DV + 63) / 64 && m_copies <= 1024, DIHIP_PARAM_ERROR, "matrix_memory: one copy of the running maximum per 64 value columns");
  if (T == 0 || E == 0 || max_count == 0) return DIHIP_SUCCESS;
  DecayArgs a{};
  a.out = out; a.ldo = ldo; a.den = den;
  a.q = q; a.ldq = ldq; a.k = k; a.ldk = ldk; a.v = v; a.ldv = ldv;
  a.q_scale = q_scale; a.k_scale = 1.f;
  a.gi = gate_i; a.gf = gate_f; a.ldg = ldg; a.cap = cap;
  a.S = state_s; a.N = state_n; a.M = state_m; a.mcopies = m_copies;
  a.ent_slot = ent_slot; a.ent_row0 = ent_row0; a.ent_count = ent_count;
  a.H = H; a.D = D; a.DV = DV;
  return decay_run(reinterpret_cast<hipStream_t>(stream), a, T, E, max_count, chunked, nullptr, 0, 0, 0, ws);
}

}  // extern "C"
