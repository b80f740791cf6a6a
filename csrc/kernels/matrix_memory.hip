// Matrix memory with exponential gates over the engine's per-sequence state slots.  Per (sequence, head), all fp32:
//
//   i = cap tanh((z_i + b_i) / cap),  f = logsigmoid(cap tanh((z_f + b_f) / cap))
//   m' = max(f + m, i)                               running maximum, 0 before the first token
//   S  = e^(f + m - m') S + e^(i - m') k v^T         [D, V]
//   n  = e^(f + m - m') n + e^(i - m') k             [D]
//   o  = S^T q / (max(|n . q|, e^-m') + den_eps)
//   out = o / rms(o) * norm_w * sigmoid(gate) * out_scale       per head, in the element type
//
// Walk (any sizes, both element types): one workgroup per (sequence, head) does everything of a token in one pass.  A
// thread owns 4 neighbouring columns of every RG-th row of S; with few enough rows per thread the state stays in
// registers between the tokens, otherwise it streams through memory.  A decode step is one token: the launch is the
// state's traffic, read and written once in 16-byte pieces.
#include "api_memory.h"
#include "common.h"

namespace dsse {
namespace {

constexpr int kWalkThreads = 512;

DEV float softcap_f(float z, float cap) { return cap * tanhf(z / cap); }
DEV float logsigmoid_f(float x) { return fminf(x, 0.0f) - log1pf(expf(-fabsf(x))); }
DEV float sigmoid_f(float x) { return 1.0f / (1.0f + expf(-x)); }

template <int VEC>
DEV void ld_vec(const float* p, float (&v)[VEC]) {
  if constexpr (VEC == 4) {
    const f32x4 t = ld_global<f32x4>(p);
#pragma unroll
    for (int e = 0; e < 4; ++e) v[e] = t[e];
  } else {
    v[0] = *p;
  }
}
template <int VEC>
DEV void st_vec(float* p, const float (&v)[VEC]) {
  if constexpr (VEC == 4) *reinterpret_cast<f32x4*>(p) = f32x4{v[0], v[1], v[2], v[3]};
  else p[0] = v[0];
}

// NR: rows of S a thread keeps in registers (every row of its share), 0: the state streams through memory per token
template <typename T, int VEC, int NR>
__global__ __launch_bounds__(kWalkThreads) void matrix_memory_walk_kernel(MatrixMemoryParams p) {
  extern __shared__ __align__(16) float lds[];
  const int h = blockIdx.x, seq = blockIdx.y;
  const int ql = p.q_len[seq];
  if (ql <= 0) return;
  const int D = p.D, V = p.V, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  constexpr int kWaves = kWalkThreads / 64;
  const int CG = V / VEC, RG = kWalkThreads / CG;  // column groups, row groups
  const int rg = tid / CG, c0 = (tid - rg * CG) * VEC;
  const bool on = rg < RG;
  float* qs = lds;            // [D] query times its scale
  float* ks = qs + D;         // [D]
  float* red = ks + D;        // [RG][V] partial read-outs
  float* sum1 = red + RG * V; // [kWaves]
  float* sum2 = sum1 + kWaves;
  const int row0 = p.q_start[seq];
  const bool fresh = p.ctx_len[seq] - ql == 0;
  const int64_t entry = (int64_t)p.state_slot[seq] * p.H + h;
  float* st = p.state + entry * D * V;
  float* nm = p.norm + entry * (D + 1);
  float S[NR > 0 ? NR : 1][VEC];
  if constexpr (NR > 0) {
#pragma unroll
    for (int j = 0; j < NR; ++j) {
      const int d = rg + j * RG;
#pragma unroll
      for (int e = 0; e < VEC; ++e) S[j][e] = 0.0f;
      if (on && d < D && !fresh) ld_vec<VEC>(st + (int64_t)d * V + c0, S[j]);
    }
  }
  float n = tid < D && !fresh ? nm[tid] : 0.0f;
  float m = fresh ? 0.0f : nm[D];
  for (int t = 0; t < ql; ++t) {
    const int64_t row = row0 + t;
    const float* z = p.gates + row * p.ldz;
    const float ig = softcap_f(z[h] + p.gate_b[h], p.cap);
    const float fg = logsigmoid_f(softcap_f(z[p.H + h] + p.gate_b[p.H + h], p.cap));
    float k = 0.f, q = 0.f;
    if (tid < D) {
      k = p.k[row * p.ldk + h * D + tid];
      q = p.q[row * p.ldq + h * D + tid] * p.q_scale;
      ks[tid] = k;
      qs[tid] = q;
    }
    float v[VEC];
#pragma unroll
    for (int e = 0; e < VEC; ++e) v[e] = on ? p.v[row * p.ldv + h * V + c0 + e] : 0.0f;
    const float mn = fmaxf(fg + m, ig);
    const float keep = expf(fg + m - mn), put = expf(ig - mn);
    m = mn;
#pragma unroll
    for (int e = 0; e < VEC; ++e) v[e] *= put;
    n = keep * n + put * k;
    const float part = wave_sum(n * q);
    if (lane == 0) sum1[wave] = part;
    __syncthreads();  // q, k and the normaliser's partial products are staged
    float o[VEC];
#pragma unroll
    for (int e = 0; e < VEC; ++e) o[e] = 0.0f;
    if (on) {
      if constexpr (NR > 0) {
#pragma unroll
        for (int j = 0; j < NR; ++j) {
          const int d = rg + j * RG;
          const float kd = d < D ? ks[d] : 0.0f, qd = d < D ? qs[d] : 0.0f;
#pragma unroll
          for (int e = 0; e < VEC; ++e) {
            S[j][e] = keep * S[j][e] + kd * v[e];
            o[e] += S[j][e] * qd;
          }
        }
      } else {
        const bool zero = fresh && t == 0;
        for (int d = rg; d < D; d += RG) {
          float s[VEC];
          float* sp = st + (int64_t)d * V + c0;
#pragma unroll
          for (int e = 0; e < VEC; ++e) s[e] = 0.0f;
          if (!zero) ld_vec<VEC>(sp, s);
#pragma unroll
          for (int e = 0; e < VEC; ++e) {
            s[e] = keep * s[e] + ks[d] * v[e];
            o[e] += s[e] * qs[d];
          }
          st_vec<VEC>(sp, s);
        }
      }
#pragma unroll
      for (int e = 0; e < VEC; ++e) red[rg * V + c0 + e] = o[e];
    }
    float nq = 0.f;
#pragma unroll
    for (int w = 0; w < kWaves; ++w) nq += sum1[w];
    const float den = fmaxf(fabsf(nq), expf(-m)) + p.den_eps;
    __syncthreads();  // the partial read-outs are complete; sum1, q and k have been read
    float y = 0.f;
    if (tid < V) {
      for (int r = 0; r < RG; ++r) y += red[r * V + tid];
      y /= den;
    }
    const float ss = wave_sum(y * y);
    if (lane == 0) sum2[wave] = ss;
    __syncthreads();
    if (tid < V) {
      float tot = 0.f;
#pragma unroll
      for (int w = 0; w < kWaves; ++w) tot += sum2[w];
      const float inv = 1.0f / sqrtf(tot / (float)V + p.eps);
      const float g = sigmoid_f(p.out_gate[row * p.ldg + h * V + tid]);
      reinterpret_cast<T*>(p.out)[row * p.ldo + h * V + tid] = (T)(y * inv * p.norm_w[h * V + tid] * g * p.out_scale);
    }
  }
  if constexpr (NR > 0) {
#pragma unroll
    for (int j = 0; j < NR; ++j) {
      const int d = rg + j * RG;
      if (on && d < D) st_vec<VEC>(st + (int64_t)d * V + c0, S[j]);
    }
  }
  if (tid < D) nm[tid] = n;
  if (tid == 0) nm[D] = m;  // every thread has read the old maximum before the first barrier
}

template <typename T, int VEC>
void launch_walk(const MatrixMemoryParams& p, hipStream_t st) {
  const int CG = p.V / VEC, RG = kWalkThreads / CG, nr = (p.D + RG - 1) / RG;
  const dim3 grid(p.H, p.nseq), block(kWalkThreads);
  const size_t lds = (size_t)(2 * p.D + RG * p.V + 2 * (kWalkThreads / 64)) * sizeof(float);
#define DSSE_WALK(n) hipLaunchKernelGGL((matrix_memory_walk_kernel<T, VEC, n>), grid, block, lds, st, p)
  if (nr <= 2) DSSE_WALK(2);
  else if (nr <= 4) DSSE_WALK(4);
  else if (nr <= 8) DSSE_WALK(8);
  else if (nr <= 16) DSSE_WALK(16);
  else DSSE_WALK(0);
#undef DSSE_WALK
}

// ---------------------------------------------------------------------------------------------------------------------
// Chunk form for prompt portions.  The running maximum only rescales, so it is settled first:
//
//   memory_gates   the maximum is a scan of the pairs (sum of f, best i + later f's); log a_t = f_t + m_(t-1) - m_t and
//                  log b_t = i_t - m_t are both <= 0.  Left behind: A_t = the sum of log a inside its 32-token chunk,
//                  u_t = log b_t - A_t (both times log2 e), and m_t.
//   memory_chunk   S_t = a_t S_(t-1) + b_t k v^T over chunks of 32 tokens.  For s <= t of one chunk the write of s weighs
//                  e^(A_t + u_s) in t's read-out, the incoming state e^(A_t):
//                      O = e^A (Q S_in) + (Q K^T * W) V,     S_out = e^(A_end) S_in + sum_s e^(A_end + u_s) k_s v_s^T
//   memory_out     division, head norm, gate
//
// memory_chunk: a wave owns 16 columns of one (sequence, head): all D rows of S for them sit in its MFMA accumulators
// (row 4 g + i of tile dt, column r) for the whole portion.  The accumulator layout of S is at the same time the A operand of
// O^T = S^T Q^T (row = column of S, k axis = its rows) when Q's coordinates are staged in the order the accumulators hold
// them, and the accumulator layout of the scores S^T[s, t] is the B operand of O^T += V^T P^T: neither passes through LDS.
// The four waves of a workgroup share the staged q, k (rows, for the scores) and k transposed (for the state's update).
// The normaliser is one more 16-column tile whose "values" are 1 in its first column.
//
// Operands are bf16 where they are projections (q, k, v); what the recurrence makes -- the state, the write strengths, the
// weighted scores -- enters as two bf16 parts (value and remainder), so a product carries about 16 bits of it; sums and the
// state itself are fp32.
constexpr int kChunk = 32;
constexpr float kLog2e = 1.4426950408889634f;

// Where a sequence's chunk sums start in acum / u: the rows keep their order, every start is a multiple of four floats.
DEV int sums_at(int row0, int seq) { return ((row0 + 3) & ~3) + 4 * seq; }

// Sixteen waves per (sequence, head) take 1024 tokens at a time: a wave scans its 64, the waves' totals meet in LDS, and
// every wave folds those before it.
constexpr int kGateWaves = 16;

__global__ __launch_bounds__(64 * kGateWaves) void memory_gates_kernel(MatrixMemoryParams p) {
  __shared__ float tot_f[2][kGateWaves], tot_m[2][kGateWaves];
  const int h = blockIdx.x, seq = blockIdx.y, lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int ql = p.q_len[seq];
  if (ql <= 0) return;
  const int row0 = p.q_start[seq];
  float* nm = p.norm + ((int64_t)p.state_slot[seq] * p.H + h) * (p.D + 1);
  float m_in = p.ctx_len[seq] - ql == 0 ? 0.0f : nm[p.D];
  const float bi = p.gate_b[h], bf = p.gate_b[p.H + h];
  float* acum = p.acum + (int64_t)h * p.ldsum + sums_at(row0, seq);
  float* us = p.u + (int64_t)h * p.ldsum + sums_at(row0, seq);
  for (int b = 0, it = 0; b < ql; b += 64 * kGateWaves, ++it) {
    const int t = b + threadIdx.x;
    const bool on = t < ql;
    const float* z = p.gates + (int64_t)(row0 + (on ? t : 0)) * p.ldz + h;
    const float i = on ? softcap_f(z[0] + bi, p.cap) : -INFINITY;
    const float f = on ? logsigmoid_f(softcap_f(z[p.H] + bf, p.cap)) : 0.0f;
    float F = f, M = i;  // sum of f; the largest i plus the f after it
#pragma unroll
    for (int o = 1; o < 64; o <<= 1) {
      const float Fp = __shfl_up(F, o), Mp = __shfl_up(M, o);
      if (lane >= o) {
        M = fmaxf(Mp + F, M);
        F += Fp;
      }
    }
    float *tf = tot_f[it & 1], *tm = tot_m[it & 1];  // two strips: one barrier per round
    if (lane == 63) tf[wave] = F, tm[wave] = M;
    __syncthreads();
    float mw = m_in;  // the maximum ahead of this wave's tokens, and after all of the round's
    for (int w = 0; w < kGateWaves; ++w) {
      if (w == wave) mw = m_in;
      m_in = fmaxf(m_in + tf[w], tm[w]);
    }
    const float m = fmaxf(mw + F, M);
    float mp = __shfl_up(m, 1);
    if (lane == 0) mp = mw;
    float A = on ? f + mp - m : 0.0f;
    const float lb = i - m;
#pragma unroll
    for (int o = 1; o < kChunk; o <<= 1) {
      const float Ap = __shfl_up(A, o);
      if ((lane & (kChunk - 1)) >= o) A += Ap;
    }
    if (on) {
      acum[t] = A * kLog2e;
      us[t] = (lb - A) * kLog2e;
      p.m[(int64_t)(row0 + t) * p.H + h] = m;
    }
  }
  if (threadIdx.x == 0) nm[p.D] = m_in;  // every thread has read the old one before the first barrier
}

// value and remainder of fp32 numbers as bf16 operands
DEV void split8(const float (&x)[8], bf16x8& hi, bf16x8& lo) {
#pragma unroll
  for (int j = 0; j < 8; ++j) {
    hi[j] = (bf16)x[j];
    lo[j] = (bf16)(x[j] - (float)hi[j]);
  }
}
// 2^x (one instruction): arguments here are at most 0 up to rounding
DEV float exp2_hw(float x) { return __builtin_amdgcn_exp2f(x); }
// uniform base, 32-bit lane offset in floats
template <typename V>
DEV V ld_at(const float* base, unsigned off) {
  return ld_global<V>(reinterpret_cast<const char*>(base) + 4u * off);
}

// NK: 32-row groups of S (D rounded up); NW: waves (16-column tiles) per workgroup; VEC: 16-byte loads of q and k rows
template <int NK, int NW, bool VEC>
__global__ __launch_bounds__(64 * NW) void memory_chunk_kernel(MatrixMemoryParams p) {
  constexpr int Dp = 32 * NK, ldr = Dp + 8, ldt = kChunk + 8;
  constexpr int Q4 = 8 * NK;                  // 4-coordinate pieces of a row
  constexpr int NB = (NK + NW - 1) / NW;      // 4 x 4 pieces (tokens x coordinates) a thread stages
  __shared__ __align__(16) bf16 qs[kChunk * ldr], ks[kChunk * ldr], kt[Dp * ldt];
  const int h = blockIdx.y, seq = blockIdx.z;
  const int ql = p.q_len[seq];
  if (ql <= 0) return;
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, r = lane & 15, g = lane >> 4;
  const int D = p.D, V = p.V;
  const int vtiles = (V + 15) / 16;
  const int ct = blockIdx.x * NW + wave;      // this wave's column tile; vtiles: the normaliser's
  const bool live = ct <= vtiles, is_norm = ct == vtiles;
  const int col = ct * 16 + r;
  const bool col_on = live && !is_norm && col < V;
  const int row0 = p.q_start[seq];
  const bool fresh = p.ctx_len[seq] - ql == 0;
  const int64_t entry = (int64_t)p.state_slot[seq] * p.H + h;
  float* st = p.state + entry * D * V + col;
  float* nm = p.norm + entry * (D + 1);
  f32x4 S[2 * NK];
#pragma unroll
  for (int dt = 0; dt < 2 * NK; ++dt)
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int d = 16 * dt + 4 * g + i;
      float s = 0.0f;
      if (!fresh && d < D) {
        if (col_on) s = st[(int64_t)d * V];
        else if (is_norm && r == 0) s = nm[d];
      }
      S[dt][i] = s;
    }
  // The next chunk's inputs, requested while the current one is in the MFMAs.  Lane offsets are 32-bit and the same for
  // every chunk, the moving part of an address is uniform.
  f32x4 nk[NB][4], nq[NB][4], nu[2];
  float nv[8], nA0, nA1, nAL;
  const int64_t sums = (int64_t)h * p.ldsum + sums_at(row0, seq);
  unsigned koff[NB], qoff[NB];
  bool piece[NB];
#pragma unroll
  for (int n = 0; n < NB; ++n) {
    const int b = n * 64 * NW + tid, d = 4 * (b % Q4), tq = 4 * (b / Q4);
    piece[n] = b < 64 * NK && d < D;
    koff[n] = piece[n] ? (unsigned)(tq * p.ldk + d) : 0u;  // pieces that do not exist read the first one and are masked
    qoff[n] = piece[n] ? (unsigned)(tq * p.ldq + d) : 0u;
  }
  const unsigned voff = col_on ? (unsigned)(4 * g * p.ldv + col) : 0u;
  const f32x4 zero4 = f32x4{0.f, 0.f, 0.f, 0.f};
  auto ld4 = [&](const float* base, unsigned off) {
    if constexpr (VEC) return ld_at<f32x4>(base, off);
    else return f32x4{ld_at<float>(base, off), ld_at<float>(base, off + 1), ld_at<float>(base, off + 2), ld_at<float>(base, off + 3)};
  };
  auto request = [&](int t0) {  // no branch around a load: all of them are in flight together
    const int nt = ql - t0 < kChunk ? ql - t0 : kChunk;
    const int64_t row = row0 + t0;
    const float* kb = p.k + row * p.ldk + h * D;
    const float* qb = p.q + row * p.ldq + h * D;
    const float* vb = p.v + row * p.ldv + h * V;
    const float *Ab = p.acum + sums + t0, *ub = p.u + sums + t0;
    if (nt == kChunk) {
#pragma unroll
      for (int n = 0; n < NB; ++n)
#pragma unroll
        for (int j = 0; j < 4; ++j) {
          nk[n][j] = ld4(kb + j * p.ldk, koff[n]);
          nq[n][j] = ld4(qb + j * p.ldq, qoff[n]);
        }
#pragma unroll
      for (int j = 0; j < 8; ++j) nv[j] = ld_at<float>(vb + ((j & 3) + 16 * (j >> 2)) * p.ldv, voff);
      nu[0] = ld_at<f32x4>(ub, 4 * g);
      nu[1] = ld_at<f32x4>(ub + 16, 4 * g);
      nA0 = ld_at<float>(Ab, r);
      nA1 = ld_at<float>(Ab + 16, r);
      nAL = Ab[kChunk - 1];
    } else {  // the last tokens: rows past the end read the first one (masked below), their sums are the last token's
#pragma unroll
      for (int n = 0; n < NB; ++n) {
        const int tq = 4 * ((n * 64 * NW + tid) / Q4);
#pragma unroll
        for (int j = 0; j < 4; ++j) {
          const bool on = piece[n] && tq + j < nt;
          nk[n][j] = ld4(kb, on ? koff[n] + j * p.ldk : 0u);
          nq[n][j] = ld4(qb, on ? qoff[n] + j * p.ldq : 0u);
        }
      }
#pragma unroll
      for (int j = 0; j < 8; ++j) {
        const int c = (j & 3) + 16 * (j >> 2), s = 4 * g + c;
        nv[j] = ld_at<float>(vb, s < nt ? voff + c * p.ldv : 0u);
        nu[j >> 2][j & 3] = ld_at<float>(ub, s < nt ? s : nt - 1);
      }
      nA0 = ld_at<float>(Ab, r < nt ? r : nt - 1);
      nA1 = ld_at<float>(Ab, 16 + r < nt ? 16 + r : nt - 1);
      nAL = Ab[nt - 1];
    }
  };
  auto place = [](int x) { return (x & ~31) + ((x & 15) >> 2) * 8 + ((x >> 4) & 1) * 4 + (x & 3); };
  request(0);
  for (int t0 = 0; t0 < ql; t0 += kChunk) {
    const int nt = ql - t0 < kChunk ? ql - t0 : kChunk;
    if (nt < kChunk || D < Dp) {  // uniform: rows and coordinates that do not exist are zeros
#pragma unroll
      for (int n = 0; n < NB; ++n)
#pragma unroll
        for (int j = 0; j < 4; ++j)
          if (!piece[n] || 4 * ((n * 64 * NW + tid) / Q4) + j >= nt) nk[n][j] = nq[n][j] = zero4;
    }
#pragma unroll
    for (int n = 0; n < NB; ++n) {
      const int b = n * 64 * NW + tid;
      if (b < 64 * NK) {
        const int d = 4 * (b % Q4), tq = 4 * (b / Q4);
#pragma unroll
        for (int j = 0; j < 4; ++j) {
          bf16x4 qv, kv, kc;
#pragma unroll
          for (int e = 0; e < 4; ++e) {
            qv[e] = (bf16)(nq[n][j][e] * p.q_scale);
            kv[e] = (bf16)nk[n][j][e];
            kc[e] = (bf16)nk[n][e][j];  // coordinate d + j of the four tokens
          }
          *reinterpret_cast<bf16x4*>(qs + (tq + j) * ldr + place(d)) = qv;
          *reinterpret_cast<bf16x4*>(ks + (tq + j) * ldr + place(d)) = kv;
          *reinterpret_cast<bf16x4*>(kt + (d + j) * ldt + place(tq)) = kc;
        }
      }
    }
    float v[8], u[8];
#pragma unroll
    for (int j = 0; j < 8; ++j) {
      const bool in = nt == kChunk || 4 * g + (j & 3) + 16 * (j >> 2) < nt;
      v[j] = is_norm ? (r == 0 && in ? 1.0f : 0.0f) : (col_on && in ? nv[j] : 0.0f);
      u[j] = nu[j >> 2][j & 3];
    }
    const float A0 = nA0, A1 = nA1, AL = nAL;
    lds_barrier();
    if (t0 + kChunk < ql) request(t0 + kChunk);
    if (live) {
      f32x4 O0 = zero4, O1 = zero4, s00 = zero4, s01 = zero4, s11 = zero4;
#pragma unroll
      for (int k = 0; k < NK; ++k) {
        const bf16x8 q0 = *reinterpret_cast<const bf16x8*>(qs + r * ldr + 32 * k + 8 * g);
        const bf16x8 q1 = *reinterpret_cast<const bf16x8*>(qs + (16 + r) * ldr + 32 * k + 8 * g);
        const bf16x8 k0 = *reinterpret_cast<const bf16x8*>(ks + r * ldr + 32 * k + 8 * g);
        const bf16x8 k1 = *reinterpret_cast<const bf16x8*>(ks + (16 + r) * ldr + 32 * k + 8 * g);
        s00 = mfma16x16x32(k0, q0, s00);
        s01 = mfma16x16x32(k0, q1, s01);
        s11 = mfma16x16x32(k1, q1, s11);
        float x[8];
#pragma unroll
        for (int i = 0; i < 4; ++i) x[i] = S[2 * k][i], x[4 + i] = S[2 * k + 1][i];
        bf16x8 hi, lo;
        split8(x, hi, lo);
        O0 = mfma16x16x32(hi, q0, O0);
        O1 = mfma16x16x32(hi, q1, O1);
        O0 = mfma16x16x32(lo, q0, O0);
        O1 = mfma16x16x32(lo, q1, O1);
      }
      const float e0 = exp2_hw(A0), e1 = exp2_hw(A1), eL = exp2_hw(AL);
      float P0[8], P1[8], vw[8];
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        O0[i] *= e0;
        O1[i] *= e1;
        const bool seen = 4 * g + i <= r;
        P0[i] = seen ? s00[i] * exp2_hw(A0 + u[i]) : 0.0f;
        P0[4 + i] = 0.0f;
        P1[i] = s01[i] * exp2_hw(A1 + u[i]);
        P1[4 + i] = seen ? s11[i] * exp2_hw(A1 + u[4 + i]) : 0.0f;
      }
      bf16x8 vb, hi, lo;
#pragma unroll
      for (int j = 0; j < 8; ++j) {
        vb[j] = (bf16)v[j];
        vw[j] = v[j] * exp2_hw(AL + u[j]);
      }
      split8(P0, hi, lo);
      O0 = mfma16x16x32(vb, hi, O0);
      O0 = mfma16x16x32(vb, lo, O0);
      split8(P1, hi, lo);
      O1 = mfma16x16x32(vb, hi, O1);
      O1 = mfma16x16x32(vb, lo, O1);
      split8(vw, hi, lo);
#pragma unroll
      for (int dt = 0; dt < 2 * NK; ++dt) {
        const bf16x8 kf = *reinterpret_cast<const bf16x8*>(kt + (16 * dt + r) * ldt + 8 * g);
        f32x4 s = S[dt];
#pragma unroll
        for (int i = 0; i < 4; ++i) s[i] *= eL;
        s = mfma16x16x32(kf, hi, s);
        S[dt] = mfma16x16x32(kf, lo, s);
      }
      const int c4 = ct * 16 + 4 * g;  // O^T: rows are columns c4 .. c4 + 3, the lane's token is r (and 16 + r)
#pragma unroll
      for (int b = 0; b < 2; ++b) {
        const f32x4 o = b == 0 ? O0 : O1;
        const int t = 16 * b + r;
        if (t >= nt) continue;
        const int64_t at = (int64_t)(row0 + t0 + t) * p.H + h;
        if (is_norm) {
          if (g == 0) p.nq[at] = o[0];
        } else if (V % 4 == 0) {
          if (c4 < V) *reinterpret_cast<f32x4*>(p.num + at * V + c4) = o;
        } else {
#pragma unroll
          for (int i = 0; i < 4; ++i)
            if (c4 + i < V) p.num[at * V + c4 + i] = o[i];
        }
      }
    }
    lds_barrier();  // the staged chunk has been read
  }
#pragma unroll
  for (int dt = 0; dt < 2 * NK; ++dt)
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int d = 16 * dt + 4 * g + i;
      if (d >= D) continue;
      if (col_on) st[(int64_t)d * V] = S[dt][i];
      else if (is_norm && r == 0) nm[d] = S[dt][i];
    }
}

// LP lanes per (row, head), VEC neighbouring coordinates per lane and step: the head stays in registers between the sum of
// squares and the write
template <typename T, int LP, int VEC, int STEPS>
__global__ __launch_bounds__(256) void memory_out_kernel(MatrixMemoryParams p) {
  const int lane = threadIdx.x % LP;
  const int64_t item = (int64_t)blockIdx.x * (256 / LP) + threadIdx.x / LP;
  if (item >= (int64_t)p.rows * p.H) return;
  const int64_t row = p.row0 + item / p.H;
  const int h = (int)(item % p.H), V = p.V;
  const int64_t at = row * p.H + h;
  const float* o = p.num + at * V;
  const float* gate = p.out_gate + row * p.ldg + h * V;
  const float* w = p.norm_w + h * V;
  float y[STEPS][VEC], gv[STEPS][VEC], wv[STEPS][VEC];
#pragma unroll
  for (int i = 0; i < STEPS; ++i) {
    const int c = (i * LP + lane) * VEC;
    if (c < V) {
      ld_vec<VEC>(o + c, y[i]);
      ld_vec<VEC>(gate + c, gv[i]);
      ld_vec<VEC>(w + c, wv[i]);
    } else {
#pragma unroll
      for (int e = 0; e < VEC; ++e) y[i][e] = 0.0f;
    }
  }
  const float inv_den = 1.0f / (fmaxf(fabsf(p.nq[at]), expf(-p.m[at])) + p.den_eps);
  float ss = 0.f;
#pragma unroll
  for (int i = 0; i < STEPS; ++i)
#pragma unroll
    for (int e = 0; e < VEC; ++e) {
      y[i][e] *= inv_den;
      ss += y[i][e] * y[i][e];
    }
#pragma unroll
  for (int m = LP / 2; m >= 1; m >>= 1) ss += __shfl_xor(ss, m);
  const float inv = 1.0f / sqrtf(ss / (float)V + p.eps) * p.out_scale;
  T* out = reinterpret_cast<T*>(p.out) + row * p.ldo + h * V;
#pragma unroll
  for (int i = 0; i < STEPS; ++i) {
    const int c = (i * LP + lane) * VEC;
    if (c >= V) continue;
#pragma unroll
    for (int e = 0; e < VEC; ++e) out[c + e] = (T)(y[i][e] * inv * wv[i][e] * sigmoid_f(gv[i][e]));
  }
}

template <typename T>
void launch_out(const MatrixMemoryParams& p, hipStream_t st) {
  const long long items = (long long)p.rows * p.H;
  auto blocks = [&](int per) { return dim3((unsigned)((items + per - 1) / per)); };
  const bool vec = p.V % 4 == 0 && p.ldg % 4 == 0 && reinterpret_cast<uintptr_t>(p.out_gate) % 16 == 0 &&
                   reinterpret_cast<uintptr_t>(p.norm_w) % 16 == 0;
  if (vec && p.V <= 128) hipLaunchKernelGGL((memory_out_kernel<T, 32, 4, 1>), blocks(8), dim3(256), 0, st, p);
  else if (vec) hipLaunchKernelGGL((memory_out_kernel<T, 64, 4, 2>), blocks(4), dim3(256), 0, st, p);
  else hipLaunchKernelGGL((memory_out_kernel<T, 64, 1, 8>), blocks(4), dim3(256), 0, st, p);
}

}  // namespace
}  // namespace dsse

extern "C" hipError_t dsse_matrix_memory_walk(const dsse::MatrixMemoryParams* p, hipStream_t st) {
  if (p->nseq <= 0 || p->H <= 0) return hipSuccess;
  if (p->D < 1 || p->V < 1 || p->D > dsse::kWalkThreads || p->V > dsse::kWalkThreads || p->nseq > 65535)
    return hipErrorInvalidValue;
  if (p->V % 4 == 0) {
    if (p->f32) dsse::launch_walk<float, 4>(*p, st);
    else dsse::launch_walk<bf16, 4>(*p, st);
  } else {
    if (p->f32) dsse::launch_walk<float, 1>(*p, st);
    else dsse::launch_walk<bf16, 1>(*p, st);
  }
  return hipGetLastError();
}

extern "C" hipError_t dsse_matrix_memory_chunk(const dsse::MatrixMemoryParams* p, hipStream_t st) {
  if (p->nseq <= 0 || p->H <= 0 || p->rows <= 0) return hipSuccess;
  if (p->f32 || p->D < 1 || p->D > 256 || p->D % 4 || p->V < 1 || p->V > 512 || p->nseq > 65535 || p->H > 65535)
    return hipErrorInvalidValue;
  hipLaunchKernelGGL(dsse::memory_gates_kernel, dim3(p->H, p->nseq), dim3(64 * dsse::kGateWaves), 0, st, *p);
  const int tiles = (p->V + 15) / 16 + 1;
  constexpr int NW = 4;
  const dim3 grid((tiles + NW - 1) / NW, p->H, p->nseq);
  switch ((p->D + 31) / 32) {
#define DSSE_CHUNK_CASE(n) \
  case n:                                                                                                      \
    if (p->vec) hipLaunchKernelGGL((dsse::memory_chunk_kernel<n, NW, true>), grid, dim3(64 * NW), 0, st, *p);  \
    else hipLaunchKernelGGL((dsse::memory_chunk_kernel<n, NW, false>), grid, dim3(64 * NW), 0, st, *p);        \
    break;
    DSSE_CHUNK_CASE(1) DSSE_CHUNK_CASE(2) DSSE_CHUNK_CASE(3) DSSE_CHUNK_CASE(4) DSSE_CHUNK_CASE(5) DSSE_CHUNK_CASE(6)
    DSSE_CHUNK_CASE(7) DSSE_CHUNK_CASE(8)
#undef DSSE_CHUNK_CASE
  }
  dsse::launch_out<bf16>(*p, st);
  return hipGetLastError();
}
