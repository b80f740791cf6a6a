// Causal softmax attention with a sink over paged keys and values of any head width (grouped key/value heads).
//
//   score_j = scale (q . k_j),  j in [max(0, pos - window + 1), pos]
//   out     = sum_j exp(score_j - m) v_j / (sum_j exp(score_j - m) + exp(sink_h - m)),  m = max(max_j score_j, sink_h)
//   out    *= sigmoid(gate[row, h])                                                      (optional)
//
// Options for designs that ask for them: capped scores, score_j = cap * tanh(scale (q . k_j) / cap); and an output
// rotation -- every head's sum is turned back by the query row's own position over the whole value width (rotate-half
// pairs (m, m + V / 2), angles from a (cos, sin) table), before the gate: with values that were rotated by THEIR
// positions when they were cached, a value then enters the output rotated by its distance to the query.
//
// A gate may also have one column per element of the output instead of one per head.  Distance bias and kept keys: an
// entry rel[h][min(pos - j, rel_len - 1)] joins the score (after the scale), and the sequence's first keep_first keys stay
// visible when the window has passed them: the kernels then walk the kept keys first and jump to the window.  The output
// rows may be a column slice of a wider buffer (rows ldo apart) and are multiplied by out_scale before they are rounded.
//
// The sink is a learned logit with no key and no value: it only enlarges the denominator, so a head can attend to
// "nothing".  Scores, the running maximum, the weights and the output sums are fp32 in both element types; queries
// arrive in fp32 (normed and rotated), keys and values are read from their pages in the cache's element type.
//
// Row kernel (any sizes, both element types; every decode step): a workgroup serves `qt` query rows of one head; for each row its four waves split the keys in chunks of
// 64 (one key per lane for the scores, then one output coordinate per lane and 64 broadcast weights for the values),
// keep their own running (max, sum, output) and are merged through LDS.  A decode row and a prompt row take the same
// path, so a position's result does not depend on how the prompt was cut.
#include "api_mixers.h"

namespace dsse {
namespace {

constexpr int kMaxV = 512;
constexpr int kMaxParts = 16;  // stretches a decode walk may be split into
constexpr int kAccs = kMaxV / 64;

// q (LDS, fp32) . key row (global): 16-byte loads when the row width allows
DEV float dot_row(const float* q, const bf16* k, int D) {
  float s = 0.f;
  int d = 0;
  if (D % 8 == 0) {
    for (; d < D; d += 8) {
      const bf16x8 kv = *reinterpret_cast<const bf16x8*>(k + d);
#pragma unroll
      for (int e = 0; e < 8; ++e) s += q[d + e] * (float)kv[e];
    }
  }
  for (; d < D; ++d) s += q[d] * (float)k[d];
  return s;
}
DEV float dot_row(const float* q, const float* k, int D) {
  float s = 0.f;
  int d = 0;
  if (D % 4 == 0) {
    for (; d < D; d += 4) {
      const f32x4 kv = *reinterpret_cast<const f32x4*>(k + d);
#pragma unroll
      for (int e = 0; e < 4; ++e) s += q[d + e] * kv[e];
    }
  }
  for (; d < D; ++d) s += q[d] * k[d];
  return s;
}

template <typename T>
__global__ __launch_bounds__(256) void sink_attention_kernel(SinkAttnParams p) {
  __shared__ float qs[512];
  __shared__ float m_s[4], l_s[4];
  __shared__ float acc_s[4][kMaxV];
  const int work = blockIdx.x, h = blockIdx.y;
  const int seq = p.work_seq[work], tile = p.work_tile[work];
  const int ql = p.q_len[seq];
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int g = h / (p.H / p.G);
  const int D = p.D, V = p.V;
  const int* bt = p.block_tables + (int64_t)seq * p.max_blocks;
  const T* kc = reinterpret_cast<const T*>(p.k);
  const T* vc = reinterpret_cast<const T*>(p.v);
  const float sink = p.sink ? p.sink[h] : -INFINITY;
  for (int i = 0; i < p.qt; ++i) {
    const int off = tile * p.qt + i;
    if (off >= ql) break;  // uniform for the workgroup
    const int row = p.q_start[seq] + off;
    const int pos = p.ctx_len[seq] - ql + off;
    const int lo = pos - p.window + 1 > 0 ? pos - p.window + 1 : 0;
    const int kept = p.keep_first < lo ? p.keep_first : lo;  // keys 0 .. kept - 1 are walked ahead of the window's
    const int nkeys = kept + pos - lo + 1;
    const int last_rel = p.rel_len - 1;
    const float* rel = p.rel ? p.rel + (int64_t)h * p.rel_len : nullptr;
    __syncthreads();  // the previous row's merge has read qs / acc_s
    for (int d = threadIdx.x; d < D; d += blockDim.x) qs[d] = p.q[((int64_t)row * p.H + h) * D + d];
    __syncthreads();
    float m = -INFINITY, l = 0.f;
    float acc[kAccs];
#pragma unroll
    for (int a = 0; a < kAccs; ++a) acc[a] = 0.f;
    for (int c = wave; c * 64 < nkeys; c += 4) {
      const int jj = c * 64 + lane;
      const bool on = jj < nkeys;
      const int j0 = on ? jj : 0;
      const int j = j0 < kept ? j0 : lo + j0 - kept;
      int page = bt[j / kBS];
      page = (unsigned)page < (unsigned)p.num_blocks ? page : 0;
      const int krow = (page * kBS + j % kBS) * p.G + g;
      const float s_dot = dot_row(qs, kc + (int64_t)krow * D, D);
      float s = s_dot * p.scale;
      if (p.softcap > 0.f) s = p.softcap * tanhf(s / p.softcap);
      if (rel) s += rel[pos - j < last_rel ? pos - j : last_rel];
      s = on ? s : -INFINITY;
      const float m_new = fmaxf(m, wave_max(s));  // finite: the chunk holds at least one key
      const float w = on ? expf(s - m_new) : 0.f;
      const float f = expf(m - m_new);            // 0 when m was -inf
      l = l * f + wave_sum(w);
      m = m_new;
#pragma unroll
      for (int a = 0; a < kAccs; ++a) acc[a] *= f;
      const int cnt = nkeys - c * 64 < 64 ? nkeys - c * 64 : 64;
      for (int t = 0; t < cnt; ++t) {
        const float wt = __shfl(w, t);
        const int vrow = __shfl(krow, t);
        const T* vp = vc + (int64_t)vrow * V;
#pragma unroll
        for (int a = 0; a < kAccs; ++a)
          if (a * 64 + lane < V) acc[a] += wt * (float)vp[a * 64 + lane];
      }
    }
    if (lane == 0) {
      m_s[wave] = m;
      l_s[wave] = l;
    }
#pragma unroll
    for (int a = 0; a < kAccs; ++a)
      if (a * 64 + lane < V) acc_s[wave][a * 64 + lane] = acc[a];
    __syncthreads();
    float mm = sink;
    for (int w = 0; w < 4; ++w) mm = fmaxf(mm, m_s[w]);
    float den = p.sink ? expf(sink - mm) : 0.f;
    float fw[4];
    for (int w = 0; w < 4; ++w) {
      fw[w] = m_s[w] == -INFINITY ? 0.f : expf(m_s[w] - mm);
      den += l_s[w] * fw[w];
    }
    const float* gp = p.gate ? p.gate + (int64_t)row * p.ldg + (p.gate_wide ? h * p.V : h) : nullptr;
    const float gate = gp && !p.gate_wide ? 1.0f / (1.0f + expf(-gp[0])) : 1.0f;
    T* out = reinterpret_cast<T*>(p.out) + (int64_t)row * p.ldo + h * V;
    const int half = V >> 1;
    const float2* orp = p.out_rope ? p.out_rope + (int64_t)(pos < p.out_rope_len ? pos : p.out_rope_len - 1) * half : nullptr;
    for (int d = threadIdx.x; d < V; d += blockDim.x) {
      float o = 0.f;
      for (int w = 0; w < 4; ++w) o += acc_s[w][d] * fw[w];
      if (orp) {  // back by the row's position: (a, b) -> (a cos + b sin, b cos - a sin)
        const bool lo_half = d < half;
        const int dp = lo_half ? d + half : d - half;
        float op = 0.f;
        for (int w = 0; w < 4; ++w) op += acc_s[w][dp] * fw[w];
        const float2 c = orp[lo_half ? d : dp];
        o = lo_half ? o * c.x + op * c.y : o * c.x - op * c.y;
      }
      o = o / den * gate;
      if (p.gate_wide) o *= 1.0f / (1.0f + expf(-gp[d]));
      out[d] = (T)(o * p.out_scale);
    }
  }
}

// ---------------------------------------------------------------------------------------------------------------------
// MFMA form for prompt portions (bf16; D % 32 == 0, V % 16 == 0): one wave per (16 query rows, head), 32 keys (one
// page) per step, a workgroup = up to four heads of the same rows (heads of one key/value group read the same pages,
// which then come from the CU's L1).
//
//   S^T[key, row] = K[key, :] . Q[row, :]    A = the page's key rows straight from global memory (16 B per lane),
//                                             B = the 16 rows' query vectors staged in LDS as bf16
//   online softmax per row in fp32 (a row's 32 scores sit in 8 registers of its 4 lanes)
//   O^T[dim, row] += V^T[dim, key] . P^T[key, row]
//                                             A = the TRANSPOSED value page vt[page][G][V][32 keys] (16 B per lane),
//                                             B = the weights exactly as the score accumulators hold them
//
// Which key an (lane group g, element j) pair of the k axis stands for only has to agree between A and B: the scores of
// lane group g are keys 4g..4g+3 of both 16-key halves, so the transposed page stores key k at position
// 8 ((k & 15) >> 2) + 4 (k >> 4) + (k & 3).  The sink enters once, when the row is finished: it only enlarges the
// denominator.
//
// SPLIT (decode steps: few rows, long contexts): the four waves of a workgroup serve the SAME (tile, head) and take
// every fourth page each; their (max, sum, O) are merged through LDS, so a sequence's keys are walked by four waves at
// once and the launch has four times the waves.
// tanh through one exponential: the bf16 form's scores carry bf16 operand rounding, far above this form's error
DEV float tanh_fast(float x) {
  const float c = fminf(fmaxf(x, -15.0f), 15.0f);
  const float e = __expf(2.0f * c);
  return (e - 1.0f) / (e + 1.0f);
}

// The MFMA forms keep scores and running maxima in units of log 2: a weight is then one instruction.
constexpr float kLog2e = 1.4426950408889634f;
DEV float exp2_hw(float x) { return __builtin_amdgcn_exp2f(x); }

// One step of the online softmax over a page: a lane's eight scores (log2 units, -inf: not seen) become weights, the
// MFMA operand pf; new maximum m and sum l; returned: the factor of the sums so far.  No branches: the next page's loads
// stay in flight across it.
DEV float softmax_step(const float (&sv)[8], float& m, float& l, bf16x8& pf) {
  float mx = sv[0];
#pragma unroll
  for (int i = 1; i < 8; ++i) mx = fmaxf(mx, sv[i]);
  const float mn = fmaxf(m, rows4_max(mx));
  const float at = mn == -INFINITY ? 0.0f : mn;  // nothing seen yet: exp2(-inf - 0) is 0
  const float corr = exp2_hw(m - at);
  float ps = 0.f;
#pragma unroll
  for (int i = 0; i < 8; ++i) {
    const float e = exp2_hw(sv[i] - at);
    ps += e;
    pf[i] = (bf16)e;
  }
  l = l * corr + rows4_sum(ps);
  m = mn;
  return corr;
}

// The distance biases of a lane's eight keys of a page: keys 0 .. 3 and 16 .. 19 from its first one, which is n0 away from
// the query.  The branches are uniform: far pages share the last entry, a table that fits its LDS strip needs no memory.
DEV void bias_entries(float (&bv)[8], bool far, float rel_far, const float* strip, const float* table, int strip_len,
                      int rel_len, int n0) {
  if (far) {
#pragma unroll
    for (int i = 0; i < 8; ++i) bv[i] = rel_far;
    return;
  }
  int at[8];
#pragma unroll
  for (int i = 0; i < 8; ++i) {
    const int n = n0 - (i < 4 ? i : 12 + i);
    at[i] = n < 0 ? 0 : (n < rel_len ? n : rel_len - 1);  // negative: a key behind the query, masked by the caller
  }
  if (strip_len >= rel_len) {
#pragma unroll
    for (int i = 0; i < 8; ++i) bv[i] = strip[at[i]];
  } else {
#pragma unroll
    for (int i = 0; i < 8; ++i) bv[i] = at[i] < strip_len ? strip[at[i]] : ld_global<float>(table + at[i]);
  }
}

// NT: V / 16 value tiles.  EXT: the kept first keys and the distance bias (its first rel_lds entries per head in LDS, the
// rest read from memory; pages whose keys are all so far away that they share the last entry look nothing up).
template <int NT, bool SPLIT, bool EXT>
__global__ __launch_bounds__(256) void sink_flash_kernel(SinkAttnParams p, const bf16* __restrict__ vt, int head_tiles,
                                                         int rel_lds) {
  extern __shared__ __align__(16) unsigned char smem_raw[];
  const int D = p.D, V = p.V;
  const int ldq = D + 8;  // bf16 elements per LDS row (16 B of padding)
  const int wave = threadIdx.x >> 6;
  const int h = SPLIT ? blockIdx.y : blockIdx.y * (blockDim.x >> 6) + wave;
  bf16* qs = reinterpret_cast<bf16*>(smem_raw) + wave * 16 * ldq;
  const int lane = threadIdx.x & 63, r = lane & 15, g = lane >> 4;
  const int seq = p.work_seq[blockIdx.x], tile = p.work_tile[blockIdx.x];
  const int ql = p.q_len[seq];
  if (tile * 16 >= ql) return;
  const bool h_ok = h < head_tiles;
  const int hh = h_ok ? h : 0;
  const int kvh = hh / (p.H / p.G);
  const int q0 = p.q_start[seq], pos0 = p.ctx_len[seq] - ql;
  const int c_off = tile * 16 + r;
  const bool c_ok = c_off < ql && h_ok;
  const int c_pos = c_ok ? pos0 + c_off : -1;
  const int64_t c_row = q0 + (c_off < ql ? c_off : 0);
  {
    const float* qa = p.q + (c_row * p.H + hh) * D;
    for (int d = 8 * g; d < D; d += 32) {
      const f32x4 lo4 = c_ok ? *reinterpret_cast<const f32x4*>(qa + d) : f32x4{0.f, 0.f, 0.f, 0.f};
      const f32x4 hi4 = c_ok ? *reinterpret_cast<const f32x4*>(qa + d + 4) : f32x4{0.f, 0.f, 0.f, 0.f};
      bf16x8 v;
#pragma unroll
      for (int j = 0; j < 4; ++j) v[j] = (bf16)lo4[j], v[4 + j] = (bf16)hi4[j];
      *reinterpret_cast<bf16x8*>(qs + r * ldq + d) = v;
    }
  }
  // the heads' bias entries behind the query tiles (SPLIT: one head; otherwise one strip per wave)
  float* rels = reinterpret_cast<float*>(smem_raw + (blockDim.x >> 6) * 16 * ldq * sizeof(bf16));
  const float* relg = nullptr;
  float rel_far = 0.f;
  if (EXT && p.rel) {
    relg = p.rel + (int64_t)hh * p.rel_len;
    rel_far = relg[p.rel_len - 1];
    if (!SPLIT) rels += wave * rel_lds;
    for (int i = SPLIT ? (int)threadIdx.x : lane; i < rel_lds; i += SPLIT ? (int)blockDim.x : 64) rels[i] = relg[i];
  }
  __syncthreads();
  if (!SPLIT && !h_ok) return;
  const int last_off = tile * 16 + 15 < ql ? tile * 16 + 15 : ql - 1;
  const int hi = pos0 + last_off;
  int lo = pos0 + tile * 16 - p.window + 1;
  lo = lo > 0 ? lo : 0;
  const int* bt = p.block_tables + (int64_t)seq * p.max_blocks;
  const bf16* kc = reinterpret_cast<const bf16*>(p.k);
  f32x4 O[NT];
#pragma unroll
  for (int n = 0; n < NT; ++n) O[n] = f32x4{0.f, 0.f, 0.f, 0.f};
  float m = -INFINITY, l = 0.f;
  // scores in log2 units; a cap acts on the plain ones
  const float cap_inv = p.softcap > 0.f ? 1.0f / p.softcap : 0.f, cap2 = p.softcap * kLog2e;
  const float scale2 = p.softcap > 0.f ? p.scale : p.scale * kLog2e;
  const int nks = D / 32;
  const int pg_lo = lo / kBS;
  int kept_pages = 0;  // whole pages of kept keys before the window's first page
  if (EXT && p.keep_first > 0) {
    kept_pages = (p.keep_first + kBS - 1) / kBS;
    kept_pages = kept_pages < pg_lo ? kept_pages : pg_lo;
  }
  const int walk = kept_pages + hi / kBS - pg_lo + 1;
  // Loads run a page ahead: the ids of the wave's next 64 pages come in one load, a page's keys (the first four k-steps)
  // and -- for values up to 128 wide -- its values are requested while the page before it is in the softmax.
  constexpr int KB = 4, STEP = SPLIT ? 4 : 1;
  constexpr bool AHEAD_V = NT <= 8;
  const int first = SPLIT ? wave : 0;
  const int mine = walk > first ? (walk - first + STEP - 1) / STEP : 0;
  auto page_at = [&](int it) {
    const int pi = first + it * STEP;
    return pi < kept_pages ? pi : pg_lo + pi - kept_pages;
  };
  auto ids_from = [&](int it0) {
    const int b = it0 + lane < mine ? bt[page_at(it0 + lane)] : 0;
    return (unsigned)b < (unsigned)p.num_blocks ? b : 0;
  };
  auto key_row = [&](int blk) { return kc + (((int64_t)blk * kBS + r) * p.G + kvh) * D + 8 * g; };  // key r, then 16 + r
  bf16x8 ka[KB], kb[KB], vf[NT];
  auto load_keys = [&](int blk) {
    const bf16* k0 = key_row(blk);
    const bf16* k1 = k0 + (int64_t)16 * p.G * D;
#pragma unroll
    for (int u = 0; u < KB; ++u)
      if (u < nks) {
        ka[u] = ld_global<bf16x8>(k0 + 32 * u);
        kb[u] = ld_global<bf16x8>(k1 + 32 * u);
      }
  };
  auto load_values = [&](int blk, bf16x8(&v)[NT]) {
    const bf16* vrow = vt + (((int64_t)blk * p.G + kvh) * V + r) * kBS + 8 * g;   // dim r of value tile 0
#pragma unroll
    for (int n = 0; n < NT; ++n) v[n] = ld_global<bf16x8>(vrow + (int64_t)n * 16 * kBS);
  };
  int blks = ids_from(0);
  if (mine > 0) {
    load_keys(__builtin_amdgcn_readlane(blks, 0));
    if (AHEAD_V) load_values(__builtin_amdgcn_readlane(blks, 0), vf);
  }
  for (int it = 0; it < mine; ++it) {
    const int pg = page_at(it);
    const int blk = __builtin_amdgcn_readlane(blks, it & 63);
    if (!AHEAD_V) load_values(blk, vf);
    f32x4 s0 = f32x4{0.f, 0.f, 0.f, 0.f}, s1 = s0;
#pragma unroll
    for (int u = 0; u < KB; ++u)
      if (u < nks) {
        const bf16x8 q8 = *reinterpret_cast<const bf16x8*>(qs + r * ldq + 32 * u + 8 * g);
        s0 = mfma16x16x32(ka[u], q8, s0);
        s1 = mfma16x16x32(kb[u], q8, s1);
      }
    for (int sb = KB; sb < nks; sb += 4) {  // wider heads: four k-steps at a time
      const bf16* k0 = key_row(blk);
      const bf16* k1 = k0 + (int64_t)16 * p.G * D;
      bf16x8 wa[4], wb[4];
#pragma unroll
      for (int u = 0; u < 4; ++u) {
        const int s = sb + u < nks ? sb + u : nks - 1;
        wa[u] = ld_global<bf16x8>(k0 + 32 * s);
        wb[u] = ld_global<bf16x8>(k1 + 32 * s);
      }
#pragma unroll
      for (int u = 0; u < 4; ++u)
        if (sb + u < nks) {
          const bf16x8 q8 = *reinterpret_cast<const bf16x8*>(qs + r * ldq + 32 * (sb + u) + 8 * g);
          s0 = mfma16x16x32(wa[u], q8, s0);
          s1 = mfma16x16x32(wb[u], q8, s1);
        }
    }
    bf16x8 vn[AHEAD_V ? NT : 1];
    if (it + 1 < mine) {
      if (((it + 1) & 63) == 0) blks = ids_from(it + 1);
      const int nb = __builtin_amdgcn_readlane(blks, (it + 1) & 63);
      load_keys(nb);
      if constexpr (AHEAD_V) load_values(nb, vn);
    }
    float sv[8];
    // uniform: every (row, key) pair of this tile and page is at least rel_len - 1 apart
    const bool far = EXT && p.rel && pos0 + tile * 16 - (pg * kBS + kBS - 1) >= p.rel_len - 1;
    float bv[8];
    if (EXT && p.rel) bias_entries(bv, far, rel_far, rels, relg, rel_lds, p.rel_len, c_pos - pg * kBS - 4 * g);
#pragma unroll
    for (int i = 0; i < 8; ++i) {
      const int key = pg * kBS + (i < 4 ? 4 * g + i : 16 + 4 * g + (i - 4));
      const bool seen = c_ok && key <= c_pos && (c_pos - key < p.window || (EXT && key < p.keep_first));
      float sc = (i < 4 ? s0[i] : s1[i - 4]) * scale2;
      if (p.softcap > 0.f) sc = cap2 * tanh_fast(sc * cap_inv);
      if (EXT && p.rel) sc += bv[i] * kLog2e;
      sv[i] = seen ? sc : -INFINITY;
    }
    bf16x8 pf;
    const float corr = softmax_step(sv, m, l, pf);
#pragma unroll
    for (int n = 0; n < NT; ++n) {
      f32x4 o = O[n];
#pragma unroll
      for (int i = 0; i < 4; ++i) o[i] *= corr;
      O[n] = mfma16x16x32(vf[n], pf, o);
    }
    if constexpr (AHEAD_V) {
#pragma unroll
      for (int n = 0; n < NT; ++n) vf[n] = vn[n];
    }
  }
  if (SPLIT) {
    // merge the four waves' partial results: [wave][16 columns][V + 2] floats, after every wave has read its queries
    float* mg = reinterpret_cast<float*>(smem_raw) + 4 * 16 * ((ldq + 1) / 2) + rel_lds;
    const int ldm = V + 2;
    float* mine = mg + (wave * 16 + r) * ldm;
#pragma unroll
    for (int n = 0; n < NT; ++n)
#pragma unroll
      for (int i = 0; i < 4; ++i) mine[16 * n + 4 * g + i] = O[n][i];
    if (g == 0) {
      mine[V] = m;
      mine[V + 1] = l;
    }
    __syncthreads();
    const int rows_on = ql - tile * 16 < 16 ? ql - tile * 16 : 16;
    for (int idx = threadIdx.x; idx < rows_on * V; idx += blockDim.x) {
      const int col = idx / V, d = idx - col * V;
      const int64_t row = q0 + tile * 16 + col;
      const float sk = p.sink ? p.sink[h] * kLog2e : -INFINITY;
      float mm = sk;
      for (int w = 0; w < 4; ++w) mm = fmaxf(mm, mg[(w * 16 + col) * ldm + V]);
      float den = p.sink ? exp2_hw(sk - mm) : 0.f, num = 0.f, nump = 0.f;
      const int half = V >> 1;
      const bool lo_half = d < half;
      const int dp = lo_half ? d + half : d - half;
      for (int w = 0; w < 4; ++w) {
        const float* src = mg + (w * 16 + col) * ldm;
        const float f = src[V] == -INFINITY ? 0.f : exp2_hw(src[V] - mm);
        den += src[V + 1] * f;
        num += src[d] * f;
        nump += src[dp] * f;
      }
      if (p.out_rope) {  // back by the row's position
        const int ps = pos0 + tile * 16 + col;
        const float2 c = p.out_rope[(int64_t)(ps < p.out_rope_len ? ps : p.out_rope_len - 1) * half + (lo_half ? d : dp)];
        num = lo_half ? num * c.x + nump * c.y : num * c.x - nump * c.y;
      }
      float o = den > 0.f ? num / den : 0.f;
      if (p.gate) o *= 1.0f / (1.0f + expf(-p.gate[row * p.ldg + (p.gate_wide ? h * V + d : h)]));
      reinterpret_cast<bf16*>(p.out)[row * p.ldo + h * V + d] = (bf16)(o * p.out_scale);
    }
    return;
  }
  if (c_ok) {
    float den = l, f = 1.0f;
    if (p.sink) {  // the sink joins the denominator under the common maximum
      const float sk = p.sink[h] * kLog2e;
      const float mm = fmaxf(m, sk);
      f = exp2_hw(m - mm);
      den = l * f + exp2_hw(sk - mm);
    }
    float inv = den > 0.f ? f / den * p.out_scale : 0.0f;
    if (p.gate && !p.gate_wide) inv *= 1.0f / (1.0f + expf(-p.gate[c_row * p.ldg + h]));
    if (p.out_rope) {  // NT is even (the host checks V % 32 == 0): dimension m = 16 n + 4 g + i pairs with tile n + NT / 2
      const float2* orp = p.out_rope + (int64_t)(c_pos < p.out_rope_len ? c_pos : p.out_rope_len - 1) * (V >> 1);
#pragma unroll
      for (int n = 0; n < NT / 2; ++n)
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          const float2 c = orp[16 * n + 4 * g + i];
          const float a = O[n][i], b = O[n + NT / 2][i];
          O[n][i] = a * c.x + b * c.y;
          O[n + NT / 2][i] = b * c.x - a * c.y;
        }
    }
    bf16* out = reinterpret_cast<bf16*>(p.out) + c_row * p.ldo + h * V;
    const float* gw = p.gate_wide ? p.gate + c_row * p.ldg + h * V + 4 * g : nullptr;
#pragma unroll
    for (int n = 0; n < NT; ++n) {
      bf16x4 v;
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        float o = O[n][i] * inv;
        if (gw) o *= 1.0f / (1.0f + expf(-gw[16 * n + i]));
        v[i] = (bf16)o;
      }
      *reinterpret_cast<bf16x4*>(out + 16 * n + 4 * g) = v;
    }
  }
}

// ---------------------------------------------------------------------------------------------------------------------
// Shared-page form for prompt portions (bf16, head widths up to 128): a workgroup takes hb heads of ONE key/value group times
// rt tiles of 16 query rows, hb rt = 8 column tiles, two per wave.  Each page's keys and transposed values are staged in LDS
// once for all eight tiles, and a fragment read from LDS feeds both tiles of a wave; the next two pages are on their way
// (in registers) while the current one is in the MFMAs, one barrier per page.  The query operands stay in registers.  Masks and
// the rescaling of the sums are branches here: pages that every row sees whole and maxima that stay skip them.  The head
// group is the fast grid dimension, so workgroups of one XCD keep to the same keys when the groups are a multiple of eight.
constexpr int kTileWidth = 128;   // widest query and value heads
constexpr int kTileLdv = kBS + 8;

template <int NT>
__global__ __launch_bounds__(256, 2) void sink_tile_kernel(SinkAttnParams p, const bf16* __restrict__ vt, int hb, int rt) {
  extern __shared__ __align__(16) unsigned char smem_raw[];
  constexpr int V = 16 * NT, KS = kTileWidth / 32, KC = kTileWidth * kBS / 8 / 256, VC = (V * kBS / 8 + 255) / 256;
  const int D = p.D, nks = D / 32, ldk = D + 8;
  const int buf_elems = kBS * ldk + V * kTileLdv;
  bf16* smem = reinterpret_cast<bf16*>(smem_raw);
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, r = lane & 15, g = lane >> 4;
  const int seq = p.work_seq[blockIdx.y], tile = p.work_tile[blockIdx.y];
  const int ql = p.q_len[seq], row_first = tile * 16 * rt;
  if (row_first >= ql) return;  // uniform for the workgroup
  const int h_first = blockIdx.x * hb, kvh = h_first / (p.H / p.G);
  const int q0 = p.q_start[seq], pos0 = p.ctx_len[seq] - ql;
  const int row_last = row_first + 16 * rt < ql ? row_first + 16 * rt - 1 : ql - 1;
  const int hi = pos0 + row_last;
  int lo = pos0 + row_first - p.window + 1;
  lo = lo > 0 ? lo : 0;
  const int pg_lo = lo / kBS;
  int kept_pages = 0;
  if (p.keep_first > 0) {
    kept_pages = (p.keep_first + kBS - 1) / kBS;
    kept_pages = kept_pages < pg_lo ? kept_pages : pg_lo;
  }
  const int walk = kept_pages + hi / kBS - pg_lo + 1;
  const int* bt = p.block_tables + (int64_t)seq * p.max_blocks;
  auto page_at = [&](int it) { return it < kept_pages ? it : pg_lo + it - kept_pages; };
  auto ids_from = [&](int it0) {
    const int b = it0 + lane < walk ? bt[page_at(it0 + lane)] : 0;
    return (unsigned)b < (unsigned)p.num_blocks ? b : 0;
  };
  // this wave's two column tiles
  int head[2], pos[2], tile_lo[2], tile_hi[2];
  bool on[2];
  int64_t row[2];
  bf16x8 qf[2][KS];
#pragma unroll
  for (int c = 0; c < 2; ++c) {
    const int ct = 2 * wave + c, off = row_first + 16 * (ct % rt) + r;
    head[c] = h_first + ct / rt;
    on[c] = off < ql;
    row[c] = q0 + (on[c] ? off : 0);
    pos[c] = on[c] ? pos0 + off : -1;
    tile_lo[c] = pos0 + row_first + 16 * (ct % rt);
    tile_hi[c] = tile_lo[c] + 15 < hi ? tile_lo[c] + 15 : hi;
    const float* q = p.q + (row[c] * p.H + head[c]) * D + 8 * g;
#pragma unroll
    for (int u = 0; u < KS; ++u) {
      qf[c][u] = zero_bf16x8();
      if (u < nks && on[c]) {
        const f32x4 a = ld_global<f32x4>(q + 32 * u), b = ld_global<f32x4>(q + 32 * u + 4);
#pragma unroll
        for (int j = 0; j < 4; ++j) qf[c][u][j] = (bf16)a[j], qf[c][u][4 + j] = (bf16)b[j];
      }
    }
  }
  int blks = ids_from(0);
  // staging: 16-byte pieces of the page's keys (rows G D apart) and of its transposed values (contiguous)
  const bf16* kc = reinterpret_cast<const bf16*>(p.k);
  const int k16 = D / 8;
  bf16x8 nk[2][KC], nv[2][VC];  // two pages on their way
  int koff[KC], kdst[KC], vdst[VC];
#pragma unroll
  for (int i = 0; i < KC; ++i) {
    const int idx = tid + 256 * i, kr = idx / k16, c = idx - kr * k16;
    const bool in = kr < kBS;
    koff[i] = in ? kr * p.G * D + 8 * c : 0;
    kdst[i] = in ? kr * ldk + 8 * c : -1;
  }
#pragma unroll
  for (int i = 0; i < VC; ++i) {
    const int idx = tid + 256 * i;
    vdst[i] = idx < V * kBS / 8 ? kBS * ldk + (idx / (kBS / 8)) * kTileLdv + 8 * (idx % (kBS / 8)) : -1;
  }
  auto request = [&](int it, bf16x8(&rk)[KC], bf16x8(&rv)[VC]) {  // pages past the walk read its last one again
    if (it < walk && (it & 63) == 0 && it > 0) blks = ids_from(it);
    const int blk = __builtin_amdgcn_readlane(blks, it < walk ? it & 63 : (walk - 1) & 63);
    const bf16* kp = kc + ((int64_t)blk * kBS * p.G + kvh) * D;
    const bf16* vp = vt + ((int64_t)blk * p.G + kvh) * V * kBS;
#pragma unroll
    for (int i = 0; i < KC; ++i) rk[i] = ld_global<bf16x8>(kp + koff[i]);
#pragma unroll
    for (int i = 0; i < VC; ++i) rv[i] = ld_global<bf16x8>(vp + (vdst[i] >= 0 ? 8 * (tid + 256 * i) : 0));
  };
  auto stash = [&](int buf, const bf16x8(&rk)[KC], const bf16x8(&rv)[VC]) {
    bf16* b = smem + buf * buf_elems;
#pragma unroll
    for (int i = 0; i < KC; ++i)
      if (kdst[i] >= 0) *reinterpret_cast<bf16x8*>(b + kdst[i]) = rk[i];
#pragma unroll
    for (int i = 0; i < VC; ++i)
      if (vdst[i] >= 0) *reinterpret_cast<bf16x8*>(b + vdst[i]) = rv[i];
  };
  f32x4 O[2][NT];
#pragma unroll
  for (int c = 0; c < 2; ++c)
#pragma unroll
    for (int n = 0; n < NT; ++n) O[c][n] = f32x4{0.f, 0.f, 0.f, 0.f};
  float m[2] = {-INFINITY, -INFINITY}, l[2] = {0.f, 0.f};
  const float cap_inv = p.softcap > 0.f ? 1.0f / p.softcap : 0.f, cap2 = p.softcap * kLog2e;
  const float scale2 = p.softcap > 0.f ? p.scale : p.scale * kLog2e;
  const int wave_lo = tile_lo[0] < tile_lo[1] ? tile_lo[0] : tile_lo[1], wave_hi = tile_hi[0] > tile_hi[1] ? tile_hi[0] : tile_hi[1];
  auto page_step = [&](int it, bf16x8(&rk)[KC], bf16x8(&rv)[VC], const bf16x8(&tk)[KC], const bf16x8(&tv)[VC]) {
    const int pg = page_at(it);
    request(it + 2, rk, rv);
    if (pg * kBS <= wave_hi) {  // uniform for the wave: some row of it may see this page
      const bf16* kb = smem + (it & 1) * buf_elems;
      const bf16* vb = kb + kBS * ldk;
      f32x4 s0[2], s1[2];
#pragma unroll
      for (int c = 0; c < 2; ++c) s0[c] = s1[c] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int u = 0; u < KS; ++u)
        if (u < nks) {
          const bf16x8 k0 = *reinterpret_cast<const bf16x8*>(kb + r * ldk + 32 * u + 8 * g);
          const bf16x8 k1 = *reinterpret_cast<const bf16x8*>(kb + (16 + r) * ldk + 32 * u + 8 * g);
#pragma unroll
          for (int c = 0; c < 2; ++c) {
            s0[c] = mfma16x16x32(k0, qf[c][u], s0[c]);
            s1[c] = mfma16x16x32(k1, qf[c][u], s1[c]);
          }
        }
      // uniform: every key of the page is at or before the wave's first row and inside the window of its last one
      const bool full = pg * kBS + kBS - 1 <= wave_lo && wave_hi - pg * kBS < p.window;
      bf16x8 pf[2];
      float corr[2];
#pragma unroll
      for (int c = 0; c < 2; ++c) {
        float sv[8];
#pragma unroll
        for (int i = 0; i < 8; ++i) {
          float sc = (i < 4 ? s0[c][i] : s1[c][i - 4]) * scale2;
          if (p.softcap > 0.f) sc = cap2 * tanh_fast(sc * cap_inv);
          sv[i] = sc;
        }
        if (!full) {
#pragma unroll
          for (int i = 0; i < 8; ++i) {
            const int key = pg * kBS + (i < 4 ? 4 * g + i : 16 + 4 * g + (i - 4));
            const bool seen = key <= pos[c] && (pos[c] - key < p.window || key < p.keep_first);
            sv[i] = seen ? sv[i] : -INFINITY;
          }
        }
        corr[c] = softmax_step(sv, m[c], l[c], pf[c]);
      }
      if (!__all(corr[0] == 1.0f && corr[1] == 1.0f)) {
#pragma unroll
        for (int n = 0; n < NT; ++n)
#pragma unroll
          for (int i = 0; i < 4; ++i) O[0][n][i] *= corr[0], O[1][n][i] *= corr[1];
      }
#pragma unroll
      for (int n = 0; n < NT; ++n) {
        const bf16x8 v = *reinterpret_cast<const bf16x8*>(vb + (16 * n + r) * kTileLdv + 8 * g);
#pragma unroll
        for (int c = 0; c < 2; ++c) O[c][n] = mfma16x16x32(v, pf[c], O[c][n]);
      }
    }
    stash((it + 1) & 1, tk, tv);  // page it + 1; that buffer was last read before the previous barrier
    lds_barrier();
  };
  request(0, nk[0], nv[0]);
  request(1, nk[1], nv[1]);
  stash(0, nk[0], nv[0]);
  lds_barrier();
  for (int it = 0; it < walk; it += 2) {
    page_step(it, nk[0], nv[0], nk[1], nv[1]);
    if (it + 1 < walk) page_step(it + 1, nk[1], nv[1], nk[0], nv[0]);  // uniform for the workgroup
  }
#pragma unroll
  for (int c = 0; c < 2; ++c) {
    if (!on[c]) continue;
    const int h = head[c];
    float den = l[c], f = 1.0f;
    if (p.sink) {
      const float sk = p.sink[h] * kLog2e, mm = fmaxf(m[c], sk);
      f = exp2_hw(m[c] - mm);
      den = l[c] * f + exp2_hw(sk - mm);
    }
    float inv = den > 0.f ? f / den * p.out_scale : 0.0f;
    if (p.gate && !p.gate_wide) inv *= 1.0f / (1.0f + expf(-p.gate[row[c] * p.ldg + h]));
    bf16* out = reinterpret_cast<bf16*>(p.out) + row[c] * p.ldo + h * V + 4 * g;
    const float* gw = p.gate_wide ? p.gate + row[c] * p.ldg + h * V + 4 * g : nullptr;
#pragma unroll
    for (int n = 0; n < NT; ++n) {
      bf16x4 v;
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        float o = O[c][n][i] * inv;
        if (gw) o *= 1.0f / (1.0f + expf(-gw[16 * n + i]));
        v[i] = (bf16)o;
      }
      *reinterpret_cast<bf16x4*>(out + 16 * n) = v;
    }
  }
}

// ---------------------------------------------------------------------------------------------------------------------
// Decode form of the MFMA kernel: one query row per work item, and the heads of ONE key/value group side by side as the
// 16 columns, so a page of keys and values is read once per group instead of once per head.  The NW waves of a workgroup
// split the pages (wave, wave + NW, ...) and are merged through LDS.  A decode step has few workgroups and short walks,
// so the walk is written against latency: a wave reads the ids of its next 64 pages in one load, requests the next
// page's keys before it needs them (heads up to 128 wide: KB k-steps of both 16-key halves stay in registers), and the
// values of a page while its scores are being made.  Same key order, masks, bias and epilogue as above.  Few sequences
// with long walks: nparts workgroups per (item, group) take a stretch of the walk each, leave sum, maximum and weights in
// `part`, and a second kernel joins the stretches.
template <int NT, int KB, int NW, bool EXT>
__global__ __launch_bounds__(NW * 64) void sink_decode_kernel(SinkAttnParams p, const bf16* __restrict__ vt, int rel_lds) {
  extern __shared__ __align__(16) unsigned char smem_raw[];
  const int D = p.D, V = p.V;
  const int ldq = D + 8;
  const int rep = p.H / p.G;
  const int kvh = blockIdx.y;
  const int parts = p.nparts > 1 ? p.nparts : 1, ctile = (int)blockIdx.z / parts, part = (int)blockIdx.z - ctile * parts;
  const int h0 = kvh * rep + ctile * 16;                            // first head of this column tile
  const int cols = rep - ctile * 16 < 16 ? rep - ctile * 16 : 16;
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, r = lane & 15, g = lane >> 4;
  const int seq = p.work_seq[blockIdx.x], off = p.work_tile[blockIdx.x];
  const int ql = p.q_len[seq];
  if (off >= ql) return;  // uniform for the workgroup
  const int64_t row = p.q_start[seq] + off;
  const int pos = p.ctx_len[seq] - ql + off;
  int lo = pos - p.window + 1;
  lo = lo > 0 ? lo : 0;
  const int pg_lo = lo / kBS;
  int kept_pages = 0;
  if (EXT && p.keep_first > 0) {
    kept_pages = (p.keep_first + kBS - 1) / kBS;
    kept_pages = kept_pages < pg_lo ? kept_pages : pg_lo;
  }
  const int walk = kept_pages + pos / kBS - pg_lo + 1;
  const int per = (walk + parts - 1) / parts, start = part * per;   // this partition's stretch of the walk
  const int stretch = walk - start < per ? walk - start : per;
  const int mine = stretch > wave ? (stretch - wave + NW - 1) / NW : 0;   // pages of this wave
  const int* bt = p.block_tables + (int64_t)seq * p.max_blocks;
  auto page_at = [&](int it) {  // logical page of this wave's it-th step
    const int pi = start + wave + it * NW;
    return pi < kept_pages ? pi : pg_lo + pi - kept_pages;
  };
  auto ids_from = [&](int it0) {  // the physical pages of this wave's steps it0 .. it0 + 63, one per lane
    int b = it0 + lane < mine ? bt[page_at(it0 + lane)] : 0;
    return (unsigned)b < (unsigned)p.num_blocks ? b : 0;
  };
  int blks = ids_from(0);
  bf16* qs = reinterpret_cast<bf16*>(smem_raw);
  float* rels = reinterpret_cast<float*>(smem_raw + 16 * ldq * sizeof(bf16));   // [cols][rel_lds]
  float* mg = rels + cols * rel_lds;                                            // [NW][cols][V + 2]
  for (int i = threadIdx.x; i < 16 * (D / 4); i += NW * 64) {
    const int col = i / (D / 4), d = (i - col * (D / 4)) * 4;
    const f32x4 q4 = col < cols ? *reinterpret_cast<const f32x4*>(p.q + (row * p.H + h0 + col) * D + d)
                                : f32x4{0.f, 0.f, 0.f, 0.f};
    bf16x4 v;
#pragma unroll
    for (int j = 0; j < 4; ++j) v[j] = (bf16)q4[j];
    *reinterpret_cast<bf16x4*>(qs + col * ldq + d) = v;
  }
  const bool c_ok = r < cols;
  const float* relg = nullptr;
  float rel_far = 0.f;
  if (EXT && p.rel) {
    for (int i = threadIdx.x; i < cols * rel_lds; i += NW * 64) {
      const int col = i / rel_lds;
      rels[i] = p.rel[(int64_t)(h0 + col) * p.rel_len + i - col * rel_lds];
    }
    relg = p.rel + (int64_t)(h0 + (c_ok ? r : 0)) * p.rel_len;
    rel_far = relg[p.rel_len - 1];
  }
  const float* relc = rels + (c_ok ? r : 0) * rel_lds;
  const bf16* kc = reinterpret_cast<const bf16*>(p.k);
  const int nks = D / 32;
  auto key_row = [&](int blk) { return kc + (((int64_t)blk * kBS + r) * p.G + kvh) * D + 8 * g; };
  bf16x8 ka[KB], kb[KB];  // the current page's keys (k-steps 0 .. KB - 1)
  auto load_keys = [&](int blk) {
    const bf16* k0 = key_row(blk);
    const bf16* k1 = k0 + (int64_t)16 * p.G * D;
#pragma unroll
    for (int u = 0; u < KB; ++u)
      if (u < nks) {
        ka[u] = ld_global<bf16x8>(k0 + 32 * u);
        kb[u] = ld_global<bf16x8>(k1 + 32 * u);
      }
  };
  f32x4 O[NT];
#pragma unroll
  for (int n = 0; n < NT; ++n) O[n] = f32x4{0.f, 0.f, 0.f, 0.f};
  float m = -INFINITY, l = 0.f;
  // scores in log2 units; a cap acts on the plain ones
  const float cap_inv = p.softcap > 0.f ? 1.0f / p.softcap : 0.f, cap2 = p.softcap * kLog2e;
  const float scale2 = p.softcap > 0.f ? p.scale : p.scale * kLog2e;
  if (mine > 0) load_keys(__builtin_amdgcn_readlane(blks, 0));
  __syncthreads();
  for (int it = 0; it < mine; ++it) {
    const int pg = page_at(it);
    const int blk = __builtin_amdgcn_readlane(blks, it & 63);
    const bf16* vrow = vt + (((int64_t)blk * p.G + kvh) * V + r) * kBS + 8 * g;
    bf16x8 vf[NT];
#pragma unroll
    for (int n = 0; n < NT; ++n) vf[n] = ld_global<bf16x8>(vrow + (int64_t)n * 16 * kBS);
    f32x4 s0 = f32x4{0.f, 0.f, 0.f, 0.f}, s1 = s0;
#pragma unroll
    for (int u = 0; u < KB; ++u)
      if (u < nks) {
        const bf16x8 q8 = *reinterpret_cast<const bf16x8*>(qs + r * ldq + 32 * u + 8 * g);
        s0 = mfma16x16x32(ka[u], q8, s0);
        s1 = mfma16x16x32(kb[u], q8, s1);
      }
    if (nks > KB) {  // wider heads: the rest of the row, no prefetch
      const bf16* k0 = key_row(blk);
      const bf16* k1 = k0 + (int64_t)16 * p.G * D;
      for (int s = KB; s < nks; ++s) {
        const bf16x8 q8 = *reinterpret_cast<const bf16x8*>(qs + r * ldq + 32 * s + 8 * g);
        s0 = mfma16x16x32(ld_global<bf16x8>(k0 + 32 * s), q8, s0);
        s1 = mfma16x16x32(ld_global<bf16x8>(k1 + 32 * s), q8, s1);
      }
    }
    if (it + 1 < mine) {
      if (((it + 1) & 63) == 0) blks = ids_from(it + 1);
      load_keys(__builtin_amdgcn_readlane(blks, (it + 1) & 63));
    }
    float sv[8];
    const bool far = EXT && p.rel && pos - (pg * kBS + kBS - 1) >= p.rel_len - 1;
    float bv[8];
    if (EXT && p.rel) bias_entries(bv, far, rel_far, relc, relg, rel_lds, p.rel_len, pos - pg * kBS - 4 * g);
#pragma unroll
    for (int i = 0; i < 8; ++i) {
      const int key = pg * kBS + (i < 4 ? 4 * g + i : 16 + 4 * g + (i - 4));
      const bool seen = c_ok && key <= pos && (pos - key < p.window || (EXT && key < p.keep_first));
      float sc = (i < 4 ? s0[i] : s1[i - 4]) * scale2;
      if (p.softcap > 0.f) sc = cap2 * tanh_fast(sc * cap_inv);
      if (EXT && p.rel) sc += bv[i] * kLog2e;
      sv[i] = seen ? sc : -INFINITY;
    }
    bf16x8 pf;
    const float corr = softmax_step(sv, m, l, pf);
#pragma unroll
    for (int n = 0; n < NT; ++n) {
      f32x4 o = O[n];
#pragma unroll
      for (int i = 0; i < 4; ++i) o[i] *= corr;
      O[n] = mfma16x16x32(vf[n], pf, o);
    }
  }
  const int ldm = V + 2;
  if (c_ok) {
    float* my = mg + (wave * cols + r) * ldm;
#pragma unroll
    for (int n = 0; n < NT; ++n)
#pragma unroll
      for (int i = 0; i < 4; ++i) my[16 * n + 4 * g + i] = O[n][i];
    if (g == 0) {
      my[V] = m;
      my[V + 1] = l;
    }
  }
  __syncthreads();
  const int half = V >> 1;
  const float2* orp = p.out_rope ? p.out_rope + (int64_t)(pos < p.out_rope_len ? pos : p.out_rope_len - 1) * half : nullptr;
  for (int idx = threadIdx.x; idx < cols * V; idx += NW * 64) {
    const int col = idx / V, d = idx - col * V, h = h0 + col;
    const float sk = p.sink && parts == 1 ? p.sink[h] * kLog2e : -INFINITY;
    float mm = sk;
#pragma unroll
    for (int w = 0; w < NW; ++w) mm = fmaxf(mm, mg[(w * cols + col) * ldm + V]);
    float den = sk > -INFINITY ? exp2_hw(sk - mm) : 0.f, num = 0.f, nump = 0.f;
    const bool lo_half = d < half;
    const int dp = orp ? (lo_half ? d + half : d - half) : d;
#pragma unroll
    for (int w = 0; w < NW; ++w) {
      const float* src = mg + (w * cols + col) * ldm;
      const float f = src[V] == -INFINITY ? 0.f : exp2_hw(src[V] - mm);
      den += src[V + 1] * f;
      num += src[d] * f;
      nump += src[dp] * f;
    }
    if (parts > 1) {  // the combine kernel finishes: the stretch's sum, its maximum and its weights
      float* dst = p.part + (((int64_t)blockIdx.x * p.H + h) * parts + part) * ldm;
      dst[d] = num;
      if (d == 0) {
        dst[V] = mm;
        dst[V + 1] = den;
      }
      continue;
    }
    if (orp) {  // back by the row's position
      const float2 cs = orp[lo_half ? d : dp];
      num = lo_half ? num * cs.x + nump * cs.y : num * cs.x - nump * cs.y;
    }
    float o = den > 0.f ? num / den : 0.f;
    if (p.gate) o *= 1.0f / (1.0f + expf(-p.gate[row * p.ldg + (p.gate_wide ? h * V + d : h)]));
    reinterpret_cast<bf16*>(p.out)[row * p.ldo + h * V + d] = (bf16)(o * p.out_scale);
  }
}

// The stretches of a split decode walk joined: one wave per (work item, head).
__global__ __launch_bounds__(256) void sink_combine_kernel(SinkAttnParams p, int num_work) {
  const int lane = threadIdx.x & 63;
  const int item = blockIdx.x * 4 + (threadIdx.x >> 6);
  if (item >= num_work * p.H) return;
  const int work = item / p.H, h = item - work * p.H, V = p.V, ldm = V + 2;
  const int seq = p.work_seq[work], off = p.work_tile[work], ql = p.q_len[seq];
  if (off >= ql) return;
  const int64_t row = p.q_start[seq] + off;
  const int pos = p.ctx_len[seq] - ql + off;
  const float* src = p.part + (int64_t)item * p.nparts * ldm;
  const float sk = p.sink ? p.sink[h] * kLog2e : -INFINITY;
  float mm = sk;
  for (int i = 0; i < p.nparts; ++i) mm = fmaxf(mm, src[i * ldm + V]);
  float den = p.sink ? exp2_hw(sk - mm) : 0.f;
  float f[kMaxParts];
#pragma unroll
  for (int i = 0; i < kMaxParts; ++i) {
    f[i] = 0.f;
    if (i < p.nparts && src[i * ldm + V] > -INFINITY) {
      f[i] = exp2_hw(src[i * ldm + V] - mm);
      den += src[i * ldm + V + 1] * f[i];
    }
  }
  const int half = V >> 1;
  const float2* orp = p.out_rope ? p.out_rope + (int64_t)(pos < p.out_rope_len ? pos : p.out_rope_len - 1) * half : nullptr;
  for (int d = lane; d < V; d += 64) {
    const bool lo_half = d < half;
    const int dp = orp ? (lo_half ? d + half : d - half) : d;
    float num = 0.f, nump = 0.f;
#pragma unroll
    for (int i = 0; i < kMaxParts; ++i)
      if (i < p.nparts) {
        num += src[i * ldm + d] * f[i];
        nump += src[i * ldm + dp] * f[i];
      }
    if (orp) {
      const float2 cs = orp[lo_half ? d : dp];
      num = lo_half ? num * cs.x + nump * cs.y : num * cs.x - nump * cs.y;
    }
    float o = den > 0.f ? num / den : 0.f;
    if (p.gate) o *= 1.0f / (1.0f + expf(-p.gate[row * p.ldg + (p.gate_wide ? h * V + d : h)]));
    reinterpret_cast<bf16*>(p.out)[row * p.ldo + h * V + d] = (bf16)(o * p.out_scale);
  }
}

constexpr size_t kFlashLds = 64 * 1024;

// LDS of the decode form with nw waves, before the bias entries
inline size_t decode_lds(const SinkAttnParams& p, int nw) {
  const int rep = p.H / p.G, cols = rep < 16 ? rep : 16;
  return 16 * (size_t)(p.D + 8) * sizeof(bf16) + (size_t)nw * cols * (p.V + 2) * sizeof(float);
}

template <int NT, int NW, bool EXT>
void launch_decode_waves(int num_work, const SinkAttnParams& p, const bf16* vt, hipStream_t st) {
  const int rep = p.H / p.G, cols = rep < 16 ? rep : 16;
  size_t lds = decode_lds(p, NW);
  int rel_lds = 0;
  if (EXT && p.rel) {
    const size_t room = (kFlashLds - lds) / (cols * sizeof(float));
    const size_t want = p.rel_len < 1024 ? (size_t)p.rel_len : 1024;
    rel_lds = (int)(want < room ? want : room);
    lds += cols * rel_lds * sizeof(float);
  }
  const int parts = p.nparts > 1 ? p.nparts : 1;
  hipLaunchKernelGGL((sink_decode_kernel<NT, 4, NW, EXT>), dim3(num_work, p.G, (rep + 15) / 16 * parts), dim3(NW * 64), lds,
                     st, p, vt, rel_lds);
  if (parts > 1)
    hipLaunchKernelGGL(sink_combine_kernel, dim3((num_work * p.H + 3) / 4), dim3(256), 0, st, p, num_work);
}

template <int NT>
void launch_decode(int num_work, const SinkAttnParams& p, const bf16* vt, hipStream_t st) {
  const bool ext = p.rel || p.keep_first > 0;
  if (decode_lds(p, 8) <= kFlashLds) {
    if (ext) launch_decode_waves<NT, 8, true>(num_work, p, vt, st);
    else launch_decode_waves<NT, 8, false>(num_work, p, vt, st);
  } else {
    if (ext) launch_decode_waves<NT, 4, true>(num_work, p, vt, st);
    else launch_decode_waves<NT, 4, false>(num_work, p, vt, st);
  }
}

template <int NT, bool EXT>
void launch_flash_ext(int num_work, const SinkAttnParams& p, const bf16* vt, int split, hipStream_t st) {
  const size_t qbytes = 16 * (size_t)(p.D + 8) * sizeof(bf16);
  auto strip = [&](size_t used, int strips) {  // bias entries per head that fit beside the rest, at most 1024
    if (!EXT || !p.rel || used >= kFlashLds) return 0;
    const size_t room = (kFlashLds - used) / (strips * sizeof(float));
    const size_t want = p.rel_len < 1024 ? (size_t)p.rel_len : 1024;
    return (int)(want < room ? want : room);
  };
  if (split) {  // one head per workgroup, its four waves share the keys; LDS: 4 query tiles + bias + the merge area
    size_t lds = 4 * 16 * (size_t)((p.D + 8 + 1) / 2) * sizeof(float) + 4 * 16 * (size_t)(p.V + 2) * sizeof(float);
    const int rel_lds = strip(lds, 1);
    lds += rel_lds * sizeof(float);
    hipLaunchKernelGGL((sink_flash_kernel<NT, true, EXT>), dim3(num_work, p.H), dim3(256), lds, st, p, vt, p.H, rel_lds);
    return;
  }
  const int wy = p.H < 4 ? p.H : 4;
  const int rel_lds = strip(wy * qbytes, wy);
  dim3 grid(num_work, (p.H + wy - 1) / wy), block(64 * wy);
  hipLaunchKernelGGL((sink_flash_kernel<NT, false, EXT>), grid, block, wy * (qbytes + rel_lds * sizeof(float)), st, p, vt,
                     p.H, rel_lds);
}

template <int NT>
void launch_flash(int num_work, const SinkAttnParams& p, const bf16* vt, int split, hipStream_t st) {
  if (p.rel || p.keep_first > 0) launch_flash_ext<NT, true>(num_work, p, vt, split, st);
  else launch_flash_ext<NT, false>(num_work, p, vt, split, st);
}

}  // namespace
}  // namespace dsse

// work_tile counts tiles of 16 rows; vt: transposed value pages [pages, G, V, kBS], keys permuted inside a page
extern "C" hipError_t dsse_sink_flash(int num_work, const dsse::SinkAttnParams* p, const void* vt, int split,
                                      hipStream_t st) {
  if (num_work <= 0 || p->H <= 0) return hipSuccess;
  if (p->f32 || p->D % 32 || p->V % 16 || p->V > 512 || p->D > 512 || p->H % p->G) return hipErrorInvalidValue;
  if (split && p->V > 128) return hipErrorInvalidValue;  // the merge area has to fit 64 KB of LDS
  if (p->out_rope && p->V % 32) return hipErrorInvalidValue;  // both halves of a rotation pair are whole 16-wide tiles
  const bf16* v = reinterpret_cast<const bf16*>(vt);
  switch (p->V / 16) {
#define DSSE_FLASH_CASE(n) case n: dsse::launch_flash<n>(num_work, *p, v, split, st); break;
    DSSE_FLASH_CASE(1) DSSE_FLASH_CASE(2) DSSE_FLASH_CASE(3) DSSE_FLASH_CASE(4) DSSE_FLASH_CASE(5) DSSE_FLASH_CASE(6)
    DSSE_FLASH_CASE(7) DSSE_FLASH_CASE(8) DSSE_FLASH_CASE(10) DSSE_FLASH_CASE(12) DSSE_FLASH_CASE(16)
    DSSE_FLASH_CASE(20) DSSE_FLASH_CASE(24) DSSE_FLASH_CASE(32)
#undef DSSE_FLASH_CASE
    default: return hipErrorInvalidValue;
  }
  return hipGetLastError();
}

// shared-page form: work_tile counts tiles of 16 rt rows, hb rt = 8; D and V up to 128, no bias and no output rotation
extern "C" hipError_t dsse_sink_tile(int num_work, const dsse::SinkAttnParams* p, const void* vt, int rt, hipStream_t st) {
  if (num_work <= 0 || p->H <= 0) return hipSuccess;
  if ((rt != 2 && rt != 4 && rt != 8) || p->H % p->G || (p->H / p->G) % (8 / rt)) return hipErrorInvalidValue;
  if (p->f32 || p->D % 32 || p->V % 16 || p->D > dsse::kTileWidth || p->V > dsse::kTileWidth || p->rel || p->out_rope ||
      num_work > 65535)
    return hipErrorInvalidValue;
  const int hb = 8 / rt;
  const dim3 grid(p->H / hb, num_work);
  const size_t lds = 2 * sizeof(bf16) * (dsse::kBS * (size_t)(p->D + 8) + (size_t)p->V * dsse::kTileLdv);
  const bf16* v = reinterpret_cast<const bf16*>(vt);
  switch (p->V / 16) {
#define DSSE_TILE_CASE(n) \
  case n: hipLaunchKernelGGL(dsse::sink_tile_kernel<n>, grid, dim3(256), lds, st, *p, v, hb, rt); break;
    DSSE_TILE_CASE(1) DSSE_TILE_CASE(2) DSSE_TILE_CASE(3) DSSE_TILE_CASE(4) DSSE_TILE_CASE(5) DSSE_TILE_CASE(6)
    DSSE_TILE_CASE(7) DSSE_TILE_CASE(8)
#undef DSSE_TILE_CASE
    default: return hipErrorInvalidValue;
  }
  return hipGetLastError();
}

// decode form: work_tile counts single rows; V / 16 as above, LDS for at least four waves
extern "C" hipError_t dsse_sink_decode(int num_work, const dsse::SinkAttnParams* p, const void* vt, hipStream_t st) {
  if (num_work <= 0 || p->H <= 0) return hipSuccess;
  if (p->f32 || p->D % 32 || p->V % 16 || p->V > 512 || p->D > 512 || p->H % p->G) return hipErrorInvalidValue;
  if (dsse::decode_lds(*p, 4) > dsse::kFlashLds) return hipErrorInvalidValue;
  if (p->nparts > dsse::kMaxParts || (p->nparts > 1 && !p->part)) return hipErrorInvalidValue;
  const bf16* v = reinterpret_cast<const bf16*>(vt);
  switch (p->V / 16) {
#define DSSE_DECODE_CASE(n) case n: dsse::launch_decode<n>(num_work, *p, v, st); break;
    DSSE_DECODE_CASE(1) DSSE_DECODE_CASE(2) DSSE_DECODE_CASE(3) DSSE_DECODE_CASE(4) DSSE_DECODE_CASE(5)
    DSSE_DECODE_CASE(6) DSSE_DECODE_CASE(7) DSSE_DECODE_CASE(8) DSSE_DECODE_CASE(10) DSSE_DECODE_CASE(12)
    DSSE_DECODE_CASE(16) DSSE_DECODE_CASE(20) DSSE_DECODE_CASE(24) DSSE_DECODE_CASE(32)
#undef DSSE_DECODE_CASE
    default: return hipErrorInvalidValue;
  }
  return hipGetLastError();
}

extern "C" hipError_t dsse_sink_attention(int num_work, const dsse::SinkAttnParams* p, hipStream_t st) {
  if (num_work <= 0 || p->H <= 0) return hipSuccess;
  if (p->D > 512 || p->V > dsse::kMaxV || p->H % p->G) return hipErrorInvalidValue;
  if (p->out_rope && p->V % 2) return hipErrorInvalidValue;
  dim3 grid(num_work, p->H);
  if (p->f32) hipLaunchKernelGGL(dsse::sink_attention_kernel<float>, grid, dim3(256), 0, st, *p);
  else hipLaunchKernelGGL(dsse::sink_attention_kernel<bf16>, grid, dim3(256), 0, st, *p);
  return hipGetLastError();
}
