// Host-visible API of the kernels that serve designs with convolved attention, attention beside a matrix memory, and
// experts chosen by token id: the rows of a fused q | k | v projection through a short convolution, an interleaved
// rotation and their pages; the matrix memory with exponential gates; the work lists of table-routed experts.
//
// Conventions as in api_mixers.h: activations between kernels are fp32, `T` (bf16 or fp32) appears where a projection
// reads or a page stores; per sequence q_start, q_len (0 = inactive) and ctx_len (tokens after this step).
#pragma once
#include "api.h"

namespace dsse {

struct ConvQkvParams {
  const float* x;        // rows ldx apart: [q (H D) | k (G D) | v (G V) | ..]
  const float* taps;     // [(H + G) D, K] or null (K = 0): no convolution; taps[c][K - 1] weighs the row itself
  float* tail;           // [slots, K - 1, (H + G) D] the sequence's last projected rows (K > 1)
  const int* q_start;
  const int* q_len;
  const int* ctx_len;
  const int* state_slot;
  const int* work_seq;
  const int* work_tile;  // tiles of qt rows
  const float2* rope;    // [rope_len, half] (cos, sin) of the interleaved pairs, or null
  const float* q_factor; // [q_factor_len] per position, or null
  const int* slots;      // [T] cache row, negative = skip
  float* q;              // [T, H, D]
  void* k;               // [pages * kBS, G, D] element type
  void* v;               // [pages * kBS, G, V or D]
  void* vt;              // transposed value pages [pages, G, V or D, kBS], or null
  int nwork, nseq, qt, H, G, D, V, K, ldx, half, rope_len, q_factor_len, num_slots, f32;  // V = 0: the values are the keys
};

struct MatrixMemoryParams {
  const float* q;        // [T, H, D] rows ldq apart
  const float* k;        // rows ldk apart
  const float* v;        // [T, H, V] rows ldv apart
  const float* gates;    // [T, 2 H] rows ldz apart: input gates, then forget gates
  const float* gate_b;   // [2 H]
  float* state;          // [slots, H, D, V]
  float* norm;           // [slots, H, D + 1]: normaliser, running maximum
  const int* q_start;
  const int* q_len;
  const int* ctx_len;
  const int* state_slot;
  const float* out_gate; // [T, H V] rows ldg apart
  const float* norm_w;   // [H V]
  void* out;             // [T, H V] rows ldo apart, element type
  int nseq, T, H, D, V, ldq, ldk, ldv, ldz, ldg, ldo, f32;
  float cap, eps, den_eps, q_scale, out_scale;
  // chunk form: its work areas and the rows that the sequences of the call cover
  float* num;            // [T, H, V] read-outs before the division
  float* nq;             // [T, H] normaliser products
  float* m;              // [T, H] running maxima
  float* acum;           // [H, ldsum] log2-decay sums inside a chunk, sequences at multiples of four
  float* u;              // [H, ldsum] log2 write strength minus that sum
  int ldsum;             // at least T + 4 nseq + 4, a multiple of 4
  int row0, rows;
  int vec;               // 16-byte loads of q and k rows allowed
};

constexpr int kTableLayers = 24;  // layers per launch of the table-routed work lists

struct MoeTableListsParams {
  const int* ids;        // [M]
  int M, vocab, layers;
  struct Layer {
    const int* table;    // [vocab, top]
    int* topk_idx;       // [M, top]
    int* sorted;
    int* tile_expert;
    int* num_tiles;
    int E, top, S, max_tiles;
  } layer[kTableLayers];
};

}  // namespace dsse

extern "C" {
hipError_t dsse_conv_qkv_rows(const dsse::ConvQkvParams* p, hipStream_t st);
// a token at a time, any widths up to 512, both element types: decode steps, and the exact form of prompt portions
hipError_t dsse_matrix_memory_walk(const dsse::MatrixMemoryParams* p, hipStream_t st);
// chunks of 32 tokens on MFMA (bf16 operands in two parts where the state enters): D <= 256, D % 4 == 0
hipError_t dsse_matrix_memory_chunk(const dsse::MatrixMemoryParams* p, hipStream_t st);
hipError_t dsse_moe_table_lists(const dsse::MoeTableListsParams* p, hipStream_t st);
}
