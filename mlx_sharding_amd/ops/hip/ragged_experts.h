// Arguments of the routed experts.
#pragma once

#include "ragged_common.h"

#define EX_TOK 16      // tokens of a router block
#define EX_GROUPS 4    // router blocks whose pairs one planning block places
#define EX_MAXTOTAL 1024
#define EX_STEP 64     // contractions are padded to this many elements

// w: matrix-core operands of 16 experts by 32 columns, [tiles, K / 32, 64, 8],
// lane = (column / 8 % 4, expert % 16)
struct RouteArgs {
  const void *h, *w, *correction;  // correction may be null
  int* idx;        // [tokens, top], >= experts: an identity expert
  float* weight;   // [tokens, top]
  int* rank;       // [tokens, top], place among its block's pairs of an expert
  int* hist;       // [blocks, experts]
  long hstride, n;
  int K, experts, total, top;
  bool sigmoid;    // scores are sigmoids instead of softmax
  bool normalize;  // weights are divided by their sum
};

struct PlanArgs {
  const int *idx, *rank, *hist;
  const float* weight;  // [tokens, top] or null
  float* scale;         // [pairs]: weight of a sorted pair
  int *where;      // [tokens, top]: row among the sorted pairs, or -1
  int *tokens;     // [pairs]: token of a sorted pair
  int *tiles;      // [n_tiles, 3]: expert, first pair, pairs (0: none)
  long n;
  int experts, top, n_blocks, n_tiles, tile;
};

// out[p, o] = act(scale[p] sum_k x[row(p), k] w[expert, o, k]) for the pairs of
// tiles.  A gated unit takes rows o (gate) and O / 2 + o (up) of w.
enum ExpertAct { EX_NONE = 0, EX_RELU2 = 1, EX_CLAMPED_GLU = 2 };

struct ExpertGemmArgs {
  const void *x, *w;
  void* out;
  const int *tokens, *tiles;  // tokens null: row(p) = p
  const float* scale;         // null: 1
  long xstride, ostride;
  int O, K, n_tiles;
  int act;                    // ExpertAct
  float limit, alpha;         // of a gated unit
};

struct CombineArgs {
  float* x;
  const void *h, *d;
  void* copy;      // x in T, or null
  const int* where;
  const float* weight;
  long hstride, dstride, n;
  int W, top;
};

struct TokenGateArgs {
  const float* x;             // [n, K]
  const void *w, *e;          // operands as the router's, [n, O]
  void* out;                  // [n, O]
  long estride;
  int n, O, K;
};
