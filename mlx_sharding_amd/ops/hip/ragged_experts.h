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
  const void *h, *w, *correction;
  int* idx;        // [tokens, top], >= experts: an identity expert
  float* weight;   // [tokens, top]
  int* rank;       // [tokens, top], place among its block's pairs of an expert
  int* hist;       // [blocks, experts]
  long hstride, n;
  int K, experts, total, top;
};

struct PlanArgs {
  const int *idx, *rank, *hist;
  int *where;      // [tokens, top]: row among the sorted pairs, or -1
  int *tokens;     // [pairs]: token of a sorted pair
  int *tiles;      // [n_tiles, 3]: expert, first pair, pairs (0: none)
  long n;
  int experts, top, n_blocks, n_tiles, tile;
};

// out[p, o] = act(sum_k x[row(p), k] w[expert, o, k]) for the pairs of tiles
struct ExpertGemmArgs {
  const void *x, *w;
  void* out;
  const int *tokens, *tiles;  // tokens null: row(p) = p
  long xstride, ostride;
  int O, K, n_tiles;
  bool act;                   // relu(.)^2
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
