// Products of rows dealt to several weights of one shape (routed experts), on the 128 x 128 tiles of the GEMMs.
#pragma once

#include "common.h"

namespace iron {

// Row tiles of 128: how many there are (read on the device), how many there can be, and the weight each belongs to.
struct GroupedTiles {
  const int* count;
  const int* which;
  int most;
};

// C[pos] = act(Bg A[a_rows[pos]]) * (Bu A[a_rows[pos]]) and C[pos] = B A[pos], of the tile's weight; K a multiple of 64.
int launch_grouped_pair(const bf16_t* A, const bf16_t* Bg, const bf16_t* Bu, bf16_t* C, int N, int K, const GroupedTiles& g,
                        const int* a_rows, int activation, hipStream_t s);
int launch_grouped(const bf16_t* A, const bf16_t* B, bf16_t* C, int N, int K, const GroupedTiles& g, hipStream_t s);

}  // namespace iron
