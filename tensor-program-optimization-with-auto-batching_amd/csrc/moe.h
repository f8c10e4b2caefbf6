// A routing plan of a mixture-of-experts layer: the (token, choice) entries sorted by expert and cut into tiles.  An entry's
// place in that order is its row in the hidden activations; every expert's places start at a multiple of 16.
#pragma once
#include "common.h"

struct MoePlan {
  const int32_t* perm;      // place -> entry (token * top + choice), -1 for the places between two experts
  const int4* tiles;        // {expert, first place, places, 0}
  const int32_t* n_tiles;   // device: tiles in use, then places in use (a multiple of 16)
};

int mlora_gemm_grouped(void* y, const void* xf, int x_tt, const void* Wp, const MoePlan& plan, int max_tiles, int K, int N, int act, float alpha,
                       void* stream);
