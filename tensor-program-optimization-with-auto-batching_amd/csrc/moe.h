// A routing plan of a mixture-of-experts layer: the (token, choice) entries sorted by expert and cut into tiles.
#pragma once
#include "common.h"

struct MoePlan {
  const int32_t* perm;      // [T * top] sorted place -> entry (token * top + choice)
  const int4* tiles;        // {expert, first place, places, 0}
  const int32_t* n_tiles;   // tiles in use (device)
};
