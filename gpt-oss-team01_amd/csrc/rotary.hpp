// Rotary positions: tables of cos and sin, and the rotation of heads in place (rotary.hip).
#pragma once
#include <vector>

#include "common.hpp"

namespace gptoss {

// What the angles are made from.  Pair i of `dims` / 2 turns by base^(-2i / dims) per position; with
// factor > 0 the slow pairs' frequencies are divided by it (YaRN: pairs that turn more than `fast` times in
// `original` positions keep theirs, those with less than `slow` turns are divided, a ramp in between) and
// cos and sin are multiplied by 0.1 ln(factor) + 1.
struct RotarySpec {
  int dims = 0;
  double base = 10000.0, factor = 0.0, original = 0.0, fast = 0.0, slow = 0.0;
  bool operator==(const RotarySpec &o) const {
    return dims == o.dims && base == o.base && factor == o.factor && original == o.original && fast == o.fast && slow == o.slow;
  }
};
// [positions][dims / 2] pairs (cos, sin), evaluated in double
std::vector<float> rotary_table(const RotarySpec &spec, int positions);

// The first `dims` dimensions of a head are rotated: pairs (2i, 2i + 1) when interleaved, else (i, i + dims / 2).
struct Rotary {
  const float *table = nullptr;   // device; nullptr: no rotation
  int dims = 0, interleaved = 0;
};
// heads of `dim` columns from column `col` on of rows `x` [n, ld], in place; row r is position lens[r] - 1
int run_rotary(const Rotary &r, float *x, int ld, int col, int heads, int dim, const int *lens, int n, hipStream_t s);

}  // namespace gptoss
