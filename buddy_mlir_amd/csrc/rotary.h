// rotary.h -- rotary positions: frequencies with their length scalings, and the angle
// of a position.
#pragma once

#include "common.h"

#include <algorithm>
#include <cmath>
#include <vector>

namespace bh {

// Per pair of dimensions the turns of the full circle per position; `gain` goes onto
// cos and sin.
struct Rotary {
  std::vector<double> turns;
  double gain = 1.0;
  explicit Rotary(int dims, double base) {
    for (int i = 0; i < dims / 2; ++i)
      turns.push_back(std::pow(base, -2.0 * i / dims) / (2.0 * M_PI));
  }
  int dims() const { return 2 * (int)turns.size(); }

  // YaRN: pairs that turn more than `fast` times over the original length keep their
  // frequency, those below `slow` turns are slowed down by `factor`, a linear ramp over
  // the pairs in between.
  void yarn(double base, double factor, double original, double fast, double slow) {
    auto pair_of = [&](double t) { // (fractional) pair that makes t turns
      return dims() * std::log(original / (2.0 * M_PI * t)) / (2.0 * std::log(base));
    };
    const double lo = std::max(std::floor(pair_of(fast)), 0.0);
    const double hi = std::min(std::ceil(pair_of(slow)), dims() - 1.0);
    for (size_t i = 0; i < turns.size(); ++i) {
      const double ramp = std::clamp(((double)i - lo) / std::max(hi - lo, 0.001), 0.0, 1.0);
      turns[i] = turns[i] / factor * ramp + turns[i] * (1.0 - ramp);
    }
    gain = 0.1 * std::log(factor) + 1.0;
  }

  // Llama 3.1: wavelengths below original / high are kept, those above original / low
  // slowed down by `factor`, with a linear passage between the two bands.
  void banded(double factor, double low, double high, double original) {
    for (double &f : turns) {
      const double per = original * f; // original / wavelength
      if (per > high)
        continue;
      if (per < low) {
        f /= factor;
      } else {
        const double s = (per - low) / (high - low);
        f = (1.0 - s) * f / factor + s * f;
      }
    }
  }
};

#if defined(__HIPCC__)
// cos and sin of position * turns; the product is reduced to a fraction of a turn in
// double, so a far position keeps its 32-bit angle
__device__ __forceinline__ void rotation(double turns, int p, float &c, float &s) {
  double t = turns * (double)p;
  t -= rint(t);
  sincospif(2.0f * (float)t, &s, &c);
}
#endif

} // namespace bh
