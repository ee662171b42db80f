// Rotation tables (/root/reference/src/ops/rope.rs:6-60), computed in double on the host.
#include <cmath>
#include <cstdlib>
#include <vector>

#include "rt.h"

namespace {

// cos and sin of position * freq, times gain
int make_tables(ornith_ctx* ctx, int npos, const std::vector<double>& freq, double gain, float* d_cos, float* d_sin) {
  const size_t half = freq.size();
  float* hc = (float*)malloc(sizeof(float) * (size_t)npos * half * 2);
  if (!hc) return ornith_fail(ORNITH_ERR_INVALID, "rope_table: out of host memory");
  float* hs = hc + (size_t)npos * half;
  for (size_t i = 0; i < half; ++i) {
    for (int pos = 0; pos < npos; ++pos) {
      const double ang = (double)pos * freq[i];
      hc[(size_t)pos * half + i] = (float)(gain * cos(ang));
      hs[(size_t)pos * half + i] = (float)(gain * sin(ang));
    }
  }
  int rc = ornith_upload(ctx, d_cos, hc, sizeof(float) * (size_t)npos * half);
  if (!rc) rc = ornith_upload(ctx, d_sin, hs, sizeof(float) * (size_t)npos * half);
  free(hc);
  return rc;
}

}  // namespace

extern "C" {

int ornith_rope_table_scaled(ornith_ctx* ctx, int npos, int dims, double theta, double factor, float* d_cos,
                             float* d_sin) {
  ORN_REQUIRE(ctx && d_cos && d_sin, "rope_table: null argument");
  ORN_REQUIRE(npos >= 1 && dims >= 2 && dims % 2 == 0 && theta > 0 && factor > 0,
              "rope_table: npos=%d dims=%d theta=%g factor=%g", npos, dims, theta, factor);
  const int half = dims / 2;
  std::vector<double> freq(half);
  for (int i = 0; i < half; ++i) freq[i] = pow(theta, -(double)i / (double)half) / factor;
  return make_tables(ctx, npos, freq, 1.0, d_cos, d_sin);
}

int ornith_rope_table_yarn(ornith_ctx* ctx, int npos, int dims, double theta, double factor, double original, double fast,
                           double slow, float* d_cos, float* d_sin) {
  ORN_REQUIRE(ctx && d_cos && d_sin, "rope_table: null argument");
  ORN_REQUIRE(npos >= 1 && dims >= 2 && dims % 2 == 0 && theta > 0 && theta != 1.0 && factor > 0 && original > 0 && fast > 0 && slow > 0,
              "rope_table: npos=%d dims=%d theta=%g, stretched %g times from %g positions between %g and %g turns", npos, dims,
              theta, factor, original, fast, slow);
  const int half = dims / 2;
  // the pair that turns so many times over the original positions
  auto pair_of = [&](double turns) { return dims * log(original / (2.0 * M_PI * turns)) / (2.0 * log(theta)); };
  const double lo = fmax(floor(pair_of(fast)), 0.0), hi = fmin(ceil(pair_of(slow)), dims - 1.0), run = fmax(hi - lo, 0.001);
  std::vector<double> freq(half);
  for (int i = 0; i < half; ++i) {
    const double f = pow(theta, -(double)i / (double)half), ramp = fmin(fmax((i - lo) / run, 0.0), 1.0);
    freq[i] = f / factor * ramp + f * (1.0 - ramp);
  }
  return make_tables(ctx, npos, freq, 0.1 * log(factor) + 1.0, d_cos, d_sin);
}

int ornith_rope_table(ornith_ctx* ctx, int npos, int dims, double theta, float* d_cos, float* d_sin) {
  return ornith_rope_table_scaled(ctx, npos, dims, theta, 1.0, d_cos, d_sin);
}

}  // extern "C"
