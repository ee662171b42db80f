// Rotation tables (/root/reference/src/ops/rope.rs:6-60), computed in double on the host.
#include <cmath>
#include <cstdlib>

#include "rt.h"

extern "C" {

int ornith_rope_table_scaled(ornith_ctx* ctx, int npos, int dims, double theta, double factor, float* d_cos,
                             float* d_sin) {
  ORN_REQUIRE(ctx && d_cos && d_sin, "rope_table: null argument");
  ORN_REQUIRE(npos >= 1 && dims >= 2 && dims % 2 == 0 && theta > 0 && factor > 0,
              "rope_table: npos=%d dims=%d theta=%g factor=%g", npos, dims, theta, factor);
  const int half = dims / 2;
  float* hc = (float*)malloc(sizeof(float) * (size_t)npos * half * 2);
  if (!hc) return ornith_fail(ORNITH_ERR_INVALID, "rope_table: out of host memory");
  float* hs = hc + (size_t)npos * half;
  for (int i = 0; i < half; ++i) {
    const double inv_freq = pow(theta, -(double)i / (double)half) / factor;
    for (int pos = 0; pos < npos; ++pos) {
      const double ang = (double)pos * inv_freq;
      hc[(size_t)pos * half + i] = (float)cos(ang);
      hs[(size_t)pos * half + i] = (float)sin(ang);
    }
  }
  int rc = ornith_upload(ctx, d_cos, hc, sizeof(float) * (size_t)npos * half);
  if (!rc) rc = ornith_upload(ctx, d_sin, hs, sizeof(float) * (size_t)npos * half);
  free(hc);
  return rc;
}

int ornith_rope_table(ornith_ctx* ctx, int npos, int dims, double theta, float* d_cos, float* d_sin) {
  return ornith_rope_table_scaled(ctx, npos, dims, theta, 1.0, d_cos, d_sin);
}

}  // extern "C"
