// Rotation tables of the decoders built from layer descriptions: cos / sin of position * frequency, one table per kind of rotation.
#pragma once
#include <algorithm>
#include <cmath>
#include <vector>

#include "decoder.h"

struct RopeTable {
    double base = 0, factor = 0, original = 0, fast = 0, slow = 0;  // factor <= 0: no scaling
    int dims = 0;
    float *cos = nullptr, *sin = nullptr;                           // [positions][dims / 2]
    bool same(const RopeTable& o) const {
        return base == o.base && dims == o.dims && factor == o.factor && (factor <= 0 || (original == o.original && fast == o.fast && slow == o.slow));
    }
    // YaRN (Peng et al., "YaRN: Efficient Context Window Extension of Large Language Models"): slow pairs are divided by `factor`, fast ones
    // kept, a ramp over the pairs in between
    double frequency(int i) const {
        const double f = std::pow(base, -2.0 * i / dims);
        if (factor <= 0) return f;
        auto pair_of = [&](double turns) { return dims * std::log(original / (2 * M_PI * turns)) / (2 * std::log(base)); };
        const double lo = std::max(std::floor(pair_of(fast)), 0.0), hi = std::min(std::ceil(pair_of(slow)), dims - 1.0);
        const double ramp = std::min(std::max((i - lo) / std::max(hi - lo, 0.001), 0.0), 1.0);
        return f / factor * ramp + f * (1 - ramp);
    }
    double magnitude() const { return factor > 0 ? 0.1 * std::log(factor) + 1.0 : 1.0; }  // of both cos and sin
    int upload(nvllm_ctx* ctx, int positions) {
        const int half = dims / 2;
        std::vector<float> hc((size_t)positions * half), hs(hc.size());
        for (int i = 0; i < half; ++i) {
            const double f = frequency(i), mag = magnitude();
            for (int p = 0; p < positions; ++p) {
                hc[(size_t)p * half + i] = (float)(std::cos(p * f) * mag);
                hs[(size_t)p * half + i] = (float)(std::sin(p * f) * mag);
            }
        }
        int rc = dmalloc(ctx, &cos, hc.size());
        if (!rc) rc = dmalloc(ctx, &sin, hs.size());
        if (rc) return rc;
        HIPCHK(ctx, hipMemcpy(cos, hc.data(), hc.size() * 4, hipMemcpyHostToDevice));
        HIPCHK(ctx, hipMemcpy(sin, hs.data(), hs.size() * 4, hipMemcpyHostToDevice));
        return NVLLM_OK;
    }
    void release() {
        if (cos) (void)hipFree(cos);
        if (sin) (void)hipFree(sin);
        cos = sin = nullptr;
    }
};
// index of the table that serves `r`, added where there is none
static inline int rope_index(std::vector<RopeTable>& all, const RopeTable& r) {
    size_t t = 0;
    while (t < all.size() && !all[t].same(r)) ++t;
    if (t == all.size()) all.push_back(r);
    return (int)t;
}
