// Routers that pick several experts a token, and what surrounds their grouped products.
//
// router_topk: from the router's fp32 logits z [T, E] the `top` experts with the largest choice
// values are taken (the lowest index wins among equals), and each gets a weight.  Four ways of scoring:
//   sigmoid (mode 0): scores s = sigmoid(z); the choice goes by s + bias (bias may be null); an expert's
//     weight is its score s without the bias, divided by the sum of the taken scores if `renorm`;
//   softmax over the taken (mode 1): the choice goes by z + bias; the weights are the softmax of the taken
//     experts' logits z alone (they add up to one; `renorm` has nothing left to do);
//   softmax over the taken, bias inside (mode 3): z + bias are the logits themselves: the choice goes by them and the
//     weights are their softmax over the taken;
//   softmax over all (mode 2): scores s = softmax(z) over every expert; choice and weights as with sigmoid.
// With `n_groups` > 1 the experts form equal groups of neighbours and only those of the `keep_groups` groups whose
// largest choice value is largest can be taken (the lowest group among equals).  The logits' rows may lie `ld` apart.
// Outputs expert[t*top + j] and weight[t*top + j] in the order of choice:
// "virtual tokens" t*top + j that the expert plan (moe_plan with its fan) sorts by expert.
// moe_combine: out[t] = sum_j weight[t*top + j] * y[t*top + j] (+ extra[t]) in fp32, j in order (no weights: all 1);
// with `gate` the extra row is multiplied by sigmoid(gate[t*ldg]).
// gated_rows: g[t] = gelu_tanh(a[t]) * table[ids[t]][col0 .. col0 + n): a gate on a per-token row
// of a table (a second, small embedding that a layer mixes into the stream).
#include "common.h"

#define TOPK_MAX_PER_LANE 8      // up to 512 experts

// NU: experts a lane, so that 64 * NU >= E.
template <int NU>
__global__ __launch_bounds__(256)
void router_topk_kernel(const float* __restrict__ logits, const float* __restrict__ bias, int* __restrict__ expert,
                        float* __restrict__ weight, int T, int E, int ld, int top, int renorm, int mode,
                        int n_groups, int keep_groups) {
    const int lane = threadIdx.x & 63;
    const int t = blockIdx.x * 4 + (threadIdx.x >> 6);
    if (t >= T) return;
    float s[NU], c[NU];
#pragma unroll
    for (int u = 0; u < NU; ++u) {
        const int e = lane + u * 64;
        s[u] = 0.f; c[u] = -INFINITY;
        if (e < E) {
            const float z = logits[(size_t)t * ld + e];
            s[u] = mode == 0 ? 1.0f / (1.0f + expf(-z)) : z;
            if (mode == 3 && bias) s[u] += bias[e];
        }
    }
    if (mode == 3) { bias = nullptr; mode = 1; }
    if (mode == 2) {
        float zm = -INFINITY, zs = 0.f;
#pragma unroll
        for (int u = 0; u < NU; ++u) if (lane + u * 64 < E) zm = fmaxf(zm, s[u]);
        zm = wave_max(zm);
#pragma unroll
        for (int u = 0; u < NU; ++u) if (lane + u * 64 < E) { s[u] = expf(s[u] - zm); zs += s[u]; }
        zs = 1.0f / wave_sum(zs);
#pragma unroll
        for (int u = 0; u < NU; ++u) s[u] *= zs;
    }
#pragma unroll
    for (int u = 0; u < NU; ++u) {
        const int e = lane + u * 64;
        if (e < E) {
            c[u] = s[u] + (bias ? bias[e] : 0.f);
            if (!(c[u] == c[u])) c[u] = -INFINITY;          // a NaN is never chosen before a number
        }
    }
    if (n_groups > 1) {
        // the best group left is the group of the best expert of the groups left
        const int gs = E / n_groups;
        int grp[NU];
#pragma unroll
        for (int u = 0; u < NU; ++u) grp[u] = (lane + u * 64) / gs;
        unsigned open = 0;                                  // bit u: this lane's expert u is in a group that stays
        for (int j = 0; j < keep_groups; ++j) {
            float best = -INFINITY; int be = 0x7fffffff;
#pragma unroll
            for (int u = 0; u < NU; ++u) {
                const int e = lane + u * 64;
                if (e < E && !(open >> u & 1) && (c[u] > best || (c[u] == best && e < be))) { best = c[u]; be = e; }
            }
#pragma unroll
            for (int o = 32; o > 0; o >>= 1) {
                const float ob = __shfl_xor(best, o, 64); const int oe = __shfl_xor(be, o, 64);
                if (ob > best || (ob == best && oe < be)) { best = ob; be = oe; }
            }
            const int gb = be / gs;
#pragma unroll
            for (int u = 0; u < NU; ++u) if (lane + u * 64 < E && grp[u] == gb) open |= 1u << u;
        }
#pragma unroll
        for (int u = 0; u < NU; ++u) if (!(open >> u & 1)) c[u] = -INFINITY;
    }
    float sum = 0.f, top_z = -INFINITY;          // mode 1: the sum of exp(z - top_z) over the taken so far
    float mine_w = 0.f; int mine_e = 0;
    for (int j = 0; j < top; ++j) {
        float best = -INFINITY; int be = 0x7fffffff; float bs = 0.f;
#pragma unroll
        for (int u = 0; u < NU; ++u) {
            const int e = lane + u * 64;
            if (e < E && (c[u] > best || (c[u] == best && e < be))) { best = c[u]; be = e; bs = s[u]; }
        }
#pragma unroll
        for (int o = 32; o > 0; o >>= 1) {
            const float ob = __shfl_xor(best, o, 64); const int oe = __shfl_xor(be, o, 64); const float os = __shfl_xor(bs, o, 64);
            if (ob > best || (ob == best && oe < be)) { best = ob; be = oe; bs = os; }
        }
        // a taken expert leaves the contest: its mark lies below every score
#pragma unroll
        for (int u = 0; u < NU; ++u) if (lane + u * 64 == be) c[u] = -INFINITY;
        if (mode == 1) {
            const float nz = fmaxf(top_z, bs);
            sum = sum * expf(top_z - nz) + expf(bs - nz);        // (exp(-inf) = 0 at the first)
            top_z = nz;
        } else {
            sum += bs;
        }
        if (lane == j % 64 && j < 64) { mine_w = bs; mine_e = be; }
        if (j >= 64 && lane == 0) { expert[(size_t)t * top + j] = be; weight[(size_t)t * top + j] = bs; }
    }
    if (mode == 1) {
        const float inv = 1.0f / sum;
        if (lane < top && lane < 64) { expert[(size_t)t * top + lane] = mine_e; weight[(size_t)t * top + lane] = expf(mine_w - top_z) * inv; }
        if (top > 64 && lane == 0) for (int j = 64; j < top; ++j) weight[(size_t)t * top + j] = expf(weight[(size_t)t * top + j] - top_z) * inv;
        return;
    }
    const float inv = renorm ? 1.0f / (sum + 1e-20f) : 1.0f;
    if (lane < top && lane < 64) { expert[(size_t)t * top + lane] = mine_e; weight[(size_t)t * top + lane] = mine_w * inv; }
    if (renorm && top > 64 && lane == 0) for (int j = 64; j < top; ++j) weight[(size_t)t * top + j] *= inv;
}

extern "C" int spite_router_topk(const float* logits, const float* bias, int* expert, float* weight, int T, int E, int ld, int top,
                                 int renorm, int mode, int n_groups, int keep_groups, hipStream_t st) {
    SP_REQUIRE(mode >= 0 && mode <= 3, "router_topk: scoring %d", mode);
    SP_REQUIRE(ld >= E, "router_topk: rows of %d logits for %d experts", ld, E);
    SP_REQUIRE(n_groups >= 1 && E > 0 && E % n_groups == 0 && keep_groups >= 1 && keep_groups <= n_groups, "router_topk: %d of %d groups of %d experts",
               keep_groups, n_groups, E);
    SP_REQUIRE(top <= keep_groups * (E / n_groups), "router_topk: %d experts out of %d groups of %d", top, keep_groups, E / n_groups);
    SP_REQUIRE(T >= 0 && E > 0 && E <= 64 * TOPK_MAX_PER_LANE, "router_topk: %d experts, at most %d", E, 64 * TOPK_MAX_PER_LANE);
    SP_REQUIRE(top > 0 && top <= E, "router_topk: %d of %d experts", top, E);
    if (T == 0) return 0;
#define SP_RT(NU) router_topk_kernel<NU><<<(T + 3) / 4, 256, 0, st>>>(logits, bias, expert, weight, T, E, ld, top, renorm, mode, n_groups, keep_groups)
    if (E <= 64) SP_RT(1);
    else if (E <= 128) SP_RT(2);
    else if (E <= 256) SP_RT(4);
    else SP_RT(TOPK_MAX_PER_LANE);
#undef SP_RT
    SP_LAUNCH_CHECK("router_topk");
    return 0;
}

// VEC elements a thread (4 where rows are a multiple of four floats and 16-byte aligned); every element is summed in
// the same order either way.
template <int VEC>
__global__ __launch_bounds__(256)
void moe_combine_kernel(const float* __restrict__ y, const float* __restrict__ weight, const float* __restrict__ extra,
                        const float* __restrict__ gate, int ldg, float* __restrict__ out, int T, int d, int top) {
    typedef float vec __attribute__((ext_vector_type(VEC)));
    const size_t i = (size_t)blockIdx.x * 256 + threadIdx.x;
    const int dv = d / VEC;
    if (i >= (size_t)T * dv) return;
    const size_t t = i / dv, c = (i - t * dv) * VEC;
    vec acc;
#pragma unroll
    for (int e = 0; e < VEC; ++e) acc[e] = 0.f;
    for (int j = 0; j < top; ++j) {
        const float w = weight ? weight[t * top + j] : 1.0f;
        const vec v = *(const vec*)(y + (t * top + j) * d + c);
#pragma unroll
        for (int e = 0; e < VEC; ++e) acc[e] = fmaf(w, v[e], acc[e]);
    }
    if (extra) {
        const vec x = *(const vec*)(extra + t * d + c);
        const float g = gate ? 1.0f / (1.0f + expf(-gate[t * ldg])) : 1.0f;
#pragma unroll
        for (int e = 0; e < VEC; ++e) acc[e] += g * x[e];
    }
    *(vec*)(out + t * d + c) = acc;
}

extern "C" int spite_moe_combine(const float* y, const float* weight, const float* extra, const float* gate, int ldg, float* out,
                                 int T, int d, int top, hipStream_t st) {
    SP_REQUIRE(T >= 0 && d > 0 && top > 0, "moe_combine: bad sizes T=%d d=%d top=%d", T, d, top);
    SP_REQUIRE(!gate || (extra && ldg >= 1), "moe_combine: a gate without the row that it gates");
    if (T == 0) return 0;
    auto al = [](const void* p) { return ((uintptr_t)p & 15) == 0; };
    const bool v4 = d % 4 == 0 && al(y) && al(extra) && al(out);
    const size_t n = (size_t)T * (v4 ? d / 4 : d);
    SP_REQUIRE((n + 255) / 256 < (1u << 31), "moe_combine: too many elements");
    const unsigned grid = (unsigned)((n + 255) / 256);
    if (v4) moe_combine_kernel<4><<<grid, 256, 0, st>>>(y, weight, extra, gate, ldg, out, T, d, top);
    else moe_combine_kernel<1><<<grid, 256, 0, st>>>(y, weight, extra, gate, ldg, out, T, d, top);
    SP_LAUNCH_CHECK("moe_combine");
    return 0;
}

template <typename TA, typename TT>
__global__ __launch_bounds__(256)
void gated_rows_kernel(const TA* __restrict__ a, const int* __restrict__ ids, const TT* __restrict__ table, int ld_table,
                       int col0, TA* __restrict__ g, int T, int n, int fast) {
    const size_t i = (size_t)blockIdx.x * 256 + threadIdx.x;
    if (i >= (size_t)T * n) return;
    const size_t t = i / n, c = i - t * n;
    const float z = to_f32<TA>(a[i]);
    const float act = 0.5f * z * (1.0f + (fast ? 1.0f - 2.0f / (__expf(2.0f * 0.7978845608028654f * (z + 0.044715f * z * z * z)) + 1.0f)
                                              : tanhf(0.7978845608028654f * (z + 0.044715f * z * z * z))));
    g[i] = from_f32<TA>(act * to_f32<TT>(table[(size_t)ids[t] * ld_table + col0 + c]));
}

extern "C" int spite_gated_rows(const void* a, int dtype, const int* ids, const void* table, int table_dtype, int ld_table,
                                int col0, void* g, int T, int n, hipStream_t st) {
    SP_REQUIRE(T >= 0 && n > 0 && col0 >= 0 && col0 + n <= ld_table, "gated_rows: columns %d..%d of %d", col0, col0 + n, ld_table);
    if (T == 0) return 0;
    const unsigned grid = (unsigned)(((size_t)T * n + 255) / 256);
    if (dtype == SP_F32 && table_dtype == SP_F32)
        gated_rows_kernel<float, float><<<grid, 256, 0, st>>>((const float*)a, ids, (const float*)table, ld_table, col0, (float*)g, T, n, 0);
    else if (dtype == SP_BF16 && table_dtype == SP_BF16)
        gated_rows_kernel<bf16, bf16><<<grid, 256, 0, st>>>((const bf16*)a, ids, (const bf16*)table, ld_table, col0, (bf16*)g, T, n, 1);
    else if (dtype == SP_BF16 && table_dtype == SP_F32)
        gated_rows_kernel<bf16, float><<<grid, 256, 0, st>>>((const bf16*)a, ids, (const float*)table, ld_table, col0, (bf16*)g, T, n, 1);
    else return sp_fail("gated_rows: dtypes %d and %d", dtype, table_dtype);
    SP_LAUNCH_CHECK("gated_rows");
    return 0;
}
