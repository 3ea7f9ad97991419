// The gated delta rule: a recurrent state per head that a token corrects instead of adding to.  Per head, S: D x V,
//
//   S <- g_t S;   u_t = beta_t (v_t - S^T k_t);   S <- S + k_t u_t^T;   o_t = S^T q_t
//
// with one decay g and one step size beta a head and token, and q, k unit vectors (q times a constant) shared by the
// H / G value heads of a q/k head.  The state lives in fp32 in a row per request slot, [slots, H, D, V].
//
// delta_gates:   the numbers that enter the recurrence beside the projected rows, fp32: the factors that make q and k
//                unit vectors, log g = -exp(A_log) softplus(a + dt_bias), beta = sigmoid(b).
// delta_scan:    the recurrence token by token, any sizes, either dtype.
// delta_step:    the same for steps of single tokens: one pass over the state.
// delta_chunk:   the same for prompts in bfloat16 on the matrix units, 32 tokens at a time (two kernels, see there).
//
// q, k, v are the run's dtype as the convolution leaves them; everything from there on is fp32: the unit vectors are formed
// by multiplying the rows with their factor in fp32, and no product or sum of the recurrence loses bits to bfloat16.
#include "common.h"

#define DR_MAXD 256

// ------------------------------------------------------------------ factors, decays, step sizes
// A wave takes one q/k head of a token (both sums of squares) or, the last item of a token, the heads' decays and
// step sizes.  qk_scale [T][2][G]: q's factor q_scale / sqrt(sum q^2 + eps), then k's; gates [T][2][H]: log g, then beta.
template <typename T>
__global__ __launch_bounds__(256)
void delta_gates_kernel(const T* __restrict__ q, const T* __restrict__ k, int ldq, int ldk, const T* __restrict__ raw_a, int lda,
                        const T* __restrict__ raw_b, int ldb, const float* __restrict__ a_log, const float* __restrict__ dt_bias,
                        float q_scale, float eps, float* __restrict__ qk_scale, float* __restrict__ gates, int Tn, int G, int H, int D) {
    const int lane = threadIdx.x & 63;
    const size_t item = (size_t)blockIdx.x * 4 + (threadIdx.x >> 6);
    if (item >= (size_t)Tn * (G + 1)) return;
    const size_t t = item / (G + 1);
    const int g = (int)(item - t * (G + 1));
    if (g < G) {
        const T* qr = q + t * ldq + (size_t)g * D;
        const T* kr = k + t * ldk + (size_t)g * D;
        float sq = 0.f, sk = 0.f;
        for (int c = lane; c < D; c += 64) {
            const float x = to_f32<T>(qr[c]), y = to_f32<T>(kr[c]);
            sq = fmaf(x, x, sq);
            sk = fmaf(y, y, sk);
        }
        sq = wave_sum(sq);
        sk = wave_sum(sk);
        if (lane == 0) {
            qk_scale[t * 2 * G + g] = q_scale / sqrtf(sq + eps);
            qk_scale[t * 2 * G + G + g] = 1.0f / sqrtf(sk + eps);
        }
        return;
    }
    for (int h = lane; h < H; h += 64) {
        const float z = to_f32<T>(raw_a[t * lda + h]) + dt_bias[h];
        const float step = z > 20.f ? z + log1pf(expf(-z)) : log1pf(expf(z));           // softplus
        gates[t * 2 * H + h] = -expf(a_log[h]) * step;
        gates[t * 2 * H + H + h] = 1.0f / (1.0f + expf(-to_f32<T>(raw_b[t * ldb + h])));
    }
}

extern "C" int spite_delta_gates(const void* q, const void* k, int ldq, int ldk, const void* raw_a, int lda, const void* raw_b, int ldb,
                                 int dtype, const float* a_log, const float* dt_bias, float q_scale, float eps, float* qk_scale,
                                 float* gates, int T, int G, int H, int D, hipStream_t st) {
    SP_REQUIRE(T >= 0 && G > 0 && H > 0 && D > 0 && eps > 0.f, "delta_gates: bad sizes T=%d G=%d H=%d D=%d", T, G, H, D);
    SP_REQUIRE(ldq >= G * D && ldk >= G * D && lda >= H && ldb >= H, "delta_gates: rows shorter than the heads");
    if (T == 0) return 0;
    const size_t items = (size_t)T * (G + 1);
    SP_REQUIRE((items + 3) / 4 < (1u << 31), "delta_gates: too many heads");
    const unsigned grid = (unsigned)((items + 3) / 4);
    if (dtype == SP_F32)
        delta_gates_kernel<float><<<grid, 256, 0, st>>>((const float*)q, (const float*)k, ldq, ldk, (const float*)raw_a, lda, (const float*)raw_b, ldb,
                                                        a_log, dt_bias, q_scale, eps, qk_scale, gates, T, G, H, D);
    else if (dtype == SP_BF16)
        delta_gates_kernel<bf16><<<grid, 256, 0, st>>>((const bf16*)q, (const bf16*)k, ldq, ldk, (const bf16*)raw_a, lda, (const bf16*)raw_b, ldb,
                                                       a_log, dt_bias, q_scale, eps, qk_scale, gates, T, G, H, D);
    else return sp_fail("delta_gates: unknown dtype %d", dtype);
    SP_LAUNCH_CHECK("delta_gates");
    return 0;
}

// ------------------------------------------------------------------ the recurrence, token by token
// A workgroup of 256 threads takes 16 value columns of one head of one entry of the step and walks the entry's tokens in
// order; 16 lanes share a column and hold the state's key channels c(r) = (r/4)*64 + 4*lane + r%4 in registers, so both
// sums over the key channels stay within a row of 16 lanes.  The tokens' rows go through LDS in blocks.  The order of every
// sum depends on D alone.
#define DS_VC 16
#define DS_NT 256
#define DS_TB 16

template <typename T, int RR>
__global__ __launch_bounds__(DS_NT)
void delta_scan_kernel(const T* __restrict__ q, const T* __restrict__ k, const T* __restrict__ v, int ldq, int ldk, int ldv,
                       const float* __restrict__ qk_scale, const float* __restrict__ gates, float* __restrict__ state,
                       const int* __restrict__ cu_seqlens, const int* __restrict__ seq_slots, float* __restrict__ out,
                       int H, int G, int D, int V) {
    constexpr int Dp = 64 * RR, PR = 4 * RR;
    __shared__ __attribute__((aligned(16))) float qs[DS_TB][Dp], ks[DS_TB][Dp];
    __shared__ float vs[DS_TB][DS_VC], gs[DS_TB][2];
    const int e = blockIdx.x, h = blockIdx.y, v0 = blockIdx.z * DS_VC;
    const int tid = threadIdx.x, vc = tid >> 4, dg = tid & 15;
    const int t_lo = cu_seqlens[e], t_hi = cu_seqlens[e + 1];
    if (t_lo >= t_hi) return;
    const int g = h / (H / G), vcol = v0 + vc;
    const bool vok = vcol < V;
    float* srow = state + ((size_t)seq_slots[e] * H + h) * (size_t)D * V;
    float S[PR];
#pragma unroll
    for (int r = 0; r < PR; ++r) {
        const int d = (r >> 2) * 64 + dg * 4 + (r & 3);
        S[r] = d < D && vok ? srow[(size_t)d * V + vcol] : 0.f;
    }
    for (int t0 = t_lo; t0 < t_hi; t0 += DS_TB) {
        const int n_tok = t_hi - t0 < DS_TB ? t_hi - t0 : DS_TB;
        __syncthreads();
        for (int i = tid; i < n_tok * Dp; i += DS_NT) {
            const int j = i / Dp, c = i % Dp;
            const size_t t = t0 + j;
            const bool ok = c < D;
            qs[j][c] = ok ? to_f32<T>(q[t * ldq + (size_t)g * D + c]) * qk_scale[t * 2 * G + g] : 0.f;
            ks[j][c] = ok ? to_f32<T>(k[t * ldk + (size_t)g * D + c]) * qk_scale[t * 2 * G + G + g] : 0.f;
        }
        for (int i = tid; i < n_tok * DS_VC; i += DS_NT) {
            const int j = i / DS_VC, c = v0 + i % DS_VC;
            vs[j][i % DS_VC] = c < V ? to_f32<T>(v[(size_t)(t0 + j) * ldv + (size_t)h * V + c]) : 0.f;
        }
        if (tid < n_tok) {
            gs[tid][0] = expf(gates[(size_t)(t0 + tid) * 2 * H + h]);
            gs[tid][1] = gates[(size_t)(t0 + tid) * 2 * H + H + h];
        }
        __syncthreads();
        for (int j = 0; j < n_tok; ++j) {
            const float decay = gs[j][0], beta = gs[j][1], vv = vs[j][vc];
            f32x4 k4[RR], q4[RR];
#pragma unroll
            for (int i = 0; i < RR; ++i) {
                k4[i] = *(const f32x4*)&ks[j][i * 64 + dg * 4];
                q4[i] = *(const f32x4*)&qs[j][i * 64 + dg * 4];
            }
            float pk = 0.f;
#pragma unroll
            for (int r = 0; r < PR; ++r) { S[r] *= decay; pk = fmaf(S[r], k4[r >> 2][r & 3], pk); }
            const float u = beta * (vv - row16_sum(pk));
            float po = 0.f;
#pragma unroll
            for (int r = 0; r < PR; ++r) { S[r] = fmaf(k4[r >> 2][r & 3], u, S[r]); po = fmaf(S[r], q4[r >> 2][r & 3], po); }
            po = row16_sum(po);
            if (dg == 0 && vok) out[(size_t)(t0 + j) * H * V + (size_t)h * V + vcol] = po;
        }
    }
#pragma unroll
    for (int r = 0; r < PR; ++r) {
        const int d = (r >> 2) * 64 + dg * 4 + (r & 3);
        if (d < D && vok) srow[(size_t)d * V + vcol] = S[r];
    }
}

// ------------------------------------------------------------------ steps of single tokens
// A workgroup of 256 threads takes 64 value columns of one head of one entry: thread (row, column group) holds rows
// row + 16 p and four columns, every load of the state in flight at once, 256 bytes of a row by 16 lanes.  Both sums over the
// key channels are taken over the old state,
//   u = beta (v - g S^T k),   o = g S^T q + (k.q) u,   S <- g S + k u^T,
// so there is one exchange across the workgroup between reading and writing the state.
template <typename T, int NP>
__global__ __launch_bounds__(256)
void delta_step_kernel(const T* __restrict__ q, const T* __restrict__ k, const T* __restrict__ v, int ldq, int ldk, int ldv,
                       const float* __restrict__ qk_scale, const float* __restrict__ gates, float* __restrict__ state,
                       const int* __restrict__ seq_slots, float* __restrict__ out, int H, int G, int D, int V) {
    __shared__ float qs[16 * NP], ks[16 * NP];
    __shared__ f32x4 part[4][2][16];
    const int t = blockIdx.x, h = blockIdx.y, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    const int cg = tid & 15, row = tid >> 4, col = blockIdx.z * 64 + cg * 4;
    const int g = h / (H / G);
    const bool cok = col < V;                                   // (V is a multiple of four)
    float* sbase = state + ((size_t)seq_slots[t] * H + h) * (size_t)D * V + col;
    f32x4 S[NP];
#pragma unroll
    for (int p = 0; p < NP; ++p) {
        const int d = row + 16 * p;
        S[p] = cok && d < D ? *(const f32x4*)(sbase + (size_t)d * V) : f32x4{0.f, 0.f, 0.f, 0.f};
    }
    const float fq = qk_scale[(size_t)t * 2 * G + g], fk = qk_scale[(size_t)t * 2 * G + G + g];
    const float decay = expf(gates[(size_t)t * 2 * H + h]), beta = gates[(size_t)t * 2 * H + H + h];
    for (int c = tid; c < 16 * NP; c += 256) {
        qs[c] = c < D ? to_f32<T>(q[(size_t)t * ldq + (size_t)g * D + c]) * fq : 0.f;
        ks[c] = c < D ? to_f32<T>(k[(size_t)t * ldk + (size_t)g * D + c]) * fk : 0.f;
    }
    f32x4 vv = {0.f, 0.f, 0.f, 0.f};
    if (cok) {
        const T* vr = v + (size_t)t * ldv + (size_t)h * V + col;
#pragma unroll
        for (int i = 0; i < 4; ++i) vv[i] = to_f32<T>(vr[i]);
    }
    __syncthreads();
    f32x4 pk = {0.f, 0.f, 0.f, 0.f}, pq = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int p = 0; p < NP; ++p) {
        const float kd = ks[row + 16 * p], qd = qs[row + 16 * p];
#pragma unroll
        for (int i = 0; i < 4; ++i) { pk[i] = fmaf(S[p][i], kd, pk[i]); pq[i] = fmaf(S[p][i], qd, pq[i]); }
    }
    float kq = 0.f;
    for (int c = lane; c < 16 * NP; c += 64) kq = fmaf(ks[c], qs[c], kq);
    kq = wave_sum(kq);
#pragma unroll
    for (int i = 0; i < 4; ++i) { pk[i] = rows4_sum(pk[i]); pq[i] = rows4_sum(pq[i]); }
    if (lane < 16) { part[wave][0][lane] = pk; part[wave][1][lane] = pq; }
    __syncthreads();
    pk = part[0][0][cg] + part[1][0][cg] + part[2][0][cg] + part[3][0][cg];
    pq = part[0][1][cg] + part[1][1][cg] + part[2][1][cg] + part[3][1][cg];
    f32x4 u, o;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
        u[i] = beta * (vv[i] - decay * pk[i]);
        o[i] = fmaf(decay, pq[i], kq * u[i]);
    }
    if (!cok) return;
    if (row == 0) *(f32x4*)(out + (size_t)t * H * V + (size_t)h * V + col) = o;
#pragma unroll
    for (int p = 0; p < NP; ++p) {
        const int d = row + 16 * p;
        if (d >= D) continue;
        const float kd = ks[d];
        f32x4 s;
#pragma unroll
        for (int i = 0; i < 4; ++i) s[i] = fmaf(kd, u[i], decay * S[p][i]);
        *(f32x4*)(sbase + (size_t)d * V) = s;
    }
}

extern "C" int spite_delta_scan(const void* q, const void* k, const void* v, int ldq, int ldk, int ldv, int dtype, const float* qk_scale,
                                const float* gates, float* state, int n_slots, const int* cu_seqlens, const int* seq_slots, int n_seqs,
                                float* out, int H, int G, int D, int V, int single, hipStream_t st) {
    SP_REQUIRE(n_seqs >= 0 && H > 0 && G > 0 && H % G == 0 && D > 0 && V > 0 && n_slots > 0, "delta_scan: bad sizes H=%d G=%d D=%d V=%d", H, G, D, V);
    SP_REQUIRE(D <= DR_MAXD, "delta_scan: %d key channels a head (at most %d)", D, DR_MAXD);
    SP_REQUIRE(ldq >= G * D && ldk >= G * D && ldv >= H * V, "delta_scan: rows shorter than the heads");
    SP_REQUIRE(H <= 65535 && (V + DS_VC - 1) / DS_VC <= 65535, "delta_scan: too many heads or value columns");
    SP_REQUIRE(dtype == SP_F32 || dtype == SP_BF16, "delta_scan: unknown dtype %d", dtype);
    if (n_seqs == 0) return 0;
    if (single && V % 4 == 0 && ((uintptr_t)state & 15) == 0 && ((uintptr_t)out & 15) == 0) {
        const dim3 grid(n_seqs, H, (V + 63) / 64);
#define DR_STEP(T, NP) delta_step_kernel<T, NP><<<grid, 256, 0, st>>>((const T*)q, (const T*)k, (const T*)v, ldq, ldk, ldv, qk_scale, gates, state, \
        seq_slots, out, H, G, D, V)
#define DR_STEPS(T) do { if (D <= 64) DR_STEP(T, 4); else if (D <= 128) DR_STEP(T, 8); else DR_STEP(T, 16); } while (0)
        if (dtype == SP_F32) DR_STEPS(float); else DR_STEPS(bf16);
#undef DR_STEPS
#undef DR_STEP
        SP_LAUNCH_CHECK("delta_step");
        return 0;
    }
    const dim3 grid(n_seqs, H, (V + DS_VC - 1) / DS_VC);
#define DR_SCAN(T, RR) delta_scan_kernel<T, RR><<<grid, DS_NT, 0, st>>>((const T*)q, (const T*)k, (const T*)v, ldq, ldk, ldv, qk_scale, gates, state, \
    cu_seqlens, seq_slots, out, H, G, D, V)
#define DR_SCANS(T) do { if (D <= 64) DR_SCAN(T, 1); else if (D <= 128) DR_SCAN(T, 2); else DR_SCAN(T, 4); } while (0)
    if (dtype == SP_F32) DR_SCANS(float); else DR_SCANS(bf16);
#undef DR_SCANS
#undef DR_SCAN
    SP_LAUNCH_CHECK("delta_scan");
    return 0;
}
