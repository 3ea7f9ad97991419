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
template <typename T>
__device__ __forceinline__ void delta_gate(const T* raw_a, int lda, const T* raw_b, int ldb, const float* a_log, const float* dt_bias,
                                           float* gates, size_t t, int h, int H) {
    const float z = to_f32<T>(raw_a[t * lda + h]) + dt_bias[h];
    const float step = z > 20.f ? z + log1pf(expf(-z)) : log1pf(expf(z));           // softplus
    gates[t * 2 * H + h] = -expf(a_log[h]) * step;
    gates[t * 2 * H + H + h] = 1.0f / (1.0f + expf(-to_f32<T>(raw_b[t * ldb + h])));
}

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
    for (int h = lane; h < H; h += 64) delta_gate(raw_a, lda, raw_b, ldb, a_log, dt_bias, gates, t, h, H);
}

// The same for bfloat16 rows that a lane reads 16 bytes at a time: 16 lanes a q/k head, four heads a wave (the token's last
// items are its decays and step sizes).
__global__ __launch_bounds__(256)
void delta_gates_vec_kernel(const bf16* __restrict__ q, const bf16* __restrict__ k, int ldq, int ldk, const bf16* __restrict__ raw_a, int lda,
                            const bf16* __restrict__ raw_b, int ldb, const float* __restrict__ a_log, const float* __restrict__ dt_bias,
                            float q_scale, float eps, float* __restrict__ qk_scale, float* __restrict__ gates, int Tn, int G, int H, int D) {
    const int l = threadIdx.x & 15;
    const int per = G + (H + 15) / 16;                          // items a token: heads, then runs of 16 value heads
    const size_t item = (size_t)blockIdx.x * 16 + (threadIdx.x >> 4);
    if (item >= (size_t)Tn * per) return;
    const size_t t = item / per;
    const int g = (int)(item - t * per);
    if (g < G) {
        const bf16* qr = q + t * ldq + (size_t)g * D;
        const bf16* kr = k + t * ldk + (size_t)g * D;
        float sq = 0.f, sk = 0.f;
        for (int c = l * 8; c < D; c += 128) {
            const bf16x8 x = *(const bf16x8*)(qr + c), y = *(const bf16x8*)(kr + c);
#pragma unroll
            for (int e = 0; e < 8; ++e) { sq = fmaf((float)x[e], (float)x[e], sq); sk = fmaf((float)y[e], (float)y[e], sk); }
        }
        sq = row16_sum(sq);
        sk = row16_sum(sk);
        if (l == 0) {
            qk_scale[t * 2 * G + g] = q_scale / sqrtf(sq + eps);
            qk_scale[t * 2 * G + G + g] = 1.0f / sqrtf(sk + eps);
        }
        return;
    }
    const int h = (g - G) * 16 + l;
    if (h < H) delta_gate(raw_a, lda, raw_b, ldb, a_log, dt_bias, gates, t, h, H);
}

extern "C" int spite_delta_gates(const void* q, const void* k, int ldq, int ldk, const void* raw_a, int lda, const void* raw_b, int ldb,
                                 int dtype, const float* a_log, const float* dt_bias, float q_scale, float eps, float* qk_scale,
                                 float* gates, int T, int G, int H, int D, hipStream_t st) {
    SP_REQUIRE(T >= 0 && G > 0 && H > 0 && D > 0 && eps > 0.f, "delta_gates: bad sizes T=%d G=%d H=%d D=%d", T, G, H, D);
    SP_REQUIRE(ldq >= G * D && ldk >= G * D && lda >= H && ldb >= H, "delta_gates: rows shorter than the heads");
    if (T == 0) return 0;
    auto on16 = [](const void* p) { return ((uintptr_t)p & 15) == 0; };
    if (dtype == SP_BF16 && D % 8 == 0 && ldq % 8 == 0 && ldk % 8 == 0 && on16(q) && on16(k)) {
        const size_t n = (size_t)T * (G + (H + 15) / 16);
        SP_REQUIRE((n + 15) / 16 < (1u << 31), "delta_gates: too many heads");
        delta_gates_vec_kernel<<<(unsigned)((n + 15) / 16), 256, 0, st>>>((const bf16*)q, (const bf16*)k, ldq, ldk, (const bf16*)raw_a, lda,
            (const bf16*)raw_b, ldb, a_log, dt_bias, q_scale, eps, qk_scale, gates, T, G, H, D);
        SP_LAUNCH_CHECK("delta_gates");
        return 0;
    }
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

// ------------------------------------------------------------------ prompts, 32 tokens at a time, on the matrix units
// Within a chunk let G_t be the sum of log g over its tokens up to t, and write k_t = sk_t K_t, q_t = sq_t Q_t with the
// bfloat16 rows K, Q and their fp32 factors.  With the state S0 before the chunk,
//
//   u_t = beta_t (v_t - exp(G_t) S0^T k_t - sum_(s<t) exp(G_t - G_s) (k_t.k_s) u_s)
//   o_t = exp(G_t) S0^T q_t + sum_(s<=t) exp(G_t - G_s) (q_t.k_s) u_s
//   S   = exp(G_C) S0 + sum_s k_s (exp(G_C - G_s) u_s)^T
//
// so U = (I + A)^-1 R with the strictly lower triangular A_ts = beta_t exp(G_t - G_s) (k_t.k_s) and the rows
// R_t = beta_t v_t - beta_t exp(G_t) S0^T k_t.  Every exponent is a sum of logarithms of decays, never above 0.
//
// The first kernel forms, for every chunk and head at once, what does not depend on the state: (I + A)^-1 (by substitution),
// the matrix M of the second line and the factors of the rows; and K, Q and K^T in operand order, zeros behind a chunk's
// last token.  The second walks a head's chunks: it copies what the first has left straight into LDS, a chunk ahead.
//
// Nothing is rounded to bfloat16 on the way: K and Q *are* bfloat16 (their factors are applied to the products' rows),
// and an fp32 operand that meets them (the state, U) is split into three bfloat16 summands, 8 bits each, that add up to
// its 24 bits, so the products on the bfloat16 units are those of the fp32 numbers, summed in fp32; the small products
// whose both operands are fp32 (the inverse and M times 16 columns) run on the fp32 units.  Sums of logarithms are
// fp64, so that a difference of two of them keeps its bits however far both are from 0.
//
// Layouts.  A wave holds 16 value columns; a state tile (j, tt) of 16 rows is the key channels 32 j + 8 a + 4 tt + r in the
// register r of lane (a, column), so that the tiles' registers of a lane are the 8 consecutive channels that the lane
// supplies as the right operand of the next product: the state never moves between lanes.  The same holds for U (a
// lane's 4 + 4 tokens): its products take their tokens in the order in which the lanes hold them.
#define DC_C 32                                      // tokens a chunk
#define DC_NW 4                                      // waves a workgroup of the walk
#define DC_TILE 256                                  // floats of a 16 x 16 tile
#define DC_REC (7 * DC_TILE)                         // a chunk's and head's record: inverse and M, three tiles each
                                                     // (0,0) (1,0) (1,1), the rows' factors, exp(G_C); whole kilobytes
typedef unsigned dc_u4 __attribute__((ext_vector_type(4)));

// element (t, s) of a 16 x 16 tile in the order of the fp32 products' left operand: lane (s/4, t), register s%4
__device__ __forceinline__ int dc_pos(int t, int s) { return (((s >> 2) * 16 + t) << 2) + (s & 3); }

// 64 threads a (chunk, head).
template <int KD>
__global__ __launch_bounds__(64) __attribute__((amdgpu_waves_per_eu(3)))
void delta_chunk_prepare_kernel(const bf16* __restrict__ q, const bf16* __restrict__ k, int ldq, int ldk, const float* __restrict__ qk_scale,
                                const float* __restrict__ gates, const int* __restrict__ chunk_t0, const int* __restrict__ chunk_n,
                                bf16* __restrict__ ops, float* __restrict__ rec, int H, int G) {
    constexpr int D = 32 * KD, LK = D + 8;
    __shared__ __attribute__((aligned(16))) bf16 krow[DC_C * LK];
    __shared__ __attribute__((aligned(16))) float at[DC_C][DC_C + 4];       // A transposed: at[s][t]
    __shared__ float diag[2][16][17];
    __shared__ double gsum[DC_C];
    __shared__ float f_q[DC_C], f_k[DC_C], f_b[DC_C];
    const int c = blockIdx.x, h = blockIdx.y, lane = threadIdx.x, row = lane & 15, a = lane >> 4;
    const int t0 = chunk_t0[c], n = chunk_n[c], g = h / (H / G);
    // the tokens' factors; behind the chunk's last token: no decay, nothing written, nothing read
    {
        const int i = lane & 31;
        const bool ok = i < n;
        const size_t t = t0 + (ok ? i : 0);
        double s = ok ? (double)gates[t * 2 * H + h] : 0.0;
#pragma unroll
        for (int o = 1; o < 32; o <<= 1) { const double up = __shfl_up(s, o, 32); if (i >= o) s += up; }
        if (lane < 32) {
            gsum[i] = s;
            f_b[i] = ok ? gates[t * 2 * H + H + h] : 0.f;
            f_q[i] = ok ? qk_scale[t * 2 * G + g] : 0.f;
            f_k[i] = ok ? qk_scale[t * 2 * G + G + g] : 0.f;
        }
    }
    bf16x8 ka[2][KD], qa[2][KD];
#pragma unroll
    for (int ti = 0; ti < 2; ++ti)
#pragma unroll
        for (int j = 0; j < KD; ++j) {
            const int i = 16 * ti + row;
            const bool ok = i < n;
            const size_t t = t0 + (ok ? i : 0);
            const int d = 32 * j + 8 * a;
            const dc_u4 x = *(const dc_u4*)(k + t * ldk + (size_t)g * D + d), y = *(const dc_u4*)(q + t * ldq + (size_t)g * D + d);
            ka[ti][j] = __builtin_bit_cast(bf16x8, ok ? x : dc_u4{0, 0, 0, 0});
            qa[ti][j] = __builtin_bit_cast(bf16x8, ok ? y : dc_u4{0, 0, 0, 0});
            *(bf16x8*)(krow + i * LK + d) = ka[ti][j];
        }
    f32x4 kk[3], qk[3];                               // tiles (0,0) (1,0) (1,1)
#pragma unroll
    for (int x = 0; x < 3; ++x) { kk[x] = f32x4{0.f, 0.f, 0.f, 0.f}; qk[x] = kk[x]; }
#pragma unroll
    for (int j = 0; j < KD; ++j)
#pragma unroll
        for (int x = 0; x < 3; ++x) {
            const int ti = x > 0, tj = x > 1;
            kk[x] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(ka[ti][j], ka[tj][j], kk[x], 0, 0, 0);
            qk[x] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(qa[ti][j], ka[tj][j], qk[x], 0, 0, 0);
        }
    __syncthreads();
    float* out = rec + ((size_t)c * H + h) * DC_REC;
#pragma unroll
    for (int x = 0; x < 3; ++x) {
        const int ti = x > 0, tj = x > 1, s = 16 * tj + row;
        f32x4 av;
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            const int tl = 4 * a + r, t = 16 * ti + tl;
            const float ratio = t >= s ? expf((float)(gsum[t] - gsum[s])) * f_k[s] : 0.f;
            av[r] = t > s ? f_b[t] * f_k[t] * ratio * kk[x][r] : 0.f;
            out[3 * DC_TILE + x * DC_TILE + dc_pos(tl, row)] = f_q[t] * ratio * qk[x][r];
        }
        *(f32x4*)&at[s][16 * ti + 4 * a] = av;
    }
    if (lane < 32) {
        const float eg = expf((float)gsum[lane]);
        float* fr = out + 6 * DC_TILE;
        fr[lane] = f_b[lane];
        fr[DC_C + lane] = f_b[lane] * eg * f_k[lane];
        fr[2 * DC_C + lane] = eg * f_q[lane];
        fr[3 * DC_C + lane] = expf((float)(gsum[DC_C - 1] - gsum[lane])) * f_k[lane];
        if (lane == 0) fr[4 * DC_C] = expf((float)gsum[DC_C - 1]);
    }
    __syncthreads();
    // the inverse of the two diagonal tiles by substitution, lane (tile, column): x_t = [t = column] - sum_(s<t) A_ts x_s
    if (lane < 32) {
        float x[16];
#pragma unroll
        for (int t = 0; t < 16; ++t) x[t] = t == row ? 1.f : 0.f;
#pragma unroll
        for (int s = 0; s < 15; ++s) {
#pragma unroll
            for (int t4 = (s + 1) / 4; t4 < 4; ++t4) {
                const f32x4 w = *(const f32x4*)&at[16 * a + s][16 * a + t4 * 4];
#pragma unroll
                for (int r = 0; r < 4; ++r) if (t4 * 4 + r > s) x[t4 * 4 + r] = fmaf(-w[r], x[s], x[t4 * 4 + r]);
            }
            asm volatile("" ::: "memory");           // (the reads of later columns stay where they are: registers)
        }
#pragma unroll
        for (int t = 0; t < 16; ++t) {
            out[2 * a * DC_TILE + dc_pos(t, row)] = x[t];
            diag[a][t][row] = x[t];
        }
    }
    __syncthreads();
    // the tile below: - T11 (A10 T00)
    {
        f32x4 y = {0.f, 0.f, 0.f, 0.f}, z = y;
#pragma unroll
        for (int r = 0; r < 4; ++r) y = __builtin_amdgcn_mfma_f32_16x16x4f32(at[4 * a + r][16 + row], diag[0][4 * a + r][row], y, 0, 0, 0);
#pragma unroll
        for (int r = 0; r < 4; ++r) z = __builtin_amdgcn_mfma_f32_16x16x4f32(diag[1][row][4 * a + r], y[r], z, 0, 0, 0);
#pragma unroll
        for (int r = 0; r < 4; ++r) out[DC_TILE + dc_pos(4 * a + r, row)] = -z[r];
    }
    if (h % (H / G) == 0) {
        // the operands: K and Q as left operands as this wave holds them, then K^T as the left operand of the state's update:
        // lane (a, row) of tile (j, tt) holds channel 32 j + 8 (row/4) + 4 tt + row%4 of the tokens 4 a .. 4 a + 3 and 16 + 4 a ..
        bf16x8* dst = (bf16x8*)(ops + ((size_t)c * G + g) * (6 * KD * 512));
#pragma unroll
        for (int ti = 0; ti < 2; ++ti)
#pragma unroll
            for (int j = 0; j < KD; ++j) {
                dst[(ti * KD + j) * 64 + lane] = ka[ti][j];
                dst[(2 * KD + ti * KD + j) * 64 + lane] = qa[ti][j];
            }
#pragma unroll
        for (int x = 0; x < 2 * KD; ++x) {
            const int d = 32 * (x >> 1) + 8 * (row >> 2) + 4 * (x & 1) + (row & 3);
            bf16x8 o;
#pragma unroll
            for (int e = 0; e < 8; ++e) o[e] = krow[((e & 4) * 4 + 4 * a + (e & 3)) * LK + d];
            dst[(4 * KD + x) * 64 + lane] = o;
        }
    }
}

// The three bfloat16 summands of eight fp32 numbers: the upper halves of what is left, cut off, 8 bits at a time.
__device__ __forceinline__ void dc_split(const f32x4& x, const f32x4& y, bf16x8& hi, bf16x8& mid, bf16x8& lo) {
    dc_u4 h, m, l;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
        const float v0 = i < 2 ? x[2 * i & 3] : y[2 * i & 3], v1 = i < 2 ? x[(2 * i + 1) & 3] : y[(2 * i + 1) & 3];
        const float r0 = v0 - __uint_as_float(__float_as_uint(v0) & 0xffff0000u), r1 = v1 - __uint_as_float(__float_as_uint(v1) & 0xffff0000u);
        const float s0 = r0 - __uint_as_float(__float_as_uint(r0) & 0xffff0000u), s1 = r1 - __uint_as_float(__float_as_uint(r1) & 0xffff0000u);
        h[i] = __builtin_amdgcn_perm(__float_as_uint(v1), __float_as_uint(v0), 0x07060302u);     // two upper halves in one register
        m[i] = __builtin_amdgcn_perm(__float_as_uint(r1), __float_as_uint(r0), 0x07060302u);
        l[i] = __builtin_amdgcn_perm(__float_as_uint(s1), __float_as_uint(s0), 0x07060302u);
    }
    hi = __builtin_bit_cast(bf16x8, h);
    mid = __builtin_bit_cast(bf16x8, m);
    lo = __builtin_bit_cast(bf16x8, l);
}

// Four waves take 16 value columns each of one head of one entry and walk the entry's chunks; the next chunk's operands are
// on their way into the other LDS buffer while this one is computed.
template <int KD>
__global__ __launch_bounds__(64 * DC_NW) __attribute__((amdgpu_waves_per_eu(2)))
void delta_chunk_scan_kernel(const bf16* __restrict__ v, int ldv, const int* __restrict__ first_chunk, const int* __restrict__ chunk_t0,
                             const int* __restrict__ chunk_n, const bf16* __restrict__ ops, const float* __restrict__ rec,
                             float* __restrict__ state, const int* __restrict__ seq_slots, float* __restrict__ out, int H, int G, int V) {
    constexpr int D = 32 * KD, TILES = 6 * KD + 7;         // kilobytes a chunk: K, Q, K^T, the record
    __shared__ __attribute__((aligned(16))) dc_u4 lds[2][TILES * 64];
    const int e = blockIdx.x, h = blockIdx.y, wave = threadIdx.x >> 6, lane = threadIdx.x & 63, a = lane >> 4;
    const int g = h / (H / G), col0 = (blockIdx.z * DC_NW + wave) * 16 + (lane & 15);
    const bool cok = col0 < V;
    const int col = cok ? col0 : V - 1;                    // a lane without a column of its own reads the last one and writes none
    const int c_lo = first_chunk[e], c_hi = first_chunk[e + 1];
    if (c_lo >= c_hi) return;
    const int t_lo = chunk_t0[c_lo], t_hi = chunk_t0[c_hi - 1] + chunk_n[c_hi - 1];
    float* sbase = state + ((size_t)seq_slots[e] * H + h) * (size_t)D * V + col;
    f32x4 S[2 * KD];
#pragma unroll
    for (int x = 0; x < 2 * KD; ++x)
#pragma unroll
        for (int r = 0; r < 4; ++r) S[x][r] = sbase[(size_t)(32 * (x >> 1) + 8 * a + 4 * (x & 1) + r) * V];
    bf16 vn[2][4];
    const unsigned v_lane = 4u * a * (unsigned)ldv + col, o_lane = 4u * a * (unsigned)(H * V) + col;    // a lane's tokens 4 a ..
    // a chunk's operands into an LDS buffer (a wave a kilobyte at a time), its values into registers; tokens behind the last
    // one read that one's values, which their step size of zero takes out
#define DC_FETCH(c, buf)                                                                                                \
    {                                                                                                                   \
        const dc_u4* so = (const dc_u4*)(ops + ((size_t)(c) * G + g) * (6 * KD * 512)) + lane;                          \
        const dc_u4* sr = (const dc_u4*)(rec + ((size_t)(c) * H + h) * DC_REC) + lane;                                  \
        _Pragma("unroll")                                                                                               \
        for (int u = 0; u < (TILES + DC_NW - 1) / DC_NW; ++u) {                                                         \
            const int x = u * DC_NW + wave;                                                                             \
            if (x < TILES)                                                                                              \
                __builtin_amdgcn_global_load_lds((const __attribute__((address_space(1))) void*)(x < 6 * KD ? so + x * 64 : sr + (x - 6 * KD) * 64), \
                                                 (__attribute__((address_space(3))) void*)(lds[buf] + x * 64), 16, 0, 0); \
        }                                                                                                               \
        const int t0 = t_lo + ((c) - c_lo) * DC_C;                                                                      \
        if (t0 + DC_C <= t_hi) {                                                                                        \
            const bf16* vb = v + (size_t)t0 * ldv + (size_t)h * V;                                                      \
            _Pragma("unroll")                                                                                           \
            for (int x = 0; x < 8; ++x) vn[x >> 2][x & 3] = (vb + (size_t)(16 * (x >> 2) + (x & 3)) * ldv)[v_lane];      \
        } else {                                                                                                        \
            _Pragma("unroll")                                                                                           \
            for (int x = 0; x < 8; ++x) {                                                                               \
                const int t = t0 + 16 * (x >> 2) + 4 * a + (x & 3);                                                     \
                vn[x >> 2][x & 3] = v[(size_t)(t < t_hi ? t : t_hi - 1) * ldv + (size_t)h * V + col];                   \
            }                                                                                                           \
        }                                                                                                               \
    }
    // a chunk's results leave at the start of the next turn: the wait for a chunk's operands never waits for stores just issued
    f32x4 O[2];
#define DC_STORE(c)                                                                                                     \
    {                                                                                                                   \
        const int t0 = t_lo + ((c) - c_lo) * DC_C;                                                                      \
        if (t0 + DC_C <= t_hi) {                                                                                        \
            float* ob = out + ((size_t)t0 * H + h) * V;                                                                 \
            if (cok) {                                                                                                  \
                _Pragma("unroll")                                                                                       \
                for (int x = 0; x < 8; ++x) (ob + (size_t)(16 * (x >> 2) + (x & 3)) * H * V)[o_lane] = O[x >> 2][x & 3]; \
            }                                                                                                           \
        } else {                                                                                                        \
            _Pragma("unroll")                                                                                           \
            for (int x = 0; x < 8; ++x) {                                                                               \
                const int t = t0 + 16 * (x >> 2) + 4 * a + (x & 3);                                                     \
                if (t < t_hi && cok) out[(size_t)t * H * V + (size_t)h * V + col] = O[x >> 2][x & 3];                   \
            }                                                                                                           \
        }                                                                                                               \
    }
    DC_FETCH(c_lo, 0)
    for (int c = c_lo; c < c_hi; ++c) {
        const int buf = (c - c_lo) & 1;
        asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
        f32x4 vv[2];
#pragma unroll
        for (int x = 0; x < 8; ++x) vv[x >> 2][x & 3] = (float)vn[x >> 2][x & 3];
        __syncthreads();                                   // this chunk has come, the one before has been read
        if (c > c_lo) DC_STORE(c - 1)
        if (c + 1 < c_hi) DC_FETCH(c + 1, buf ^ 1)
        const bf16x8* kop = (const bf16x8*)lds[buf] + lane;
        const bf16x8* qop = kop + 2 * KD * 64;
        const bf16x8* ktop = qop + 2 * KD * 64;
        const f32x4* inv = (const f32x4*)(lds[buf] + 6 * KD * 64);
        const f32x4* mm = inv + 3 * 64;
        const f32x4* fr = mm + 3 * 64;                     // the rows' factors, four tokens each
        // S0^T k and S0^T q, the smallest summands first
        f32x4 R[2];
#pragma unroll
        for (int i = 0; i < 2; ++i) { R[i] = f32x4{0.f, 0.f, 0.f, 0.f}; O[i] = R[i]; }
#pragma unroll
        for (int j = 0; j < KD; ++j) {
            bf16x8 s3[3];
            dc_split(S[2 * j], S[2 * j + 1], s3[2], s3[1], s3[0]);
#pragma unroll
            for (int y = 0; y < 3; ++y)
#pragma unroll
                for (int i = 0; i < 2; ++i) {
                    R[i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kop[(i * KD + j) * 64], s3[y], R[i], 0, 0, 0);
                    O[i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(qop[(i * KD + j) * 64], s3[y], O[i], 0, 0, 0);
                }
        }
#pragma unroll
        for (int i = 0; i < 2; ++i) {
            const f32x4 b4 = fr[4 * i + a], c4 = fr[8 + 4 * i + a], e4 = fr[16 + 4 * i + a];
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                R[i][r] = b4[r] * vv[i][r] - c4[r] * R[i][r];
                O[i][r] *= e4[r];
            }
        }
        // U = (I + A)^-1 R, then O += M U
        f32x4 U[2];
#pragma unroll
        for (int i = 0; i < 2; ++i) U[i] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int x = 0; x < 3; ++x) {
            const int ti = x > 0, tj = x > 1;
            const f32x4 w = inv[x * 64 + lane];
#pragma unroll
            for (int r = 0; r < 4; ++r) U[ti] = __builtin_amdgcn_mfma_f32_16x16x4f32(w[r], R[tj][r], U[ti], 0, 0, 0);
        }
#pragma unroll
        for (int x = 0; x < 3; ++x) {
            const int ti = x > 0, tj = x > 1;
            const f32x4 w = mm[x * 64 + lane];
#pragma unroll
            for (int r = 0; r < 4; ++r) O[ti] = __builtin_amdgcn_mfma_f32_16x16x4f32(w[r], U[tj][r], O[ti], 0, 0, 0);
        }
        // S <- exp(G_C) S + K (factors U)^T
#pragma unroll
        for (int i = 0; i < 2; ++i) {
            const f32x4 f4 = fr[24 + 4 * i + a];
#pragma unroll
            for (int r = 0; r < 4; ++r) U[i][r] *= f4[r];
        }
        bf16x8 u3[3];
        dc_split(U[0], U[1], u3[2], u3[1], u3[0]);
        const float whole = fr[32][0];
#pragma unroll
        for (int x = 0; x < 2 * KD; ++x)
#pragma unroll
            for (int r = 0; r < 4; ++r) S[x][r] *= whole;
#pragma unroll
        for (int y = 0; y < 3; ++y)
#pragma unroll
            for (int x = 0; x < 2 * KD; ++x) S[x] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(ktop[x * 64], u3[y], S[x], 0, 0, 0);
    }
    DC_STORE(c_hi - 1)
#undef DC_STORE
#undef DC_FETCH
    if (!cok) return;
#pragma unroll
    for (int x = 0; x < 2 * KD; ++x)
#pragma unroll
        for (int r = 0; r < 4; ++r) sbase[(size_t)(32 * (x >> 1) + 8 * a + 4 * (x & 1) + r) * V] = S[x][r];
}

// Bytes of scratch for n_chunks chunks: the operands, then the records.
extern "C" size_t spite_delta_chunk_workspace(int n_chunks, int H, int G, int D) {
    return (size_t)n_chunks * ((size_t)G * 3 * D * DC_C * sizeof(bf16) + (size_t)H * DC_REC * sizeof(float));
}
extern "C" int spite_delta_chunk_tokens() { return DC_C; }

// chunks: int32 [n_seqs + 1] the first chunk of every entry, [n_chunks] the chunks' first tokens, [n_chunks] their lengths.
extern "C" int spite_delta_chunk(const void* q, const void* k, const void* v, int ldq, int ldk, int ldv, const float* qk_scale, const float* gates,
                                 float* state, int n_slots, const int* chunks, int n_chunks, const int* seq_slots, int n_seqs,
                                 void* scratch, float* out, int H, int G, int D, int V, hipStream_t st) {
    SP_REQUIRE(n_seqs >= 0 && n_chunks >= 0 && H > 0 && G > 0 && H % G == 0 && V > 0 && n_slots > 0, "delta_chunk: bad sizes H=%d G=%d V=%d", H, G, V);
    SP_REQUIRE(D == 32 || D == 64 || D == 96 || D == 128, "delta_chunk: %d key channels a head (32, 64, 96 or 128)", D);
    SP_REQUIRE(ldq >= G * D && ldk >= G * D && ldv >= H * V, "delta_chunk: rows shorter than the heads");
    SP_REQUIRE(H <= 65535 && V <= 65535, "delta_chunk: too many heads or value columns");
    auto on16 = [](const void* p) { return ((uintptr_t)p & 15) == 0; };
    SP_REQUIRE(ldq % 8 == 0 && ldk % 8 == 0 && on16(q) && on16(k) && on16(scratch), "delta_chunk: q and k rows must start on 16 bytes");
    if (n_seqs == 0 || n_chunks == 0) return 0;
    bf16* ops = (bf16*)scratch;
    float* rec = (float*)(ops + (size_t)n_chunks * G * 3 * D * DC_C);
    const int *first = chunks, *t0 = chunks + n_seqs + 1, *n = t0 + n_chunks;
#define DC_RUN(KD) do { \
        delta_chunk_prepare_kernel<KD><<<dim3(n_chunks, H), 64, 0, st>>>((const bf16*)q, (const bf16*)k, ldq, ldk, qk_scale, gates, t0, n, ops, rec, H, G); \
        SP_LAUNCH_CHECK("delta_chunk_prepare"); \
        delta_chunk_scan_kernel<KD><<<dim3(n_seqs, H, (V + 16 * DC_NW - 1) / (16 * DC_NW)), 64 * DC_NW, 0, st>>>( \
            (const bf16*)v, ldv, first, t0, n, ops, rec, state, seq_slots, out, H, G, V); } while (0)
    if (D == 32) DC_RUN(1); else if (D == 64) DC_RUN(2); else if (D == 96) DC_RUN(3); else DC_RUN(4);
#undef DC_RUN
    SP_LAUNCH_CHECK("delta_chunk");
    return 0;
}
