// jl_scan.hip — linear recurrence with one decay per head (and token): S_t = a_t S_(t-1) + k_t (u_t v_t)^T, o_t = S_t^T q_t + skip v_t.
// Fixed decays are lightning attention, decays and step sizes from a projection (u = softplus, a = exp(-exp(A_log) u)) are the state-space
// duality of Mamba-2; one float state [D, Dv] per (request slot, head).
#include "jl_common.h"

// ---- token by token: decoded tokens, short portions, float activations ----------------------------------------------------------------------
// The columns of S never interact, so a workgroup is ONE wavefront that owns 32 columns of one head's state (grid.y walks the head's
// columns): two adjacent lanes per column, each with DMAX / 2 consecutive rows in registers.  Rows of S are read and written as 128
// consecutive bytes.  Eight tokens at a time go through LDS; the next group's inputs travel while the current one is worked on.
constexpr int SC_TT = 8, SC_COLS = 32;
// silu in the activations' dtype: both forms of the recurrence see the same q, k and v, however a prompt is cut
template <typename T> __device__ __forceinline__ float silu_as(float z) {
    T t;
    st_f(&t, silu_f(z));
    return ld_f(&t);
}

template <typename T, int DMAX>
__global__ __launch_bounds__(64) void scan_kernel(jl_scan_args a) {
    constexpr int DPER = DMAX / 2, PRE = SC_TT * DMAX / 64, ROW = DMAX + 8;
    __shared__ __attribute__((aligned(16))) float qs[SC_TT * ROW], ks[SC_TT * ROW];
    __shared__ float as[SC_TT], us[SC_TT];
    auto at = [](int tt, int d) { return tt * ROW + d + (d / DPER) * 4; };      // the two lanes of a column read different banks
    const int H = a.H, D = a.D, Dv = a.Dv;
    const int b = blockIdx.x / H, h = blockIdx.x - b * H, kh = h / (H / a.G);
    const int row0 = a.seq[4 * b], cnt = a.seq[4 * b + 1], pos0 = a.seq[4 * b + 2], slot = a.seq[4 * b + 3];
    if (cnt <= 0) return;
    const int lane = threadIdx.x, j = blockIdx.y * SC_COLS + (lane >> 1), sub = lane & 1, d0 = sub * DPER;
    const bool live = j < Dv;
    const T *src = (const T *)a.src, *dtp = (const T *)a.dt;
    const bool fixed = a.decay != nullptr, act = a.act == JL_ACT_SILU;
    const float gamma = fixed ? a.decay[h] : 0.f, rate = fixed ? 0.f : -expf(a.A_log[h]), bias = fixed ? 0.f : a.dt_bias[h];
    const float skip = a.skip ? a.skip[h] : 0.f;
    float *sp = a.state + ((int64_t)slot * H + h) * D * Dv;
    float S[DPER];
#pragma unroll
    for (int i = 0; i < DPER; ++i) S[i] = (live && d0 + i < D && pos0 > 0) ? sp[(int64_t)(d0 + i) * Dv + j] : 0.f;
    float pq[PRE], pk[PRE], pv[SC_TT], pd = 0.f;
    auto fetch = [&](int t0) {
        const int nt = cnt - t0 < SC_TT ? cnt - t0 : SC_TT;
#pragma unroll
        for (int i = 0; i < PRE; ++i) {
            const int e = i * 64 + lane, tt = e / DMAX, d = e - tt * DMAX;
            pq[i] = pk[i] = 0.f;
            if (tt < nt && d < D) {
                const T *row = src + (int64_t)(row0 + t0 + tt) * a.ld + kh * D + d;
                pq[i] = ld_f(row + a.q_col);
                pk[i] = ld_f(row + a.k_col);
            }
        }
#pragma unroll
        for (int tt = 0; tt < SC_TT; ++tt) pv[tt] = (tt < nt && live) ? ld_f(src + (int64_t)(row0 + t0 + tt) * a.ld + a.v_col + (int64_t)h * Dv + j) : 0.f;
        if (!fixed && lane < nt) pd = ld_f(dtp + (int64_t)(row0 + t0 + lane) * a.dt_ld + a.dt_col + h);
    };
    fetch(0);
    for (int t0 = 0; t0 < cnt; t0 += SC_TT) {
        const int nt = cnt - t0 < SC_TT ? cnt - t0 : SC_TT;
        __syncthreads();                                        // the group before has been read
#pragma unroll
        for (int i = 0; i < PRE; ++i) {
            const int e = i * 64 + lane, tt = e / DMAX, d = e - tt * DMAX;
            if (tt < nt) {
                qs[at(tt, d)] = act ? silu_as<T>(pq[i]) : pq[i];
                ks[at(tt, d)] = act ? silu_as<T>(pk[i]) : pk[i];
            }
        }
        if (lane < nt) {
            const float u = fixed ? 1.0f : softplus_f(pd + bias);
            us[lane] = u;
            as[lane] = fixed ? gamma : expf(rate * u);
        }
        float v[SC_TT];
#pragma unroll
        for (int tt = 0; tt < SC_TT; ++tt) v[tt] = act ? silu_as<T>(pv[tt]) : pv[tt];
        __syncthreads();
        if (t0 + SC_TT < cnt) fetch(t0 + SC_TT);                // in flight while this group's steps run
#pragma unroll
        for (int tt = 0; tt < SC_TT; ++tt) {
            if (tt < nt) {
                const float *qp = qs + tt * ROW + d0 + sub * 4, *kp = ks + tt * ROW + d0 + sub * 4;
                const float g = as[tt], u = us[tt] * v[tt];
                float acc[4] = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
                for (int i = 0; i < DPER; i += 4) {
                    const float4 k4 = *(const float4 *)(kp + i), q4 = *(const float4 *)(qp + i);
                    S[i] = g * S[i] + k4.x * u;             acc[0] += S[i] * q4.x;
                    S[i + 1] = g * S[i + 1] + k4.y * u;     acc[1] += S[i + 1] * q4.y;
                    S[i + 2] = g * S[i + 2] + k4.z * u;     acc[2] += S[i + 2] * q4.z;
                    S[i + 3] = g * S[i + 3] + k4.w * u;     acc[3] += S[i + 3] * q4.w;
                }
                float o = (acc[0] + acc[1]) + (acc[2] + acc[3]);
                o += __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(o), 0xB1, 0xF, 0xF, true));      // quad_perm [1, 0, 3, 2]: the column's other lane
                if (live && sub == 0) a.out[(int64_t)(row0 + t0 + tt) * ((int64_t)H * Dv) + (int64_t)h * Dv + j] = o + skip * v[tt];
            }
        }
    }
    if (live)
#pragma unroll
        for (int i = 0; i < DPER; ++i)
            if (d0 + i < D) sp[(int64_t)(d0 + i) * Dv + j] = S[i];
}

template <typename T> static int scan_launch(const jl_scan_args &a, hipStream_t st) {
    const dim3 grid((unsigned)(a.B * a.H), (unsigned)((a.Dv + SC_COLS - 1) / SC_COLS));
    if (a.D <= 32) scan_kernel<T, 32><<<grid, 64, 0, st>>>(a);
    else if (a.D <= 64) scan_kernel<T, 64><<<grid, 64, 0, st>>>(a);
    else if (a.D <= 128) scan_kernel<T, 128><<<grid, 64, 0, st>>>(a);
    else scan_kernel<T, 256><<<grid, 64, 0, st>>>(a);
    return jl_check_launch("scan_kernel");
}

// ---- long portions on the matrix cores (bfloat16): pieces side by side, 64 tokens at a time --------------------------------------------------
// With L_t the running sum of log a inside a group of 64 tokens, the recurrence of the group is three products:
//   o_i = exp(L_i) S^T q_i + sum_{j <= i} (q_i . k_j) exp(L_i - L_j) u_j v_j,        S <- exp(L_end) S + sum_j k_j (exp(L_end - L_j) u_j v_j)^T.
// A request's portion is cut into pieces (whole groups, except the last) that run side by side in three launches: every piece's own
// contribution to the state from a zero state (CH_LOCAL, not for a request's last piece), scan_join_kernel (the state every piece starts
// from), outputs (CH_OUT; the last piece leaves the request's final state in its slot).  A workgroup of four wavefronts owns 64 columns of one
// head's state and walks its piece's groups with the state in accumulators; the next group's rows travel while the current one is multiplied.
// q, k and v enter the products as bfloat16 (what the projection, the convolution and their activation give); everything else stays float
// and crosses the matrix cores as the sum of THREE bfloat16 numbers, which hold all 24 bits of it: the state, the decayed weights of a pair,
// the decayed values.  Accumulator r of lane l of a 32 x 32 product is row 8 (r / 4) + 4 (l / 32) + r % 4, column l % 32; lane l supplies row (A) or column
// (B) l % 32 with depths 8 (l / 32) .. + 7 of a 16-deep step.
typedef __bf16 ch_bf16x8 __attribute__((ext_vector_type(8)));
typedef __bf16 ch_bf16x4 __attribute__((ext_vector_type(4)));
typedef float ch_f32x4 __attribute__((ext_vector_type(4)));
typedef float ch_f32x16 __attribute__((ext_vector_type(16)));
constexpr int CH_T = 64, CH_C = 64, CH_THREADS = 256, CH_TROW = CH_T, CH_PROW = CH_T + 8;
constexpr int CH_TERMS = 3;
constexpr int CH_OUT = 0, CH_LOCAL = 1;

__device__ __forceinline__ ch_f32x16 ch_mfma(const bf16_t *a, const bf16_t *b, ch_f32x16 c) {
    return __builtin_amdgcn_mfma_f32_32x32x16_bf16(*(const ch_bf16x8 *)a, *(const ch_bf16x8 *)b, c, 0, 0, 0);
}
__device__ __forceinline__ uint2 ch_round4(const float (&v)[4]) {
    const ch_f32x4 f = {v[0], v[1], v[2], v[3]};
    return __builtin_bit_cast(uint2, __builtin_convertvector(f, ch_bf16x4));
}
// four floats as the sum of CH_TERMS bfloat16 numbers each, term x of them at dst + x * stride
__device__ __forceinline__ void ch_split4(float (&v)[4], bf16_t *dst, int stride) {
#pragma unroll
    for (int x = 0; x < CH_TERMS; ++x) {
        const uint2 w = ch_round4(v);
        *(uint2 *)(dst + x * stride) = w;
        v[0] -= __uint_as_float(w.x << 16); v[1] -= __uint_as_float(w.x & 0xffff0000u); v[2] -= __uint_as_float(w.y << 16); v[3] -= __uint_as_float(w.y & 0xffff0000u);
    }
}
__device__ __forceinline__ uint2 ch_silu4(uint2 w) {
    float v[4] = {__uint_as_float(w.x << 16), __uint_as_float(w.x & 0xffff0000u), __uint_as_float(w.y << 16), __uint_as_float(w.y & 0xffff0000u)};
#pragma unroll
    for (int i = 0; i < 4; ++i) v[i] *= __builtin_amdgcn_rcpf(1.0f + __expf(-v[i]));          // rounded to bfloat16 next
    return ch_round4(v);
}
// a row of 64 tokens of a transposed tile, eight tokens (16 bytes) at a time in an order that depends on the row: writers spread over rows and
// readers of 16 consecutive rows meet different banks
__device__ __forceinline__ int ch_tr(int row, int t) { return row * CH_TROW + ((((t >> 3) ^ (row >> 1) ^ (row >> 4)) & 7) << 3) + (t & 7); }
// two tokens' four values, turned into four rows' two tokens
__device__ __forceinline__ void ch_turn(bf16_t *dst, int row, int t, uint2 a, uint2 b) {
    *(uint32_t *)(dst + ch_tr(row, t)) = (a.x & 0xffffu) | (b.x << 16);
    *(uint32_t *)(dst + ch_tr(row + 1, t)) = (a.x >> 16) | (b.x & 0xffff0000u);
    *(uint32_t *)(dst + ch_tr(row + 2, t)) = (a.y & 0xffffu) | (b.y << 16);
    *(uint32_t *)(dst + ch_tr(row + 3, t)) = (a.y >> 16) | (b.y & 0xffff0000u);
}

static constexpr size_t ch_lds_bytes(int DP, bool out) {
    return 2 * ((size_t)DP * CH_TROW + CH_C * CH_TROW + CH_TERMS * CH_T * CH_PROW + (out ? 2 * CH_T * (DP + 8) + CH_TERMS * CH_C * (DP + 8) : 0)) + 3 * CH_T * 4;
}

template <int DP, int MODE>
__global__ __launch_bounds__(CH_THREADS) void scan_chunk_kernel(jl_scan_args a) {
    extern __shared__ __attribute__((aligned(16))) char smem[];
    constexpr int QROW = DP + 8, UD = DP / 4, KIT = 32 * UD / CH_THREADS, VIT = 2, NS = DP >= 64 ? DP / 64 : 1, PT = CH_T * CH_PROW, ST = CH_C * QROW;
    constexpr bool OUT = MODE == CH_OUT;
    const int H = a.H, D = a.D, Dv = a.Dv;
    const int piece = blockIdx.x, h = blockIdx.y, kh = h / (H / a.G), c_base = blockIdx.z * CH_C;
    const int row0 = a.chunk_rec[4 * piece], cnt = a.chunk_rec[4 * piece + 1], slot = a.chunk_rec[4 * piece + 2], last = a.chunk_rec[4 * piece + 3];
    if (cnt <= 0 || (!OUT && last)) return;
    bf16_t *KT = (bf16_t *)smem;                                    // [DP][64] keys, turned
    bf16_t *VT = KT + DP * CH_TROW;                                 // [64][64] values, turned
    bf16_t *Ps = VT + CH_C * CH_TROW;                               // terms x [64][72] weights of the pairs; then the decayed values (turned)
    bf16_t *Qs = Ps + CH_TERMS * PT, *Ks = Qs + CH_T * QROW;        // [64][DP + 8]
    bf16_t *Ss = Ks + CH_T * QROW;                                  // terms x [64][DP + 8] the state, turned
    float *Ls = (float *)(OUT ? Ss + CH_TERMS * ST : Qs);           // [64] running log decay
    float *us = Ls + CH_T, *es = us + CH_T;                         // [64] u; [64] exp(L_end - L) u
    const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63, l32 = lane & 31, hi = lane >> 5, w0 = wave & 1, w1 = wave >> 1;
    const bf16_t *src = (const bf16_t *)a.src, *dtp = (const bf16_t *)a.dt;
    const bool fixed = a.decay != nullptr, act = a.act == JL_ACT_SILU;
    const float glog = fixed ? fmaxf(logf(a.decay[h]), -1e30f) : 0.f, rate = fixed ? 0.f : -expf(a.A_log[h]), bias = fixed ? 0.f : a.dt_bias[h];
    const float skip = a.skip ? a.skip[h] : 0.f;

    // the state: wavefront (w1, w0) has rows 32 (w1 + 2 x) .. + 31 of columns 32 w0 .. + 31
    ch_f32x16 S[NS];
    const int sc = c_base + 32 * w0 + l32;
    const float *sp = a.scratch + ((int64_t)piece * H + h) * D * Dv;
#pragma unroll
    for (int x = 0; x < NS; ++x)
#pragma unroll
        for (int r = 0; r < 16; ++r) {
            const int d = 32 * (w1 + 2 * x) + 8 * (r >> 2) + 4 * hi + (r & 3);
            S[x][r] = (OUT && d < D && sc < Dv) ? sp[(int64_t)d * Dv + sc] : 0.f;
        }
    auto state_out = [&]() {                                        // the state in LDS
#pragma unroll
        for (int x = 0; x < NS; ++x) {
            if (32 * (w1 + 2 * x) >= DP) continue;
#pragma unroll
            for (int g = 0; g < 4; ++g) {
                float v[4] = {S[x][4 * g], S[x][4 * g + 1], S[x][4 * g + 2], S[x][4 * g + 3]};
                ch_split4(v, Ss + (32 * w0 + l32) * QROW + 32 * (w1 + 2 * x) + 8 * g + 4 * hi, ST);
            }
        }
    };
    if (OUT) state_out();

    uint2 rq[KIT][2], rk[KIT][2], rv[VIT][2];
    float rd = 0.f;
    auto fetch = [&](int t0) {
        const int nt = cnt - t0;
        const bf16_t *base = src + (int64_t)(row0 + t0) * a.ld;
#pragma unroll
        for (int it = 0; it < KIT; ++it) {
            const int e = tid + it * CH_THREADS, p = e / UD, d = (e - p * UD) * 4;
#pragma unroll
            for (int y = 0; y < 2; ++y) {
                rk[it][y] = make_uint2(0, 0);
                if (OUT) rq[it][y] = make_uint2(0, 0);
                if (2 * p + y < nt && d < D) {
                    const bf16_t *row = base + (int64_t)(2 * p + y) * a.ld + kh * D + d;
                    rk[it][y] = *(const uint2 *)(row + a.k_col);
                    if (OUT) rq[it][y] = *(const uint2 *)(row + a.q_col);
                }
            }
        }
#pragma unroll
        for (int it = 0; it < VIT; ++it) {
            const int e = tid + it * CH_THREADS, p = e >> 4, c = c_base + (e & 15) * 4;
#pragma unroll
            for (int y = 0; y < 2; ++y) {
                rv[it][y] = make_uint2(0, 0);
                if (2 * p + y < nt && c < Dv) rv[it][y] = *(const uint2 *)(base + (int64_t)(2 * p + y) * a.ld + a.v_col + (int64_t)h * Dv + c);
            }
        }
        if (wave == 0 && !fixed) rd = lane < nt ? ld_f(dtp + (int64_t)(row0 + t0 + lane) * a.dt_ld + a.dt_col + h) : 0.f;
    };
    fetch(0);
    float l_all = 0.f;                                              // log decay of the piece up to here
    for (int t0 = 0; t0 < cnt; t0 += CH_T) {
        const int nt = cnt - t0 < CH_T ? cnt - t0 : CH_T;
        __syncthreads();                                            // the group before has been read; the state is in LDS
#pragma unroll
        for (int it = 0; it < KIT; ++it) {
            const int e = tid + it * CH_THREADS, p = e / UD, d = (e - p * UD) * 4;
            if (act) {
#pragma unroll
                for (int y = 0; y < 2; ++y) {
                    rk[it][y] = ch_silu4(rk[it][y]);                // silu(0) = 0: rows and columns beyond the tile stay zero
                    if (OUT) rq[it][y] = ch_silu4(rq[it][y]);
                }
            }
            ch_turn(KT, d, 2 * p, rk[it][0], rk[it][1]);
            if (OUT) {
#pragma unroll
                for (int y = 0; y < 2; ++y) {
                    *(uint2 *)(Ks + (2 * p + y) * QROW + d) = rk[it][y];
                    *(uint2 *)(Qs + (2 * p + y) * QROW + d) = rq[it][y];
                }
            }
        }
#pragma unroll
        for (int it = 0; it < VIT; ++it) {
            const int e = tid + it * CH_THREADS, p = e >> 4, c = (e & 15) * 4;
            if (act) {
                rv[it][0] = ch_silu4(rv[it][0]);
                rv[it][1] = ch_silu4(rv[it][1]);
            }
            ch_turn(VT, c, 2 * p, rv[it][0], rv[it][1]);
        }
        if (wave == 0) {                                            // a token per lane: step size, running log decay
            const bool in = lane < nt;
            const float u = !in ? 0.f : fixed ? 1.0f : softplus_f(rd + bias);
            float l = !in ? 0.f : fixed ? glog : rate * u;
#pragma unroll
            for (int off = 1; off < 64; off <<= 1) {
                const float y = __shfl_up(l, off, 64);
                if (lane >= off) l += y;
            }
            const float end = __shfl(l, 63, 64);
            Ls[lane] = l;
            us[lane] = u;
            es[lane] = expf(end - l) * u;
        }
        __syncthreads();
        if (t0 + CH_T < cnt) fetch(t0 + CH_T);                      // in flight while this group is multiplied
        const float l_end = Ls[CH_T - 1];
        l_all += l_end;
        if (OUT) {
            if (w0 <= w1) {                                         // scores, turned: keys 32 w0 .. of queries 32 w1 ..; keys behind every query are left out
                ch_f32x16 s;
#pragma unroll
                for (int r = 0; r < 16; ++r) s[r] = 0.f;
#pragma unroll
                for (int kk = 0; kk < DP; kk += 16) s = ch_mfma(Ks + (32 * w0 + l32) * QROW + kk + 8 * hi, Qs + (32 * w1 + l32) * QROW + kk + 8 * hi, s);
                const int i = 32 * w1 + l32;
                const float li = Ls[i];
#pragma unroll
                for (int g = 0; g < 4; ++g) {
                    const int j0 = 32 * w0 + 8 * g + 4 * hi;
                    float v[4];
#pragma unroll
                    for (int x = 0; x < 4; ++x) v[x] = j0 + x <= i ? s[4 * g + x] * (__expf(li - Ls[j0 + x]) * us[j0 + x]) : 0.f;
                    ch_split4(v, Ps + i * CH_PROW + j0, PT);
                }
            }
            __syncthreads();
            {   // outputs: queries 32 w1 .., columns 32 w0 ..
                ch_f32x16 o;
#pragma unroll
                for (int r = 0; r < 16; ++r) o[r] = 0.f;
                const int ai = (32 * w1 + l32) * QROW + 8 * hi, bi = (32 * w0 + l32) * QROW + 8 * hi;
#pragma unroll
                for (int kk = 0; kk < DP; kk += 16) {
#pragma unroll
                    for (int x = 0; x < CH_TERMS; ++x) o = ch_mfma(Qs + ai + kk, Ss + x * ST + bi + kk, o);
                }
#pragma unroll
                for (int r = 0; r < 16; ++r) o[r] *= __expf(Ls[32 * w1 + 8 * (r >> 2) + 4 * hi + (r & 3)]);
#pragma unroll
                for (int kk = 0; kk < CH_T; kk += 16) {
                    if (kk >= 32 && w1 == 0) continue;              // no key of the second half is visible to the first half's queries
                    const bf16_t *vp = VT + ch_tr(32 * w0 + l32, kk + 8 * hi);
#pragma unroll
                    for (int x = 0; x < CH_TERMS; ++x) o = ch_mfma(Ps + x * PT + (32 * w1 + l32) * CH_PROW + kk + 8 * hi, vp, o);
                }
                if (sc < Dv) {
#pragma unroll
                    for (int r = 0; r < 16; ++r) {
                        const int i = 32 * w1 + 8 * (r >> 2) + 4 * hi + (r & 3);
                        if (i < nt) {
                            float v = o[r];
                            if (a.skip) v += skip * ld_f(VT + ch_tr(32 * w0 + l32, i));
                            a.out[(int64_t)(row0 + t0 + i) * ((int64_t)H * Dv) + (int64_t)h * Dv + sc] = v;
                        }
                    }
                }
            }
            if (t0 + CH_T >= cnt && !last) break;                   // nobody reads this piece's final state: the next piece has its own
            __syncthreads();
        }
        {   // decayed values in the weights' place: column tid / 4, sixteen tokens
            const int c = tid >> 2, tq = (tid & 3) * 16;
#pragma unroll
            for (int x = 0; x < 4; ++x) {
                const int t = tq + 4 * x, o = ch_tr(c, t);
                float v[4];
                ld4_f(VT + o, v);
#pragma unroll
                for (int y = 0; y < 4; ++y) v[y] *= es[t + y];
                ch_split4(v, Ps + o, PT);
            }
        }
        __syncthreads();
        {
            const float g = expf(l_end);
#pragma unroll
            for (int x = 0; x < NS; ++x) {
                if (32 * (w1 + 2 * x) >= DP) continue;
#pragma unroll
                for (int r = 0; r < 16; ++r) S[x][r] *= g;
#pragma unroll
                for (int kk = 0; kk < CH_T; kk += 16) {
                    const bf16_t *kp = KT + ch_tr(32 * (w1 + 2 * x) + l32, kk + 8 * hi);
                    const int o = ch_tr(32 * w0 + l32, kk + 8 * hi);
#pragma unroll
                    for (int y = 0; y < CH_TERMS; ++y) S[x] = ch_mfma(kp, Ps + y * PT + o, S[x]);
                }
            }
            if (OUT && t0 + CH_T < cnt) state_out();                // its readers of this group are two barriers behind
        }
    }
    if (OUT && !last) return;
    float *dst = OUT ? a.state + ((int64_t)slot * H + h) * D * Dv : a.scratch + ((int64_t)piece * H + h) * D * Dv;
#pragma unroll
    for (int x = 0; x < NS; ++x)
#pragma unroll
        for (int r = 0; r < 16; ++r) {
            const int d = 32 * (w1 + 2 * x) + 8 * (r >> 2) + 4 * hi + (r & 3);
            if (32 * (w1 + 2 * x) < DP && d < D && sc < Dv) dst[(int64_t)d * Dv + sc] = S[x][r];
        }
    if (!OUT && tid == 0 && blockIdx.z == 0) a.scratch[(int64_t)a.chunks * H * D * Dv + (int64_t)piece * H + h] = l_all;
}

// The state every piece starts from, in place of its own contribution: S = the request's state (zero at position 0); for each piece in order
// its contribution is replaced by S, then S = exp(its log decay) S + contribution (a request's last piece has none: nobody reads on).
__global__ __launch_bounds__(256) void scan_join_kernel(jl_scan_args a) {
    const int b = blockIdx.x / a.H, h = blockIdx.x - b * a.H;
    const int p0 = a.req[4 * b], np = a.req[4 * b + 1], pos0 = a.req[4 * b + 2], slot = a.req[4 * b + 3];
    const int64_t ddv = (int64_t)a.D * a.Dv;
    const float *sp = a.state + ((int64_t)slot * a.H + h) * ddv, *ll = a.scratch + (int64_t)a.chunks * a.H * ddv;
    for (int64_t e = (int64_t)blockIdx.y * 256 + threadIdx.x; e < ddv; e += (int64_t)gridDim.y * 256) {
        float S = pos0 > 0 ? sp[e] : 0.f;
        float *lp = a.scratch + ((int64_t)p0 * a.H + h) * ddv + e;
        float local = np > 1 ? *lp : 0.f;
        for (int p = 0; p < np; ++p, lp += a.H * ddv) {
            const float next = p + 2 < np ? lp[a.H * ddv] : 0.f;    // on its way while this piece is joined
            *lp = S;
            if (p + 1 < np) S = expf(ll[(int64_t)(p0 + p) * a.H + h]) * S + local;
            local = next;
        }
    }
}

template <int DP> static int scan_chunk_launch(const jl_scan_args &a, hipStream_t st) {
    const dim3 grid((unsigned)a.chunks, (unsigned)a.H, (unsigned)((a.Dv + CH_C - 1) / CH_C));
    auto out = scan_chunk_kernel<DP, CH_OUT>;
    constexpr size_t lds = ch_lds_bytes(DP, true);
    if (lds > 64 * 1024) {
        hipError_t e = hipFuncSetAttribute((const void *)out, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
        if (e != hipSuccess) return jl_fail(JL_E_LAUNCH, "jl_linear_scan: cannot get %zu bytes of LDS: %s", lds, hipGetErrorString(e));
    }
    if (a.chunks > a.B) scan_chunk_kernel<DP, CH_LOCAL><<<grid, CH_THREADS, ch_lds_bytes(DP, false), st>>>(a);
    const int64_t ddv = (int64_t)a.D * a.Dv;
    scan_join_kernel<<<dim3((unsigned)(a.B * a.H), (unsigned)((ddv + 255) / 256 < 64 ? (ddv + 255) / 256 : 64)), 256, 0, st>>>(a);
    out<<<grid, CH_THREADS, lds, st>>>(a);
    return jl_check_launch("scan_chunk_kernel");
}

extern "C" int jl_linear_scan_chunked_ok(int dtype, int32_t D, int32_t Dv) { return dtype == JL_BF16 && D > 0 && D <= 128 && D % 4 == 0 && Dv > 0 && Dv % 4 == 0; }

extern "C" int jl_linear_scan(const jl_scan_args *ap, void *stream) {
    if (!ap) return jl_fail(JL_E_INVALID, "jl_linear_scan: null arguments");
    const jl_scan_args &a = *ap;
    if (a.B <= 0) return JL_OK;
    if (!a.src || !a.seq || !a.state || !a.out || (!a.decay && (!a.dt || !a.A_log || !a.dt_bias))) return jl_fail(JL_E_INVALID, "jl_linear_scan: null pointer");
    if (a.H <= 0 || a.G <= 0 || a.H % a.G || a.D <= 0 || a.D > 256 || a.Dv <= 0) return jl_fail(JL_E_INVALID, "jl_linear_scan: heads must be a multiple of the key heads, D <= 256");
    if (a.q_col < 0 || a.k_col < 0 || a.v_col < 0 || a.q_col + (int64_t)a.G * a.D > a.ld || a.k_col + (int64_t)a.G * a.D > a.ld || a.v_col + (int64_t)a.H * a.Dv > a.ld ||
        (!a.decay && (a.dt_col < 0 || a.dt_col + (int64_t)a.H > a.dt_ld)))
        return jl_fail(JL_E_INVALID, "jl_linear_scan: columns do not fit the rows");
    if (a.act != JL_ACT_SILU && a.act != JL_ACT_NONE) return jl_fail(JL_E_INVALID, "jl_linear_scan: unknown activation %d", a.act);
    hipStream_t st = (hipStream_t)stream;
    if (a.chunks > 0) {
        if (!a.chunk_rec || !a.req || !a.scratch) return jl_fail(JL_E_INVALID, "jl_linear_scan: pieces need their records and a scratch");
        if (!jl_linear_scan_chunked_ok(a.dtype, a.D, a.Dv) || a.ld % 4 || a.q_col % 4 || a.k_col % 4 || a.v_col % 4 || (uintptr_t)a.src % 8)
            return jl_fail(JL_E_INVALID, "jl_linear_scan: pieces take bfloat16, D a multiple of four up to 128, Dv, columns and rows in multiples of four");
        if (a.D <= 32) return scan_chunk_launch<32>(a, st);
        if (a.D <= 64) return scan_chunk_launch<64>(a, st);
        return scan_chunk_launch<128>(a, st);
    }
    JL_DISPATCH(a.dtype, return scan_launch<T>(a, st));
    return JL_OK;
}
