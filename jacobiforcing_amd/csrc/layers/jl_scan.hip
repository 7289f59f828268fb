// jl_scan.hip — linear recurrence with one decay per head (and token): S_t = a_t S_(t-1) + k_t (u_t v_t)^T, o_t = S_t^T q_t + skip v_t.
// Fixed decays are lightning attention, decays and step sizes from a projection (u = softplus, a = exp(-exp(A_log) u)) are the state-space
// duality of Mamba-2; one float state [D, Dv] per (request slot, head).
#include "jl_common.h"

// ---- token by token: decoded tokens, short portions, float activations ----------------------------------------------------------------------
// The columns of S never interact, so a workgroup is ONE wavefront that owns 32 columns of one head's state (grid.y walks the head's
// columns): two adjacent lanes per column, each with DMAX / 2 consecutive rows in registers.  Rows of S are read and written as 128
// consecutive bytes.  Eight tokens at a time go through LDS; the next group's inputs travel while the current one is worked on.
constexpr int SC_TT = 8, SC_COLS = 32;

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
                qs[at(tt, d)] = act ? silu_f(pq[i]) : pq[i];
                ks[at(tt, d)] = act ? silu_f(pk[i]) : pk[i];
            }
        }
        if (lane < nt) {
            const float u = fixed ? 1.0f : softplus_f(pd + bias);
            us[lane] = u;
            as[lane] = fixed ? gamma : expf(rate * u);
        }
        float v[SC_TT];
#pragma unroll
        for (int tt = 0; tt < SC_TT; ++tt) v[tt] = act ? silu_f(pv[tt]) : pv[tt];
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

extern "C" int jl_linear_scan_chunked_ok(int, int32_t, int32_t) { return 0; }

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
    if (a.chunks > 0) return jl_fail(JL_E_INVALID, "jl_linear_scan: sizes not taken in pieces");
    JL_DISPATCH(a.dtype, return scan_launch<T>(a, st));
    return JL_OK;
}
