// Skinny GEMM of the latent-attention family: y[m, n] = x[m, :] . W[n, :], one 16-row weight panel per workgroup, the panel's
// K range split over the workgroup's waves, batch rows in blocks of 16 * MT.  Same weight packing and wave structure as
// csrc/gemv.hip (a wave's weight load is one contiguous run per 16x32 tile, partial tiles meet in LDS), with the element type
// a template parameter and the epilogues of this family:
//   IN        the four projections that read the layer's one norm (query latent, key latent | key, gate, feed-forward up):
//             raw fp32 outputs plus per-panel sums of squares (the norms of the two latents need them), gelu on the last part
//   QUERY     query latent normalised in the operand load, heads written as unrotated | rotated; spare workgroups of the same
//             launch normalise, rotate and store the cache rows
//   LATENT    per head: query through the transposed key up-projection, next to the rotated part
//   GATED     per head: value up-projection of the attended latent, times the output gate
//   RESIDUAL  attention output and feed-forward down in one matrix, added to the fp32 residual
//   TOKEN     per-layer token input: gelu times the token's row of a table
#include "latent_common.h"

template <typename T, int XMODE>
__device__ __forceinline__ typename El<T>::Frag load_x(const void* x, int64_t off, float inv, const float* nw) {
    if constexpr (XMODE == TFL_X_T) {
        return load_frag((const T*)x + off);
    } else {
        const f32x8 v = *reinterpret_cast<const f32x8*>((const float*)x + off);
        typename El<T>::Frag f;
        if constexpr (XMODE == TFL_X_F32_NORM) {
            const f32x8 w = *reinterpret_cast<const f32x8*>(nw);
#pragma unroll
            for (int e = 0; e < 8; ++e) f[e] = (T)(v[e] * inv * w[e]);
        } else {
#pragma unroll
            for (int e = 0; e < 8; ++e) f[e] = (T)v[e];
        }
        return f;
    }
}

template <typename T, int XMODE, int EPI, int MT, int WAVES>
__global__ __launch_bounds__(WAVES * 64) void latent_gemm_kernel(const TflGemm a) {
    typedef typename El<T>::Frag Frag;
    constexpr int U = sizeof(T) == 2 ? 4 : 2;                // weight tiles in flight per wave and batch
    __shared__ f32x4 part[WAVES][MT][64];
    __shared__ float red[4];
    const int ppg = a.n >> 4, npan = ppg * a.groups;
    const int tid = threadIdx.x;
    if constexpr (EPI == TFL_EPI_QUERY) {
        if ((int)blockIdx.x >= npan) {                       // cache row of batch row m (256-thread part of the workgroup)
            const int m = blockIdx.y * (gridDim.x - npan) + blockIdx.x - npan;
            if (m >= a.rows) return;
            const int slot = a.slot[m];
            if (slot < 0 || slot >= a.cache_rows) return;
            int p = a.pos[m];
            p = p < 0 ? 0 : (p >= a.max_pos ? a.max_pos - 1 : p);
            const float* src = a.kv_raw + (int64_t)m * a.ld_kv;
            cache_row_256<T>([src](int c) { return src[c]; }, a.C, a.c_real, a.R, a.kv_norm_w, a.eps, a.cos + (int64_t)p * a.half,
                             a.sin + (int64_t)p * a.half, a.half, (T*)a.cache + (int64_t)slot * (a.C + a.R), (T*)nullptr, red);
            return;
        }
    }
    const int wave = tid >> 6, lane = tid & 63, g = lane >> 4, i = lane & 15;
    const int panel = blockIdx.x, grp = panel / ppg, pin = panel - grp * ppg;
    const int m0 = blockIdx.y * 16 * MT;
    const int chunks = a.k >> 5;
    const int per = (chunks + WAVES - 1) / WAVES;
    const int c_beg = wave * per, c_end = min(chunks, c_beg + per);
    const T* wp = (const T*)a.wp + (int64_t)panel * chunks * 512 + lane * 8;
    int64_t xoff[MT];
    float inv[MT];
#pragma unroll
    for (int t = 0; t < MT; ++t) {
        const int m = min(m0 + 16 * t + i, a.rows - 1);
        xoff[t] = (int64_t)m * a.ld_x + (int64_t)grp * a.x_group + 8 * g;
        inv[t] = 1.f;
        if constexpr (XMODE == TFL_X_F32_NORM) {             // the row's scale from the producer's per-panel sums of squares
            float s = 0.f;
            for (int p = g; p < a.ss_n; p += 4) s += a.ss_in[(int64_t)m * a.ss_ld + p];
            s += __shfl_xor(s, 16, 64);
            s += __shfl_xor(s, 32, 64);
            inv[t] = 1.0f / sqrtf(s / (float)a.k_real + a.eps);
        }
    }
    f32x4 acc[MT];
#pragma unroll
    for (int t = 0; t < MT; ++t) acc[t] = f32x4{0.f, 0.f, 0.f, 0.f};
    if (c_beg < c_end) {
        Frag w[U], wn[U];
        const int last = c_end - 1;
#pragma unroll
        for (int u = 0; u < U; ++u) w[u] = load_frag_stream(wp + (int64_t)min(c_beg + u, last) * 512);
        for (int c0 = c_beg; c0 < c_end; c0 += U) {
            Frag xv[U][MT];
#pragma unroll
            for (int u = 0; u < U; ++u) {
                const int c = min(c0 + u, last);
#pragma unroll
                for (int t = 0; t < MT; ++t)
                    xv[u][t] = load_x<T, XMODE>(a.x, xoff[t] + 32 * (int64_t)c, inv[t], (const float*)a.norm_w + 32 * c + 8 * g);
            }
#pragma unroll
            for (int u = 0; u < U; ++u) wn[u] = load_frag_stream(wp + (int64_t)min(c0 + U + u, last) * 512);
#pragma unroll
            for (int u = 0; u < U; ++u)
                if (c0 + u < c_end) {
#pragma unroll
                    for (int t = 0; t < MT; ++t) acc[t] = El<T>::mma(w[u], xv[u][t], acc[t]);
                }
#pragma unroll
            for (int u = 0; u < U; ++u) w[u] = wn[u];
        }
    }
#pragma unroll
    for (int t = 0; t < MT; ++t) part[wave][t][lane] = acc[t];
    __syncthreads();
    if (wave >= MT) return;                                  // wave t finishes row block t
    const int t = wave;
    f32x4 s = part[0][t][lane];
#pragma unroll
    for (int w = 1; w < WAVES; ++w) {
        const f32x4 o = part[w][t][lane];
#pragma unroll
        for (int r = 0; r < 4; ++r) s[r] += o[r];
    }
    const int m = m0 + 16 * t + i;                           // this lane: outputs n .. n+3 of row m
    const bool live = m < a.rows;
    const int n = 16 * pin + 4 * g;
    if constexpr (EPI == TFL_EPI_IN) {
        if (16 * pin < a.n_raw) {
            float q = s[0] * s[0] + s[1] * s[1] + s[2] * s[2] + s[3] * s[3];
            q += __shfl_xor(q, 16, 64);
            q += __shfl_xor(q, 32, 64);
            if (live) {
                *reinterpret_cast<f32x4*>(a.out_f + (int64_t)m * a.ld_f + n) = s;
                if (g == 0) a.ss_out[(int64_t)m * a.ss_ld + pin] = q;
            }
        } else if (live) {
#pragma unroll
            for (int r = 0; r < 4; ++r) s[r] = gelu_tanh(s[r]);
            store_quad((T*)a.out_t + (int64_t)m * a.ld_t + (n - a.n_raw), s);
        }
        return;
    }
    if (!live) return;
    if constexpr (EPI == TFL_EPI_F32) {
        float* y = a.out_f + (int64_t)m * a.ld_f + n;
#pragma unroll
        for (int r = 0; r < 4; ++r)
            if (n + r < a.n_real) y[r] = s[r];
    } else if constexpr (EPI == TFL_EPI_QUERY) {
        const int per_head = a.N + a.R, h = n / per_head, e = n - h * per_head;
        const int64_t row = (int64_t)m * a.H + h;
        if (e < a.N) {
            store_quad((T*)a.out_t2 + row * a.N + e, s);
        } else {
            const int d = e - a.N;
            int p = a.pos[m];
            p = p < 0 ? 0 : (p >= a.max_pos ? a.max_pos - 1 : p);
#pragma unroll
            for (int r = 0; r < 4; r += 2) {
                const int pr = (d + r) >> 1;
                if (pr < a.half) {
                    const float cs = a.cos[(int64_t)p * a.half + pr], sn = a.sin[(int64_t)p * a.half + pr];
                    const float u = s[r], v = s[r + 1];
                    s[r] = u * cs - v * sn;
                    s[r + 1] = v * cs + u * sn;
                }
            }
            store_quad((T*)a.out_t + row * (a.C + a.R) + a.C + d, s);
        }
    } else if constexpr (EPI == TFL_EPI_LATENT) {
        store_quad((T*)a.out_t + ((int64_t)m * a.H + grp) * (a.C + a.R) + n, s);
    } else if constexpr (EPI == TFL_EPI_GATED) {
        const int col = grp * a.n + n;
        const f32x4 z = *reinterpret_cast<const f32x4*>(a.gate + (int64_t)m * a.ld_gate + col);
#pragma unroll
        for (int r = 0; r < 4; ++r) s[r] *= sigmoid(z[r]);
        store_quad((T*)a.out_t + (int64_t)m * a.ld_t + col, s);
    } else if constexpr (EPI == TFL_EPI_RESIDUAL) {
        f32x4* y = reinterpret_cast<f32x4*>(a.out_f + (int64_t)m * a.ld_f + n);
        f32x4 o = *y;
#pragma unroll
        for (int r = 0; r < 4; ++r) o[r] += s[r];
        *y = o;
    } else if constexpr (EPI == TFL_EPI_TOKEN) {
        int64_t id = a.ids[m];
        id = id < 0 ? 0 : (id >= a.vocab ? a.vocab - 1 : id);
        const T* e = (const T*)a.tok_table + id * a.ld_tok;
#pragma unroll
        for (int r = 0; r < 4; ++r) s[r] = n + r < a.n_real ? gelu_tanh(s[r]) * (float)e[n + r] : 0.f;
        store_quad((T*)a.out_t + (int64_t)m * a.ld_t + n, s);
    }
}

template <typename T, int XMODE, int EPI>
static int launch_gemm(const TflGemm& a, hipStream_t st) {
    const int panels = (a.n >> 4) * a.groups;
    const int mt = a.rows <= 16 ? 1 : 2;
    const int rb = (a.rows + 16 * mt - 1) / (16 * mt);
    int extra = 0;
    if (EPI == TFL_EPI_QUERY && a.kv_raw) extra = (a.rows + rb - 1) / rb;
    const dim3 grid(panels + extra, rb);
    // few panels: more waves per panel keep the weight stream deep enough; the cache-row workgroups are written for 4 waves
    if (EPI == TFL_EPI_QUERY || panels > 1024) {
        if (mt == 1) hipLaunchKernelGGL((latent_gemm_kernel<T, XMODE, EPI, 1, 4>), grid, dim3(256), 0, st, a);
        else hipLaunchKernelGGL((latent_gemm_kernel<T, XMODE, EPI, 2, 4>), grid, dim3(256), 0, st, a);
    } else if (panels > 128) {
        if (mt == 1) hipLaunchKernelGGL((latent_gemm_kernel<T, XMODE, EPI, 1, 8>), grid, dim3(512), 0, st, a);
        else hipLaunchKernelGGL((latent_gemm_kernel<T, XMODE, EPI, 2, 8>), grid, dim3(512), 0, st, a);
    } else {
        if (mt == 1) hipLaunchKernelGGL((latent_gemm_kernel<T, XMODE, EPI, 1, 16>), grid, dim3(1024), 0, st, a);
        else hipLaunchKernelGGL((latent_gemm_kernel<T, XMODE, EPI, 2, 16>), grid, dim3(1024), 0, st, a);
    }
    TFL_LAUNCH_CHECK();
    return TF_OK;
}

template <typename T>
static int dispatch_gemm(const TflGemm& a, int x_mode, int epi, hipStream_t st) {
#define CASE(X, E) if (x_mode == X && epi == E) return launch_gemm<T, X, E>(a, st);
    CASE(TFL_X_T, TFL_EPI_F32)
    CASE(TFL_X_T, TFL_EPI_IN)
    CASE(TFL_X_F32_NORM, TFL_EPI_QUERY)
    CASE(TFL_X_T, TFL_EPI_LATENT)
    CASE(TFL_X_T, TFL_EPI_GATED)
    CASE(TFL_X_T, TFL_EPI_RESIDUAL)
    CASE(TFL_X_F32, TFL_EPI_TOKEN)
#undef CASE
    return TF_EINVAL;
}

extern "C" int tfl_gemm(const TflGemm* p, int dtype, int x_mode, int epi, void* stream) {
    if (!p || !p->wp || !p->x) return TF_EINVAL;
    const TflGemm a = *p;
    if (a.rows < 1 || a.rows > (1 << 20) || a.n < 16 || (a.n & 15) || a.k < 32 || (a.k & 31) || a.groups < 1) return TF_EINVAL;
    if (a.ld_x & 7 || a.x_group & 7) return TF_EINVAL;
    if (dtype != 0 && dtype != 1) return TF_EINVAL;
    switch (epi) {
        case TFL_EPI_F32:
            if (!a.out_f || a.groups != 1 || a.n_real < 1 || a.n_real > a.n || a.ld_f < a.n_real) return TF_EINVAL;
            break;
        case TFL_EPI_IN:
            if (!a.out_f || !a.ss_out || a.groups != 1 || a.n_raw < 16 || (a.n_raw & 15) || a.n_raw > a.n || a.ld_f < a.n_raw
                || (a.ld_f & 3) || a.ss_ld < a.n_raw / 16) return TF_EINVAL;
            if (a.n_raw < a.n && (!a.out_t || (a.ld_t & 3) || a.ld_t < a.n - a.n_raw)) return TF_EINVAL;
            break;
        case TFL_EPI_QUERY:
            if (!a.out_t || !a.out_t2 || !a.pos || a.groups != 1 || a.H < 1 || a.N < 16 || a.R < 0 || a.C < 16) return TF_EINVAL;
            if ((a.N & 15) || (a.R & 15) || (a.C & 15) || a.n != a.H * (a.N + a.R)) return TF_EINVAL;
            if (!a.norm_w || !a.ss_in || a.ss_n < 1 || a.ss_ld < a.ss_n || a.k_real < 1 || a.k_real > a.k) return TF_EINVAL;
            if (a.half < 0 || 2 * a.half > a.R || a.max_pos < 1 || (a.half && (!a.cos || !a.sin))) return TF_EINVAL;
            if (a.kv_raw && (!a.kv_norm_w || !a.cache || !a.slot || a.ld_kv < a.C + a.R || a.c_real < 1 || a.c_real > a.C
                             || a.cache_rows < 1)) return TF_EINVAL;
            break;
        case TFL_EPI_LATENT:
            if (!a.out_t || a.groups != a.H || a.C != a.n || a.R < 0 || (a.R & 3)) return TF_EINVAL;
            break;
        case TFL_EPI_GATED:
            if (!a.out_t || !a.gate || a.ld_t < (int64_t)a.groups * a.n || a.ld_gate < (int64_t)a.groups * a.n || (a.ld_t & 3)
                || (a.ld_gate & 3)) return TF_EINVAL;
            break;
        case TFL_EPI_RESIDUAL:
            if (!a.out_f || a.groups != 1 || a.ld_f < a.n || (a.ld_f & 3)) return TF_EINVAL;
            break;
        case TFL_EPI_TOKEN:
            if (!a.out_t || !a.ids || !a.tok_table || a.groups != 1 || a.n_real < 1 || a.n_real > a.n || a.ld_tok < a.n_real
                || a.ld_t < a.n || (a.ld_t & 3) || a.vocab < 1) return TF_EINVAL;
            break;
        default:
            return TF_EINVAL;
    }
    return dtype == 0 ? dispatch_gemm<bf16>(a, x_mode, epi, (hipStream_t)stream)
                      : dispatch_gemm<float>(a, x_mode, epi, (hipStream_t)stream);
}
