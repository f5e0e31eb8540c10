//! PiralixModel over the model driver of libagpu_hip.so (include/agpu_piralix.h).  The reference has no such model; the
//! calls follow `Int4Gpt2Model`.  The caller fills the configuration structs and hands every tensor over by name.
use std::ffi::CString;
use std::sync::Arc;

use agpu_sys as sys;

use crate::error::Result;
use crate::registry::KernelRegistry;

pub struct PiralixModel {
    reg: Arc<KernelRegistry>,
    handle: *mut sys::agpu_piralix,
    vocab: usize,
}

impl PiralixModel {
    pub fn new(cfg: &sys::agpu_piralix_config, layers: &[sys::agpu_piralix_layer], reg: &Arc<KernelRegistry>) -> Result<Self> {
        assert_eq!(layers.len(), cfg.n_layer as usize);
        let mut handle = std::ptr::null_mut();
        reg.check(unsafe { sys::agpu_piralix_create(reg.raw(), cfg, layers.as_ptr(), &mut handle) })?;
        Ok(PiralixModel { reg: reg.clone(), handle, vocab: cfg.vocab_size as usize })
    }

    /// One weight tensor, bf16 bits in the file's shape (a vector has rows = 1).
    pub fn set_tensor(&self, name: &str, bits: &[u16], rows: i64, cols: i64) -> Result<()> {
        assert_eq!(bits.len() as i64, rows * cols);
        let name = CString::new(name).expect("tensor name");
        self.reg.check(unsafe {
            sys::agpu_piralix_set_tensor(self.handle, name.as_ptr(), bits.as_ptr().cast(), sys::AGPU_DTYPE_BF16, rows, cols)
        })
    }

    pub fn reset_cache(&self) -> Result<()> {
        self.reg.check(unsafe { sys::agpu_piralix_reset_cache(self.handle) })
    }

    pub fn cache_len(&self) -> usize {
        unsafe { sys::agpu_piralix_cache_len(self.handle) as usize }
    }

    pub fn generate_cached(&self, prompt: &[u32], max_new_tokens: usize, eos: Option<u32>) -> Result<Vec<u32>> {
        let mut out = vec![0u32; prompt.len() + max_new_tokens];
        let mut len = 0i32;
        self.reg.check(unsafe {
            sys::agpu_piralix_generate_cached(self.handle, prompt.as_ptr(), 1, prompt.len() as i32, max_new_tokens as i32,
                eos.map_or(-1, |e| e as i32), out.as_mut_ptr(), &mut len, std::ptr::null_mut())
        })?;
        out.truncate(len as usize);
        Ok(out)
    }

    pub fn generate_cached_sampling(&self, prompt: &[u32], max_new_tokens: usize, top_k: usize, temperature: f32, rng_state: &mut u64,
                                    eos: Option<u32>) -> Result<Vec<u32>> {
        let mut out = vec![0u32; prompt.len() + max_new_tokens];
        let mut len = 0i32;
        self.reg.check(unsafe {
            sys::agpu_piralix_generate_cached_sampling(self.handle, prompt.as_ptr(), prompt.len() as i32, max_new_tokens as i32, top_k as i32,
                temperature, rng_state, eos.map_or(-1, |e| e as i32), out.as_mut_ptr(), &mut len)
        })?;
        out.truncate(len as usize);
        Ok(out)
    }

    /// Logits of the last position as the most recent forward or decode step left them.
    pub fn last_logits(&self) -> Result<Vec<f32>> {
        let mut out = vec![0f32; self.vocab];
        self.reg.check(unsafe { sys::agpu_piralix_last_logits(self.handle, 1, out.as_mut_ptr()) })?;
        Ok(out)
    }
}

impl Drop for PiralixModel {
    fn drop(&mut self) {
        unsafe { sys::agpu_piralix_destroy(self.handle) };
    }
}
